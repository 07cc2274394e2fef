"""Token embedding and output head (reference src/infer/model/qwen2.py:30-33,39-52)."""
from __future__ import annotations

import torch

from tokenmill_amd import profiling
from tokenmill_amd.hip import ops
from tokenmill_amd.parts.base import Part, StateSpec, StateView, StepContext
from tokenmill_amd.parts.linear import Linear
from tokenmill_amd.weights.loader import TensorSpec


class LearnedPositions(Part):
    """A table with one learned row per position, added (unscaled) to the token's embedding row."""

    def __init__(self, max_positions: int, hidden: int, name: str = "weight"):
        self.max_positions, self.hidden, self.name = max_positions, hidden, name
        self.weight: torch.Tensor | None = None

    def tensor_specs(self, prefix: str):
        return {f"{prefix}{self.name}": TensorSpec((self.max_positions, self.hidden))}

    def load(self, tensors, prefix: str) -> None:
        self.weight = tensors[f"{prefix}{self.name}"]


class PositionWaves(Part):
    """Waves of the token's position, added (unscaled) to its embedding row: channel 2i is sin(p f_i), channel 2i + 1 is cos(p f_i),
    f_i = base^(-2i / width). The frequencies are computed in 64-bit and rounded once; angles and waves are 32-bit, made by the
    embedding's kernel. Nothing bounds a position."""

    def __init__(self, hidden: int, base: float = 10000.0):
        self.hidden, self.base = hidden, float(base)
        self.frequencies: torch.Tensor | None = None

    def load(self, tensors, prefix: str) -> None:
        i = torch.arange((self.hidden + 1) // 2, dtype=torch.float64)
        self.frequencies = (self.base ** (-2.0 * i / self.hidden)).float().to(next(iter(tensors.values())).device)


class PairRows(Part):
    """A table with a row per bucket of token pairs, added (unscaled) to a token's embedding row: bucket
    (previous token * mul_prev + token * mul_cur) mod buckets, and one row more, the last, for a request's first token. The
    previous token is per-request state: one int32 a request, carried from step to step."""

    def __init__(self, buckets: int, hidden: int, mul_prev: int, mul_cur: int, name: str = "weight"):
        if buckets < 1:
            raise ValueError("a table of token pairs has at least one bucket")
        self.buckets, self.hidden, self.mul_prev, self.mul_cur, self.name = buckets, hidden, int(mul_prev), int(mul_cur), name
        self.weight: torch.Tensor | None = None

    def tensor_specs(self, prefix: str):
        return {f"{prefix}{self.name}": TensorSpec((self.buckets + 1, self.hidden))}

    def load(self, tensors, prefix: str) -> None:
        self.weight = tensors[f"{prefix}{self.name}"]

    def state_spec(self) -> StateSpec:
        return StateSpec((1,), torch.int32)


class TokenEmbedding(Part):
    """x = E[ids] * scale (``scale`` 1 unless the model says otherwise); rows are widened into the 32-bit residual stream.
    With ``places`` (a ``LearnedPositions``) the row of the token's position is added, with ``pairs`` (a ``PairRows``) the
    row of the token and the one before it, with ``waves`` (a ``PositionWaves``) the waves of its position, in 32-bit."""

    def __init__(self, vocab: int, hidden: int, name: str = "weight", places: LearnedPositions | None = None, scale: float = 1.0,
                 pairs: PairRows | None = None, waves: PositionWaves | None = None):
        if places is not None and (scale != 1.0 or pairs is not None):
            raise ValueError("an embedding with position rows has no scale and no rows of pairs")
        self.vocab, self.hidden, self.name, self.places, self.scale = vocab, hidden, name, places, float(scale)
        if waves is not None and (places is not None or pairs is not None):
            raise ValueError("an embedding with waves of the position adds nothing else")
        self.pairs, self.waves = pairs, waves
        self.weight: torch.Tensor | None = None

    @property
    def by_position(self) -> bool:
        """Does ``forward`` need the tokens' positions beside their ids?"""
        return self.places is not None or self.waves is not None

    def cache_spec(self) -> StateSpec | None:
        """State the embedding keeps per request (the token before), or None."""
        return self.pairs.state_spec() if self.pairs is not None else None

    def _tables(self):
        return [p for p in (self.places, self.pairs, self.waves) if p is not None]

    def tensor_specs(self, prefix: str):
        specs = {f"{prefix}{self.name}": TensorSpec((self.vocab, self.hidden))}
        for part in self._tables():
            specs.update(part.tensor_specs(prefix))
        return specs

    def load(self, tensors, prefix: str) -> None:
        self.weight = tensors[f"{prefix}{self.name}"]
        for part in self._tables():
            part.load(tensors, prefix)

    def emit(self, program) -> int | None:
        if self._tables() or self.scale != 1.0:
            return None                         # the library's operation gathers token rows only, as they are
        return program.embedding(self, self.weight)

    def cost(self, label, step, rows):
        rows_read = 1 + len(self._tables()) - (1 if self.waves is not None else 0)
        return rows * self.hidden * (self.weight.element_size() * rows_read + 4), 0

    def forward(self, token_ids: torch.Tensor, positions: torch.Tensor | None = None) -> torch.Tensor:
        out = torch.empty((token_ids.numel(), self.hidden), dtype=torch.float32, device=token_ids.device)
        with profiling.label("embed", lambda: self.cost("embed", None, token_ids.numel())):
            if self.places is not None:
                return ops.embed_gather_pos(self.weight, self.places.weight, token_ids, positions, out)
            if self.waves is not None:
                return ops.embed_waves(self.weight, token_ids, positions, self.waves.frequencies, out, self.scale)
            return ops.embed_gather(self.weight, token_ids, out, self.scale)

    def forward_step(self, step: StepContext, cache: StateView) -> torch.Tensor:
        """The rows of an embedding that keeps state, for a step's tokens; the state moves on to the step's last tokens."""
        pairs = self.pairs
        out = torch.empty((step.num_tokens, self.hidden), dtype=torch.float32, device=step.token_ids.device)
        with profiling.label("embed", lambda: self.cost("embed", None, step.num_tokens)):
            return ops.embed_pairs(self.weight, pairs.weight, step.token_ids, step.positions, step.cu_q_lens, step.state_slots,
                                   step.seq_of_token, step.num_seqs, cache.state, out, self.scale, pairs.mul_prev, pairs.mul_cur)


class OutputHead(Part):
    """logits = h W^T in 32-bit, W the embedding table itself when tied (no second copy); then times ``scale``, and with ``cap`` capped
    smoothly: cap * tanh(logits / cap)."""

    def __init__(self, hidden: int, vocab: int, tied_to: TokenEmbedding | None, name: str = "lm_head",
                 suffixes: tuple[str, str] = (".weight", ".bias"), scale: float = 1.0, cap: float | None = None):
        if cap is not None and not cap > 0:
            raise ValueError("a cap of the logits is positive")
        self.hidden, self.vocab, self.tied_to, self.scale, self.cap = hidden, vocab, tied_to, float(scale), cap
        self.proj = Linear(hidden, vocab, name, bias=False, library_first=True, suffixes=suffixes)

    def tensor_specs(self, prefix: str):
        return {} if self.tied_to is not None else self.proj.tensor_specs(prefix)

    def load(self, tensors, prefix: str) -> None:
        if self.tied_to is not None:
            self.proj.use_weight(self.tied_to.weight)
        else:
            self.proj.load(tensors, prefix)

    def emit(self, program, norm) -> int | None:
        """logits = proj(norm(resid[logit rows])): the final norm and this head as one operation."""
        if self.scale != 1.0 or self.cap is not None:
            return None                         # the library's operation ends at the product
        return program.head(self, norm, self.proj, self.vocab)

    def cost(self, label, step, rows):
        n = step.num_logit_rows if step is not None else rows
        if label == "norm":
            e = self.proj.weight.element_size()
            return n * self.hidden * (4 + e), 0
        return self.proj.cost(n, out_bytes=4)

    def forward(self, h: torch.Tensor) -> torch.Tensor:
        with profiling.label("head", lambda: self.proj.cost(h.shape[0], out_bytes=4)):
            logits = self.proj.forward(h, out_dtype=torch.float32)
            if self.scale != 1.0 or self.cap is not None:
                ops.scale_cap(logits, self.scale, self.cap or 0.0)
            return logits
