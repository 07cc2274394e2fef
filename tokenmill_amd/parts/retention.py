"""Retention: a recurrent mixer with a matrix of state per request and head and one fixed decay per head.

    q_t, k_t = rotate(W_q h_t), rotate(W_k h_t) / sqrt(D)     [heads, D]
    v_t, g_t = W_v h_t, W_g h_t                               [heads, Dv]
    S_t = decay_h S_(t-1) + k_t v_t^T                         [D, Dv] per head, 32-bit, zero at a request's first token
    o_t = S_t^T q_t
    y_t = W_o (concat over heads of unit_rms(o_t) * silu(g_t))

What another model may ask for, each a constructor parameter: q, k and v that are silu of their projection (``silu``); another
scale of k (``k_scale``); one norm over the heads side by side with a weight per channel in place of a norm per head
(``whole_norm``); a sigmoid gate (``sigmoid_gate``).

with the rotation of ``rotary`` (by the token's position, over the first channels of a head) or none. The state is the mixer's
cache: a ``StateSpec`` slot per request, advanced in token order inside a step's portion and carried from step to step. What
lies between the projections and the norm of the result is 32-bit. It is gated linear attention with decays that do not
change from token to token, and runs that recurrence's kernels. A step of single tokens works on the step's device tensors
alone, so it can be recorded into a HIP graph.
"""
from __future__ import annotations

import torch

from tokenmill_amd import profiling
from tokenmill_amd.hip import ops
from tokenmill_amd.parts.base import Mixer, StateSpec, StateView, StepContext, as_tensor, step_segments
from tokenmill_amd.parts.gla import MAX_KEY_DIM
from tokenmill_amd.parts.linear import Linear
from tokenmill_amd.parts.position import RotaryEmbedding
from tokenmill_amd.weights.loader import TensorSpec


class Retention(Mixer):
    def __init__(self, hidden: int, num_heads: int, key_dim: int, value_dim: int, decay: list[float], norm_eps: float,
                 rotary: RotaryEmbedding | None = None, names: tuple[str, ...] = ("q", "k", "v", "g", "o"),
                 suffixes: tuple[str, str] = ("", ".b"), silu: bool = False, k_scale: float | None = None, whole_norm: bool = False,
                 sigmoid_gate: bool = False, norm_name: str = "norm"):
        """``k_scale``: None for 1 / sqrt(key size)."""
        if not 0 < key_dim <= MAX_KEY_DIM or value_dim <= 0:
            raise ValueError(f"key size {key_dim}: the recurrence kernel takes up to {MAX_KEY_DIM}")
        if len(decay) != num_heads:
            raise ValueError(f"{len(decay)} decays for {num_heads} heads")
        if rotary is not None and (rotary.interleaved or rotary.rotary_dim > key_dim):
            raise ValueError("a retention rotates pairs half the rotated width apart, inside a head")
        self.hidden, self.num_heads, self.key_dim, self.value_dim = hidden, num_heads, key_dim, value_dim
        self.norm_eps, self.rotary, self.decay_values = float(norm_eps), rotary, [float(d) for d in decay]
        self.silu, self.k_scale, self.whole_norm, self.sigmoid_gate = silu, float(k_scale) if k_scale is not None else key_dim ** -0.5, whole_norm, sigmoid_gate
        self.norm_name = norm_name
        self.norm_w: torch.Tensor | None = None         # float32 [H * Dv] with a norm over all heads
        self.k_size, self.v_size = num_heads * key_dim, num_heads * value_dim
        self.proj = Linear(hidden, [self.k_size, self.k_size, self.v_size, self.v_size], list(names[:4]), bias=False, suffixes=suffixes)
        self.o = Linear(self.v_size, hidden, names[4], bias=False, suffixes=suffixes)
        self.decay: torch.Tensor | None = None          # float32 [1, H * D]: every token's

    def tensor_specs(self, prefix: str):
        specs = {**self.proj.tensor_specs(prefix), **self.o.tensor_specs(prefix)}
        if self.whole_norm:
            specs[prefix + self.norm_name] = TensorSpec((self.v_size,), init="ones")
        return specs

    def load(self, tensors, prefix: str) -> None:
        self.proj.load(tensors, prefix)
        self.o.load(tensors, prefix)
        if self.rotary is not None:
            self.rotary.load(tensors, prefix)
        if self.whole_norm:
            self.norm_w = tensors[prefix + self.norm_name].float().contiguous()
        per_head = torch.tensor(self.decay_values, dtype=torch.float32)
        self.decay = per_head.repeat_interleave(self.key_dim)[None].contiguous().to(self.o.weight.device)

    def prepare(self, pack_weights: bool) -> None:
        self.proj.prepare(pack_weights)
        self.o.prepare(pack_weights)

    def cache_spec(self):
        return StateSpec((self.num_heads, self.key_dim, self.value_dim), torch.float32)

    def cost(self, label: str, step: StepContext | None, rows: int) -> tuple[int, int]:
        if label == "qkv":
            return self.proj.cost(rows)
        if label == "o_proj":
            return self.o.cost(rows)
        # the recurrence: q, k, v and the result once; the state read and written once per request; per token and head
        # D * Dv multiply-adds for the state and as many for the result
        e = self.proj.weight.element_size()
        seqs = step.num_seqs if step is not None else 1
        moved = rows * ((2 * self.k_size + self.v_size) * e + self.v_size * 4) + 2 * seqs * self.num_heads * self.key_dim * self.value_dim * 4
        return moved, 4 * rows * self.num_heads * self.key_dim * self.value_dim

    # Rows of a request's portion from which the recurrence runs in chunks on the matrix unit, or (keys it does not take) in
    # segments of this many rows (see ``_scan``)
    CHUNKS_FROM = 32
    SEGMENT = 64

    def forward(self, x, step: StepContext, cache: StateView, residual: torch.Tensor | None = None):
        x = as_tensor(x)
        T = x.shape[0]
        H, D, Dv, rot = self.num_heads, self.key_dim, self.value_dim, self.rotary
        if rot is not None and step.max_context_len > rot.max_positions:
            raise ValueError(f"position {step.max_context_len - 1} is beyond the rotary table ({rot.max_positions} positions)")
        with profiling.label("qkv", lambda: self.cost("qkv", step, T)):
            proj = self.proj.forward(x)                                          # [T, q | k | v | g]
        y = torch.empty((T, self.v_size), dtype=x.dtype, device=x.device)
        cos, sin = (rot.cos, rot.sin) if rot is not None else (None, None)
        # the step's single tokens (its last rows and requests) go through one kernel from here to y, where it takes the sizes
        singles = step.num_decode if ops.retention_step_takes(D, Dv) and (self.whole_norm or not self.sigmoid_gate) else 0
        P, Tp = step.num_seqs - singles, T - singles
        with profiling.label("recurrence", lambda: self.cost("attention", step, T)):
            o = torch.empty((T if self.whole_norm else Tp, self.v_size), dtype=torch.float32, device=x.device)
            if Tp:
                rows = torch.empty((Tp, ops.retention_row_width(H, D, Dv)), dtype=torch.float32, device=x.device)
                ops.retention_prepare(proj[:Tp], cos, sin, step.positions, rows, H, D, Dv, self.k_scale, silu=self.silu)
                self._scan(rows, o[:Tp], cache.state, step, P)
                if not self.whole_norm:
                    ops.gla_out_gate(o, proj[:Tp, 2 * self.k_size + self.v_size:], None, y[:Tp], H, Dv, self.norm_eps, sigmoid=self.sigmoid_gate)
            if singles and self.whole_norm:
                ops.retention_step(proj[Tp:], cos, sin, step.positions[Tp:], self.decay, cache.state, step.state_slots[P:], None, H, D, Dv,
                                   self.k_scale, self.norm_eps, silu=self.silu, o=o[Tp:])
            elif singles:
                ops.retention_step(proj[Tp:], cos, sin, step.positions[Tp:], self.decay, cache.state, step.state_slots[P:], y[Tp:], H, D, Dv,
                                   self.k_scale, self.norm_eps, silu=self.silu)
            if self.whole_norm:                     # the heads side by side as one
                ops.gla_out_gate(o, proj[:, 2 * self.k_size + self.v_size:], self.norm_w, y, 1, self.v_size, self.norm_eps, sigmoid=self.sigmoid_gate)
        with profiling.label("o_proj", lambda: self.o.cost(T)):
            return self.o.forward(y)

    def _scan(self, rows, o, state, step: StepContext, num_seqs: int) -> None:
        """The recurrence over the rows of the step's first ``num_seqs`` requests: one scan from the requests' states; for longer portions chunks of 64 rows as
        products of small matrices (``ops.retention_chunk_scan``), with a scan of single tokens among the requests beside them; or, with
        keys of more channels than that takes, (as in gated linear attention) two scans of a portion's segments side by side with a
        chain of the segments' states between them."""
        H, D, Dv, ks = self.num_heads, self.key_dim, self.value_dim, self.k_size
        if step.max_q_len >= self.CHUNKS_FROM and D <= ops.CHUNK_MAX_KEY_DIM:
            cu_chunk, _, first, n = step_segments(step, ops.CHUNK, rows.device, portions_only=True)
            portions = step.num_seqs - step.num_decode
            ops.retention_chunk_scan(rows, self.decay, o, state, cu_chunk, first, n, step.state_slots, portions, H, D, Dv)
            if num_seqs > portions:
                ops.gla_scan(rows, 0, ks, 2 * ks, self.decay, o, state, step.cu_q_lens[portions:], step.state_slots[portions:],
                             num_seqs - portions, H, D, Dv, 1.0)
            return
        if step.max_q_len < 2 * self.SEGMENT:
            ops.gla_scan(rows, 0, ks, 2 * ks, self.decay, o, state, step.cu_q_lens, step.state_slots, num_seqs, H, D, Dv, 1.0)
            return
        cu_seg, ids, first, n_seg = step_segments(step, self.SEGMENT, rows.device, portions_only=num_seqs < step.num_seqs)
        local = torch.zeros((n_seg, H, D, Dv), dtype=torch.float32, device=rows.device)
        states_only = ops.gla_scan_states_only(rows, 0, ks, self.decay, D)       # else o is written and overwritten below
        ops.gla_scan(rows, 0, ks, 2 * ks, self.decay, None if states_only else o, local, cu_seg, ids, n_seg, H, D, Dv, 1.0)
        products = torch.empty((n_seg, ks), dtype=torch.float32, device=rows.device)
        ops.gla_segment_decay(self.decay, cu_seg, n_seg, products)
        start = torch.empty_like(local)
        ops.gla_combine(state, step.state_slots, first, products, local, start, num_seqs)
        ops.gla_scan(rows, 0, ks, 2 * ks, self.decay, o, start, cu_seg, ids, n_seg, H, D, Dv, 1.0)
