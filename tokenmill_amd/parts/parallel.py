"""Two mixers side by side: both read the same input. Either each result is RMS-normed over the model's width with a weight
of its own, and the mixer's result is half their sum,

    y = (rms_norm(left(h); w_left) + rms_norm(right(h); w_right)) / 2,

or the results are added with two constant weights (``scales``),

    y = scale_left * left(h) + scale_right * right(h),

which a block that takes several results at once (``forward_parts``) adds into the residual stream in 32-bit.

The two may be any mixers of which at most one keeps pages (an attention beside a recurrence); each may keep state slots. The
layer's cache is then those pages with the states of the left and then of the right mixer beside them.
"""
from __future__ import annotations

import torch

from tokenmill_amd import profiling
from tokenmill_amd.hip import ops
from tokenmill_amd.parts.base import KVCacheSpec, KVCacheView, LayerCacheSpec, Mixer, StateSpec, StateView, StepContext, as_tensor
from tokenmill_amd.weights.loader import TensorSpec


def _split(spec):
    """(pages, states) that a mixer's cache spec asks for."""
    if spec is None:
        return None, None
    if isinstance(spec, KVCacheSpec):
        return spec, None
    if isinstance(spec, StateSpec):
        return None, spec
    return spec.kv, spec.state


class ParallelMixer(Mixer):
    def __init__(self, hidden: int, left: Mixer, right: Mixer, norm_eps: float | None = None,
                 prefixes: tuple[str, str] = ("left.", "right."), norm_names: tuple[str, str] = ("left.out", "right.out"),
                 scales: tuple[float, float] | None = None):
        if (norm_eps is None) == (scales is None):
            raise ValueError("the two results are either normed or weighted by constants")
        self.hidden, self.left, self.right = hidden, left, right
        self.norm_eps = float(norm_eps) if norm_eps is not None else None
        self.scales = (float(scales[0]), float(scales[1])) if scales is not None else None
        self.prefixes, self.norm_names = prefixes, norm_names if scales is None else ()
        (lk, ls), (rk, rs) = _split(left.cache_spec()), _split(right.cache_spec())
        if lk is not None and rk is not None:
            raise ValueError("of two mixers side by side, one may keep pages")
        self.pages_of = 0 if lk is not None else 1 if rk is not None else None
        self.state_of = 0 if ls is not None else 1 if rs is not None else None
        # with state on both sides the layer holds a tuple: the left mixer's, then the right one's
        self.states_of = tuple(len(s) if isinstance(s, tuple) else 1 for s in (ls, rs)) if ls is not None and rs is not None else None
        self._single = (not isinstance(ls, tuple), not isinstance(rs, tuple))
        states = ls if ls is not None else rs
        if self.states_of is not None:
            states = tuple(s for side in (ls, rs) for s in (side if isinstance(side, tuple) else (side,)))
        self._spec = LayerCacheSpec(lk or rk, states) if (self.pages_of is not None or self.state_of is not None) else None
        self.w_left: torch.Tensor | None = None
        self.w_right: torch.Tensor | None = None

    @property
    def capturable(self) -> bool:
        return self.left.capturable and self.right.capturable

    def tensor_specs(self, prefix: str):
        specs = {**self.left.tensor_specs(prefix + self.prefixes[0]), **self.right.tensor_specs(prefix + self.prefixes[1])}
        for name in self.norm_names:
            specs[prefix + name] = TensorSpec((self.hidden,), init="ones")
        return specs

    def load(self, tensors, prefix: str) -> None:
        self.left.load(tensors, prefix + self.prefixes[0])
        self.right.load(tensors, prefix + self.prefixes[1])
        if self.scales is None:
            self.w_left = tensors[prefix + self.norm_names[0]].float().contiguous()
            self.w_right = tensors[prefix + self.norm_names[1]].float().contiguous()

    def prepare(self, pack_weights: bool) -> None:
        self.left.prepare(pack_weights)
        self.right.prepare(pack_weights)

    def cache_spec(self):
        return self._spec

    def _cache_for(self, which: int, cache):
        """What mixer ``which`` is handed of the layer's cache: the pages, the state, or nothing."""
        if cache is None:
            return None
        if self.states_of is not None:
            n = self.states_of[0]
            mine = cache.state[:n] if which == 0 else cache.state[n:]
            mine = mine[0] if self._single[which] else mine
            if isinstance(cache, KVCacheView) and which == self.pages_of:
                return KVCacheView(cache.k, cache.v, cache.group, cache.write, mine)
            return StateView(mine)
        if isinstance(cache, KVCacheView):
            if which == self.pages_of:
                return cache
            return StateView(cache.state) if which == self.state_of and cache.state is not None else None
        return cache if which == self.state_of else None

    def _both(self, x: torch.Tensor, step: StepContext, cache):
        return self.left.forward(x, step, self._cache_for(0, cache)), self.right.forward(x, step, self._cache_for(1, cache))

    def forward_parts(self, x, step: StepContext, cache) -> list:
        """[(result [T, hidden], its weight), ...]: what is to be added into the residual stream."""
        if self.scales is None:
            return [(self.forward(x, step, cache), 1.0)]
        a, b = self._both(as_tensor(x), step, cache)
        return [(a, self.scales[0]), (b, self.scales[1])]

    def forward(self, x, step: StepContext, cache, residual: torch.Tensor | None = None):
        if self.scales is not None:
            from tokenmill_amd.parts.norm import WeightedAdd
            (a, s), other = self.forward_parts(x, step, cache)
            total = torch.zeros(a.shape, dtype=torch.float32, device=a.device)
            WeightedAdd(s, [other]).add_normed(total, a)
            return total if a.dtype == torch.float32 else ops.convert(total, torch.empty_like(a))
        a, b = self._both(as_tensor(x), step, cache)
        out = torch.empty_like(a)
        with profiling.label("norm", lambda: (3 * a.numel() * a.element_size(), 0)):
            return ops.pair_norm_mean(a, b, self.w_left, self.w_right, out, self.norm_eps)
