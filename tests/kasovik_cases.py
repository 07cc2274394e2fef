"""Small Kasovik configurations for the tests: sizes that are no powers of two and differ from each other, every option on
and off, layers that use another's tensors next to it and far from it.

A: two rotated channels out of five in the retention and values of another size than keys; three query heads a key head and a
   window of 9 in the attention (head size 20: a wavefront a token and head); two value heads a query/key head in the
   recurrence; a parallel layer without a feed-forward that runs twice; one tap (no convolution state) in the last layer.
B: sizes the matrix-unit kernels take; a negative and a unit weight on the two mixers; two taps; the parallel layer first; a
   window of 24 and one of 64.
C: keys of 160 channels in both recurrences, no rotation, a window of a single token, an embedding scale of 1, five taps, an
   attention group of five heads of 96 channels; a chain of three runs of one layer's tensors.
"""
from __future__ import annotations


def _retention(heads, dim, vdim, decay, rot=None):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}
    if rot:
        m["rot"] = {"base": rot[0], "dims": rot[1]}
    return {"type": "retention", "mixer": m}


def _parallel(left, right, left_scale, right_scale):
    return {"type": "parallel", "mixer": {"left": left, "right": right, "left_scale": left_scale, "right_scale": right_scale}}


def _left(heads, kv_heads, dim, window, scale):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "mask": {"size": window}, "scale": scale}


def _right(heads, kv_heads, dim, vdim, conv):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}


def _with(layer, ff=None, limit=None):
    return {**layer, "mlp": {"kind": "dense", "ff": ff, "limit": limit} if ff else None}


def _again(layer, of):
    return {**layer, "weights_of": of}


def _model(vocab, width, eps, scale, pairs, layers):
    return {"architecture": "Kasovik", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "embedding": {"scale": scale, "bigram": {"buckets": pairs[0], "mul_prev": pairs[1], "mul_cur": pairs[2]}}, "layers": layers}


_A0 = _with(_retention(3, 20, 12, [0.9, 0.995, 0.75], rot=(500.0, 8)), 56, 1.2)
_A1 = _with(_parallel(_left(6, 2, 20, 9, 0.8), _right(4, 2, 12, 20, 4), 0.7, 1.3))
_A4 = _with(_parallel(_left(3, 3, 16, 33, 1.1), _right(3, 1, 20, 12, 1), 0.4, 0.9), 30, 0.5)
A = _model(211, 88, 3e-5, 2.5, (37, 19, 3), [_A0, _A1, _again(_A1, 1), _again(_A0, 0), _A4])

_B0 = _with(_parallel(_left(4, 2, 32, 24, 0.6), _right(2, 2, 64, 48, 2), 1.0, -0.6), 96, 7.0)
_B1 = _with(_retention(2, 64, 32, [0.5, 0.998], rot=(2e4, 64)))
_B2 = _with(_parallel(_left(6, 1, 64, 64, 0.3), _right(6, 3, 32, 16, 3), 0.8, 1.4), 64, 1.0)
B = _model(150, 128, 1e-6, 0.7, (64, 150, 1), [_B0, _B1, _B2, _again(_B1, 1), _again(_B0, 0)])

_C0 = _with(_retention(1, 160, 24, [0.97]), 100, 2.0)
_C1 = _with(_parallel(_left(5, 1, 96, 1, 0.5), _right(2, 1, 160, 24, 5), 0.9, 0.9), 44, 0.8)
C = _model(97, 72, 1e-5, 1.0, (11, 5, 2), [_C1, _again(_C1, 0), _C0, _again(_C1, 0)])

CASES = {"A": (A, 41, 0.1, 0.15), "B": (B, 42, 0.08, 0.1), "C": (C, 43, 0.1, 0.2)}      # config, seed, std of matrices, std of norm weights around 1


def lively(cfg, w, seed):
    """The same weights with decays of the recurrence between a few tokens and hundreds, and sinks that count (drawn around
    zero alike they would all forget within a token or two, and all weigh one key)."""
    import torch
    g = torch.Generator().manual_seed(seed)
    out = dict(w)
    for name in sorted(w):
        if name.endswith(".A_log"):
            out[name] = (torch.rand(w[name].shape, generator=g) * 6.0 - 6.0).to(w[name].dtype)
        elif name.endswith(".sink"):
            out[name] = (torch.randn(w[name].shape, generator=g) * 1.5).to(w[name].dtype)
        elif name.endswith(".dt_bias") or name.endswith(".b") and ".mlp." in name:
            out[name] = (torch.randn(w[name].shape, generator=g) * 0.5).to(w[name].dtype)
        elif name.endswith(".conv"):
            out[name] = (torch.randn(w[name].shape, generator=g) * 0.5).to(w[name].dtype)
    return out
