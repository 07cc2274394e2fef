"""Small Sanazen configurations for the tests: sizes that are no powers of two and differ from each other, every option on and off.

A: values of another size than keys (a wavefront a token and head), three query heads a key head, a window of 9 beside 3 kept tokens;
   a layer without a feed-forward; keys and values of one size on the 32-bit matrix unit with one tap (no convolution state) and kept
   tokens over a page border; three of seven experts.
B: sizes the matrix-unit kernels take; a negative and a unit weight on the two mixers; windows of 24 and 64 beside 5 and 18 kept
   tokens; two and three taps; values of the recurrence wider than a wavefront's columns; no cap, all experts at once, no shared
   expert in one layer.
C: keys of 160 channels in the recurrence, no window at all in one layer and a window of a single token in another (beside more kept
   tokens than the window holds), an embedding scale of 1, five taps, an attention group of five heads of 96 channels, one expert a
   token.
"""
from __future__ import annotations


def _layer(left, right, left_scale, right_scale, mlp=None):
    return {"type": "parallel", "mixer": {"left": left, "right": right, "left_scale": left_scale, "right_scale": right_scale}, "mlp": mlp}


def _left(heads, kv_heads, dim, vdim, conv, scale, window=None, keep=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv, "scale": scale}
    if window is not None:
        m["mask"] = {"size": window, "keep_first": keep}
    return m


def _right(heads, dim, vdim, decay):
    return {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}


def _moe(ff, limit, experts, top, shared=None):
    m = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}
    if shared:
        m["shared"] = {"ff": shared[0], "limit": shared[1]}
    return m


def _model(vocab, width, eps, scale, layers, logit_scale, cap):
    c = {"architecture": "Sanazen", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
         "logit_scale": logit_scale, "layers": layers}
    if cap:
        c["logit_softcap"] = cap
    return c


A = _model(211, 88, 3e-5, 2.5, [
    _layer(_left(6, 2, 20, 12, 4, 0.3, 9, 3), _right(3, 20, 12, [0.9, 0.995, 0.75]), 0.7, 1.3, _moe(28, 1.2, 7, 3, (20, 0.8))),
    _layer(_left(3, 3, 16, 16, 1, 0.4, 33, 20), _right(2, 12, 30, [0.5, 0.99]), 0.4, 0.9),
    _layer(_left(4, 1, 24, 40, 3, 0.25, 17, 1), _right(1, 36, 20, [0.97]), 1.1, 0.6, _moe(12, 0.5, 3, 1, (36, 2.0))),
], 0.7, 5.0)

B = _model(150, 128, 1e-6, 0.7, [
    _layer(_left(4, 2, 32, 32, 2, 0.3, 24, 5), _right(2, 64, 48, [0.5, 0.998]), 1.0, -0.6, _moe(48, 7.0, 4, 4, (32, 1.0))),
    _layer(_left(6, 1, 64, 64, 3, 0.15, 64, 18), _right(2, 32, 160, [0.96, 0.8]), 0.8, 1.0, _moe(24, 1.0, 5, 2)),
], 1.0, None)

C = _model(97, 72, 1e-5, 1.0, [
    _layer(_left(5, 1, 96, 96, 5, 0.12), _right(1, 160, 24, [0.97]), 0.9, 0.9, _moe(20, 2.0, 6, 1, (8, 0.7))),
    _layer(_left(2, 2, 32, 32, 4, 0.2, 1, 35), _right(2, 16, 16, [1.0, 0.6]), 0.5, 1.5),
], 2.5, 30.0)

CASES = {"A": (A, 51, 0.1, 0.15), "B": (B, 52, 0.08, 0.1), "C": (C, 53, 0.1, 0.2)}      # config, seed, std of matrices, std of norm weights around 1


def lively(cfg, w, seed):
    """The same weights with convolutions and biases that count, and routers whose choice hangs on no close call: hidden channel 2 of
    every embedding row is a constant of one sign or the other, and a router output follows that channel with a slope of its own
    (descending for one sign, ascending for the other), so that two sets of experts are in use."""
    import torch
    g = torch.Generator().manual_seed(seed)
    out = dict(w)
    for name in sorted(w):
        shape, dt = w[name].shape, w[name].dtype
        if name.endswith(".conv"):
            out[name] = (torch.randn(shape, generator=g) * 0.5).to(dt)
        elif name.endswith(".b"):
            out[name] = (torch.randn(shape, generator=g) * 0.5).to(dt)
        elif name.endswith(".router"):
            E = shape[0]
            z = torch.randn(shape, generator=g) * 0.004
            z[:, 2] = (torch.arange(E).float() - (E - 1) / 2)[torch.randperm(E, generator=g)] * (2.0 / max(E - 1, 1)) if E > 1 else 0.5
            out[name] = z.to(dt)
    emb = w["embed"].float().clone()
    sign = torch.where(torch.rand(emb.shape[0], generator=g) < 0.5, -1.0, 1.0)
    emb[:, 2] = sign * 3.0 / float(cfg["embedding"]["scale"])
    out["embed"] = emb.to(w["embed"].dtype)
    return out
