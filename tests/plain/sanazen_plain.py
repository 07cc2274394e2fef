"""A plain, slow implementation of the Sanazen decoder on the CPU, one function per mechanism.

It shares no code with the engine: it reads a config dictionary and a dictionary of tensors and computes with ordinary
tensor expressions. ``dtype`` says what the engine's storage type is; the places where the engine rounds to it are the
places where ``rnd`` is applied here (inputs of matrix products and those of their results that the engine stores, cached
keys and values, each sublayer's result), and everything else is 32-bit.

Notation: x is the 32-bit residual stream [T, W]; a layer is
    x += mixer(unit(x) * w1) + ff(unit(x) * w2)                (without ff where the layer has none)
with unit(v) = v / sqrt(mean(v^2) + eps): two norms of one x, and the sublayers run side by side.
"""
from __future__ import annotations

import torch

WAVE_BASE = 10000.0     # of the position waves: the mechanism's own constant


def rnd(t: torch.Tensor, dtype) -> torch.Tensor:
    return t.to(dtype).float()


def linear(x, w, b=None, dtype=torch.float32):
    y = rnd(x, dtype) @ w.float().T
    if b is not None:
        y = y + b.float()
    return y


def unit(v, eps):
    return v / torch.sqrt((v * v).mean(-1, keepdim=True) + eps)


def rms(v, w, eps):
    return unit(v, eps) * w.float()


def silu(z):
    return z * torch.sigmoid(z)


def position_waves(positions, width):
    """[T, width]: channel 2i is sin(p f_i), channel 2i + 1 is cos(p f_i), f_i = 10000^(-2i / width)."""
    c = torch.arange(width)
    f = (WAVE_BASE ** (-2.0 * (c // 2).double() / width)).float()
    a = positions.float()[:, None] * f[None, :]
    return torch.where(c[None, :] % 2 == 0, a.sin(), a.cos())


def embed(ids, positions, config, t):
    return t["embed"].float()[ids] * float(config["embedding"]["scale"]) + position_waves(positions, int(config["width"]))


def short_conv(z, w):
    """z [T, C], w [C, taps]: out_t = sum_j w[:, j] z_(t - taps + 1 + j), zeros before the first row."""
    taps = w.shape[1]
    padded = torch.cat([torch.zeros(taps - 1, z.shape[1]), z])
    return sum(w[:, j].float() * padded[j:j + z.shape[0]] for j in range(taps))


def visible(T, window, keep):
    """[T, T] of bools: token i sees token j. ``window`` None: every token up to itself; else the ``window`` tokens that end
    with itself, and the first ``keep`` of the sequence."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    seen = j <= i
    if window is not None:
        seen = seen & ((i - j < int(window)) | (j < int(keep or 0)))
    return seen


def kept_window_attention(q, k, v, scale, window=None, keep=0):
    """q [T, H, D], k [T, H, D], v [T, H, Dv] of one sequence (keys already spread over the query heads)."""
    s = (q.transpose(0, 1) @ k.permute(1, 2, 0)) * scale
    p = torch.softmax(s.masked_fill(~visible(q.shape[0], window, keep), float("-inf")), dim=-1)
    return (p @ v.transpose(0, 1)).transpose(0, 1)


def gated_attention(h, m, t, pre, eps, dtype):
    """Biased projections, a short convolution over each, q and k normed over the whole projection, window attention with kept
    first tokens, a gate per channel of the result, a biased output projection."""
    T = h.shape[0]
    H, G, D, Dv = (int(m[n]) for n in ("heads", "kv_heads", "dim", "vdim"))

    def branch(name):
        return short_conv(rnd(linear(h, t[pre + name], t[pre + name + ".b"], dtype), dtype), t[pre + name + ".conv"])

    q = rnd(rms(branch("q"), t[pre + "q.norm"], eps), dtype).view(T, H, D)
    k = rnd(rms(branch("k"), t[pre + "k.norm"], eps), dtype).view(T, G, D)
    v = rnd(branch("v"), dtype).view(T, G, Dv)
    mask = m.get("mask") or {}
    o = kept_window_attention(q, k.repeat_interleave(H // G, 1), v.repeat_interleave(H // G, 1), float(m["scale"]), mask.get("size"),
                              mask.get("keep_first", 0))
    y = o.reshape(T, H * Dv) * torch.sigmoid(rnd(linear(h, t[pre + "g"], dtype=dtype), dtype))
    return rnd(linear(y, t[pre + "o"], t[pre + "o.b"], dtype), dtype)


def decay_scan(q, k, v, decay):
    """S_t = decay S_(t-1) + k_t v_t^T, o_t = S_t^T q_t, head by head, from a zero state. q, k [T, H, D]; v [T, H, Dv];
    decay [H]. Returns o [T, H, Dv]."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1])
    out = []
    for i in range(T):
        S = decay[:, None, None] * S + k[i][:, :, None] * v[i][:, None, :]
        out.append((S * q[i][:, :, None]).sum(1))
    return torch.stack(out)


def lightning(h, m, t, pre, eps, dtype):
    T = h.shape[0]
    H, D, Dv = (int(m[n]) for n in ("heads", "dim", "vdim"))
    q, k, v = (silu(rnd(linear(h, t[pre + n], dtype=dtype), dtype)).view(T, H, d) for n, d in (("q", D), ("k", D), ("v", Dv)))
    o = decay_scan(q, k, v, torch.tensor(m["decay"], dtype=torch.float32)).reshape(T, H * Dv)
    y = rms(o, t[pre + "norm"], eps) * torch.sigmoid(rnd(linear(h, t[pre + "g"], dtype=dtype), dtype))
    return rnd(linear(y, t[pre + "o"], dtype=dtype), dtype)


def mixer(h, m, t, pre, eps, dtype):
    return float(m["left_scale"]) * gated_attention(h, m["left"], t, pre + "left.", eps, dtype) + \
        float(m["right_scale"]) * lightning(h, m["right"], t, pre + "right.", eps, dtype)


def clamped_glu(g, u, limit):
    g, u = g.clamp(max=limit), u.clamp(-limit, limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1.0)


def expert(h, t, pre, limit, dtype, weight=1.0):
    """The expert on weight * h (``weight`` a number, or one per row)."""
    g = linear(h, t[pre + "gate"], dtype=dtype) * weight
    u = linear(h, t[pre + "up"], dtype=dtype) * weight
    return linear(clamped_glu(g, u, float(limit)), t[pre + "down"], dtype=dtype)


def route(h, w_router, top, dtype):
    """(experts [T, top], weights [T, top]): the largest sigmoids, as they are."""
    s = torch.sigmoid(linear(h, w_router, dtype=dtype))
    weights, chosen = s.topk(int(top), dim=-1)
    return chosen, weights


def feed_forward(h, mlp, t, pre, dtype):
    chosen, weights = route(h, t[pre + "router"], mlp["router"]["top"], dtype)
    rows = []
    for i in range(h.shape[0]):
        hi = h[i:i + 1]
        rows.append(sum(expert(hi, t, pre + f"e{int(e)}.", mlp["expert"]["limit"], dtype, w) for e, w in zip(chosen[i], weights[i])))
    y = torch.cat(rows)
    if mlp.get("shared") is not None:
        y = y + torch.sigmoid(linear(h, t[pre + "shared.sg"], dtype=dtype)) * expert(h, t, pre + "shared.", mlp["shared"]["limit"], dtype)
    return rnd(y, dtype)


def logits_of(h, config, t, dtype):
    z = linear(h, t["head"], dtype=dtype) * float(config.get("logit_scale", 1.0))
    cap = config.get("logit_softcap")
    return float(cap) * torch.tanh(z / float(cap)) if cap else z


def forward(ids, config, t, dtype=torch.float32, collect=None):
    """ids [T] of one sequence from its first token on -> float32 logits [T, vocab]; ``collect``: a list that receives the
    residual stream behind every layer."""
    ids = torch.as_tensor(ids, dtype=torch.long)
    eps = float(config["norm"]["eps"])
    x = embed(ids, torch.arange(len(ids)), config, t)
    for i, layer in enumerate(config["layers"]):
        p = f"l{i}."
        add = mixer(rnd(rms(x, t[p + "norm1"], eps), dtype), layer["mixer"], t, p + "mix.", eps, dtype)
        if layer.get("mlp") is not None:
            add = add + feed_forward(rnd(rms(x, t[p + "norm2"], eps), dtype), layer["mlp"], t, p + "mlp.", dtype)
        x = x + add
        if collect is not None:
            collect.append(x.clone())
    return logits_of(rms(x, t["final.norm"], eps), config, t, dtype)
