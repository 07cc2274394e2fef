"""A plain, slow implementation of the Kasovik decoder on the CPU, one function per mechanism.

It shares no code with the engine: it reads a config dictionary and a dictionary of tensors and computes with ordinary
tensor expressions. ``dtype`` says what the engine's storage type is; the places where the engine rounds to it are the
places where ``rnd`` is applied here (inputs of matrix products and those of their results that the engine stores, cached
keys and values, each sublayer's result), and everything else is 32-bit.

Notation: x is the 32-bit residual stream [T, W]; a layer is
    h = unit(x) * w;   x += mixer(h) + ff(h)                   (without ff where the layer has none)
with unit(v) = v / sqrt(mean(v^2) + eps): one norm, and both sublayers read its result.
"""
from __future__ import annotations

import math

import torch
import torch.nn.functional as F


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


def embed(ids, config, t):
    """ids [T], a sequence from its first token on: the token's row times a constant plus a row that the token and the one
    before it choose together (the table's last row for the first token)."""
    e = config["embedding"]
    big = e["bigram"]
    table = t["bigram"].float()
    rows = [int(big["buckets"])]
    for prev, cur in zip(ids[:-1].tolist(), ids[1:].tolist()):
        rows.append((prev * int(big["mul_prev"]) + cur * int(big["mul_cur"])) % int(big["buckets"]))
    return t["embed"].float()[ids] * float(e["scale"]) + table[torch.tensor(rows)]


def frequencies(rot: dict):
    """f [dims/2]: pair i turns by p * f[i] at position p."""
    dims, base = int(rot["dims"]), float(rot["base"])
    i = torch.arange(dims // 2, dtype=torch.float64)
    return (base ** (-2.0 * i / dims)).float()


def rotate_half(v, positions, rot: dict | None):
    """v [T, heads, D]: of every head's first rot.dims channels, channel i and channel i + dims/2 turn as a pair."""
    dims = int(rot["dims"]) if rot else 0
    if dims == 0:
        return v
    a = positions.float()[:, None] * frequencies(rot)[None, :]
    c, s = a.cos()[:, None, :], a.sin()[:, None, :]
    h = dims // 2
    x, y = v[..., :h], v[..., h:dims]
    out = v.clone()
    out[..., :h] = x * c - y * s
    out[..., h:dims] = y * c + x * s
    return out


def retention_scan(q, k, v, decay):
    """S_t = decay S_(t-1) + k_t v_t^T, o_t = S_t^T q_t, head by head, from a zero state. q, k [T, H, D]; v [T, H, Dv];
    decay [H]. Returns o [T, H, Dv]."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1])
    out = []
    for i in range(T):
        S = decay[:, None, None] * S + k[i][:, :, None] * v[i][:, None, :]
        out.append((S * q[i][:, :, None]).sum(1))
    return torch.stack(out)


def retention(h, m, t, pre, eps, positions, dtype):
    T = h.shape[0]
    H, D, Dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q = rotate_half(rnd(linear(h, t[pre + "q"], dtype=dtype), dtype).view(T, H, D), positions, m.get("rot"))
    k = rotate_half(rnd(linear(h, t[pre + "k"], dtype=dtype), dtype).view(T, H, D), positions, m.get("rot")) * D ** -0.5
    v = rnd(linear(h, t[pre + "v"], dtype=dtype), dtype).view(T, H, Dv)
    o = unit(retention_scan(q, k, v, torch.tensor(m["decay"], dtype=torch.float32)), eps)
    y = o.reshape(T, H * Dv) * silu(rnd(linear(h, t[pre + "g"], dtype=dtype), dtype))
    return rnd(linear(y, t[pre + "o"], dtype=dtype), dtype)


def window_attention(q, k, v, scale, window, sink):
    """q [T, H, D], k [T, H, D], v [T, H, Dv] of one sequence (keys already spread over the query heads). Token i sees the
    ``window`` tokens that end with itself (None: every token up to itself). ``sink`` [H]: one more term exp(sink) in each
    row's denominator, with no key and no value."""
    T = q.shape[0]
    i = torch.arange(T)
    back = i[:, None] - i[None, :]
    seen = back >= 0 if window is None else (back >= 0) & (back < window)
    s = (q.transpose(0, 1) @ k.permute(1, 2, 0)) * scale
    s = s.masked_fill(~seen, float("-inf"))
    z = sink.float()[:, None, None].expand(-1, T, 1)
    p = torch.softmax(torch.cat([s, z], dim=-1), dim=-1)[..., :T]
    return (p @ v.transpose(0, 1)).transpose(0, 1)


def key_value_attention(h, m, t, pre, eps, dtype):
    """The values are the projected keys; queries and keys (not values) are unit-RMS per head; no positions."""
    T = h.shape[0]
    H, G, D = int(m["heads"]), int(m["kv_heads"]), int(m["dim"])
    q = rnd(unit(linear(h, t[pre + "q"], dtype=dtype).view(T, H, D), eps), dtype)
    raw = linear(h, t[pre + "k"], dtype=dtype).view(T, G, D)
    k, v = rnd(unit(raw, eps), dtype), rnd(raw, dtype)
    each = H // G
    window = (m.get("mask") or {}).get("size")
    o = window_attention(q, k.repeat_interleave(each, 1), v.repeat_interleave(each, 1), float(m["scale"]), window, t[pre + "sink"])
    return rnd(linear(o.reshape(T, H * D), t[pre + "o"], dtype=dtype), dtype)


def short_conv(z, w):
    """z [T, C], w [C, taps]: out_t = sum_j w[:, j] z_(t - taps + 1 + j), zeros before the first row."""
    taps = w.shape[1]
    padded = torch.cat([torch.zeros(taps - 1, z.shape[1]), z])
    return sum(w[:, j].float() * padded[j:j + z.shape[0]] for j in range(taps))


def delta_scan(q, k, v, g, beta):
    """S <- g S (row by row), u = beta (v - S^T k), S <- S + k u^T, o = S^T q. q, k, g [T, H, D]; v [T, H, Dv]; beta [T, H]."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1])
    out = []
    for i in range(T):
        S = g[i][:, :, None] * S
        u = beta[i][:, None] * (v[i] - (S * k[i][:, :, None]).sum(1))
        S = S + k[i][:, :, None] * u[:, None, :]
        out.append((S * q[i][:, :, None]).sum(1))
    return torch.stack(out)


def channel_decay(z, a_log, dt_bias, heads):
    """z [T, heads * D] -> g [T, heads, D] in (0, 1)."""
    z = (z + dt_bias.float()).view(z.shape[0], heads, -1)
    return torch.exp(-torch.exp(a_log.float())[None, :, None] * F.softplus(z, threshold=60.0))


def delta_rule(h, m, t, pre, eps, dtype):
    T = h.shape[0]
    H, G, D, Dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])

    def branch(name, heads, dim):
        z = rnd(linear(h, t[pre + name], dtype=dtype), dtype)
        return silu(short_conv(z, t[pre + name + ".conv"])).view(T, heads, dim)

    def narrow(first, second):
        return linear(h, t[pre + first], dtype=dtype) @ t[pre + second].float().T

    q, k, v = branch("q", G, D), branch("k", G, D), branch("v", H, Dv)
    q = q / torch.sqrt((q * q).sum(-1, keepdim=True) + 1e-6) / math.sqrt(D)
    k = k / torch.sqrt((k * k).sum(-1, keepdim=True) + 1e-6)
    beta = torch.sigmoid(linear(h, t[pre + "b"], dtype=dtype))
    g = channel_decay(narrow("a1", "a2"), t[pre + "A_log"], t[pre + "dt_bias"], H)
    o = delta_scan(q.repeat_interleave(H // G, 1), k.repeat_interleave(H // G, 1), v, g, beta)
    y = rms(o, t[pre + "norm"], eps) * torch.sigmoid(narrow("g1", "g2")).view(T, H, Dv)
    return rnd(linear(y.reshape(T, H * Dv), t[pre + "o"], dtype=dtype), dtype)


def mixer(h, layer, t, pre, eps, positions, dtype):
    m = layer["mixer"]
    if layer["type"] == "retention":
        return retention(h, m, t, pre, eps, positions, dtype)
    return float(m["left_scale"]) * key_value_attention(h, m["left"], t, pre + "left.", eps, dtype) + \
        float(m["right_scale"]) * delta_rule(h, m["right"], t, pre + "right.", eps, dtype)


def clamped_glu(g, u, limit):
    g, u = g.clamp(max=limit), u.clamp(-limit, limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1.0)


def feed_forward(h, mlp, t, pre, dtype):
    g = rnd(linear(h, t[pre + "gate"], t[pre + "gate.b"], dtype), dtype)
    u = rnd(linear(h, t[pre + "up"], t[pre + "up.b"], dtype), dtype)
    y = clamped_glu(g, u, float(mlp["limit"]))
    return rnd(linear(y, t[pre + "down"], t[pre + "down.b"], dtype), dtype)


def owner(config, i):
    """The layer whose tensors layer i uses."""
    while config["layers"][i].get("weights_of") is not None:
        i = int(config["layers"][i]["weights_of"])
    return i


def forward(ids, config, t, dtype=torch.float32, collect=None):
    """ids [T] of one sequence from its first token on -> float32 logits [T, vocab]; ``collect``: a list that receives the
    residual stream behind every layer."""
    ids = torch.as_tensor(ids, dtype=torch.long)
    eps = float(config["norm"]["eps"])
    positions = torch.arange(len(ids))
    x = embed(ids, config, t)
    for i, layer in enumerate(config["layers"]):
        p = f"l{owner(config, i)}."
        h = rnd(rms(x, t[p + "norm1"], eps), dtype)
        add = mixer(h, layer, t, p + "mix.", eps, positions, dtype)
        if layer.get("mlp") is not None:
            add = add + feed_forward(h, layer["mlp"], t, p + "mlp.", dtype)
        x = x + add
        if collect is not None:
            collect.append(x.clone())
    return linear(rms(x, t["final.norm"], eps), t["embed"], dtype=dtype)
