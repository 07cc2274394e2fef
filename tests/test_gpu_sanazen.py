"""Sanazen on the GPU against the plain implementation (``tests/plain/sanazen_plain.py``): every mechanism alone, then whole
models through the replay session and the engine: whole prompts, prefill + decoding, portions down to two tokens, mixed
batches with pages and state slots used again, edges of windows and of the kept first tokens that show, a far token through the
recurrence, the first tokens, long decoding, greedy generation through the scheduler."""
from __future__ import annotations

import json
import math

import pytest
import torch

from conftest import random_ids
from plain import sanazen_plain as P
from sanazen_cases import B, CASES, lively
from test_gpu_kasovik import _weights
from test_gpu_luzevik import CUTS, _alone, _run_cuts, close, ints, poison_freed_slots, q
from tolerances import F32_REL

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DTS = [torch.float32, torch.bfloat16]


# ----------------------------------------------------------------------------------------------- small kernels

@pytest.mark.parametrize("dt", DTS)
@pytest.mark.parametrize("W,scale", [(72, 2.5), (7, 1.0), (1030, 0.3), (4096, 1.0)])
def test_embedding_with_waves_of_the_position(dt, W, scale):
    from tokenmill_amd.parts import PositionWaves, TokenEmbedding
    torch.manual_seed(W)
    emb = TokenEmbedding(31, W, name="embed", scale=scale, waves=PositionWaves(W))
    t = {"embed": q(torch.randn(31, W), dt)}
    emb.load({"embed": t["embed"].to(dt).to(DEV)}, "")
    assert emb.by_position and emb.emit(None) is None and set(emb.tensor_specs("")) == {"embed"}
    places = [0, 1, 2, 63, 64, 1023, 4095, 100000]
    ids = torch.tensor([5, 0, 30, 7, 7, 2, 9, 11])
    got = emb.forward(ids.to(torch.int32).to(DEV), ints(places)).cpu()
    want = P.embed(ids, torch.tensor(places), {"embedding": {"scale": scale}, "width": W}, t)
    close(got[:7], want[:7], torch.float32, "rows")
    assert float((got[7] - want[7]).abs().max()) < 0.02, "a position whose angles 32-bit hardly resolves"


@pytest.mark.parametrize("dt", DTS)
@pytest.mark.parametrize("W", [72, 88, 1000, 1026, 4096, 5000])
def test_two_norms_of_one_sum(dt, W):
    from tokenmill_amd.parts import GroupRMSNorm, WeightedAdd
    from tokenmill_amd.parts.norm import norm_pair
    torch.manual_seed(W)
    T, eps = 7, 1e-5
    x = torch.randn(T, W) * 3
    x[3] *= 1e-4                                           # a row so small that eps matters
    ys = [torch.randn(T, W) * s for s in (1.0, 4.0, 0.02, 1.5)]
    for y in ys:
        y[3] *= 1e-4
    ys = [q(y, dt) for y in ys]
    scales = [0.7, -1.25, 1.0, 0.3]
    w1, w2 = q(torch.rand(W) + 0.5, dt), q(torch.randn(W), dt)
    dev = [y.to(dt).to(DEV) for y in ys]
    for wide in (False, True):                             # the weights in the model's type, or in 32-bit
        norms = []
        for w in (w1, w2):
            norms.append(GroupRMSNorm(W, eps, name="w"))
            norms[-1].load({"w": w.to(DEV) if wide else w.to(dt).to(DEV)}, "")
        for n in range(5):                                 # nothing pending, and one to four results (four: added in front)
            want = x + sum((s * y for s, y in zip(scales[:n], ys)), torch.zeros(()))
            resid = x.clone().to(DEV)
            way = WeightedAdd(scales[0], list(zip(dev[1:n], scales[1:n]))) if n else None
            a, b = norm_pair(norms[0], norms[1], resid, dev[0] if n else None, dt, way)
            close(resid.cpu(), want, torch.float32, f"the sum of {n}")
            close(a.float().cpu(), q(P.rms(want, w1, eps), dt), dt, f"first norm, {n}", bf16=2.0 ** -8)
            close(b.float().cpu(), q(P.rms(want, w2, eps), dt), dt, f"second norm, {n}", bf16=2.0 ** -8)
        resid = x.clone().to(DEV)
        a, b = norm_pair(norms[0], norms[1], resid, dev[1], dt)         # one plain result
        close(resid.cpu(), x + ys[1], torch.float32, "a plain result")
        close(b.float().cpu(), q(P.rms(x + ys[1], w2, eps), dt), dt, "second norm of a plain result", bf16=2.0 ** -8)


def test_scaled_and_capped_logits():
    from tokenmill_amd.parts import OutputHead
    torch.manual_seed(2)
    w = torch.randn(333, 40) * 4
    h = torch.randn(5, 40)
    for scale, cap in ((0.25, 30.0), (3.0, 0.5), (0.5, None), (1.0, 20.0), (1.0, None)):
        head = OutputHead(40, 333, None, name="head", suffixes=("", ".b"), scale=scale, cap=cap)
        head.load({"head": w.to(DEV)}, "")
        want = P.logits_of(h, {"logit_scale": scale, "logit_softcap": cap}, {"head": w}, torch.float32)
        close(head.forward(h.to(DEV)).cpu(), want, torch.float32, f"scale {scale}, cap {cap}")
        if scale != 1.0 or cap:
            assert head.emit(None, None) is None


# ----------------------------------------------------------------------------------------------- window attention with kept tokens

MASKS = [(6, 2, 64, 16, 40, 4, 150), (4, 1, 32, 16, 1, 33, 90), (8, 8, 128, 16, 100, 70, 330), (5, 1, 96, 32, 64, 1, 150), (3, 3, 20, 8, 9, 3, 60),
         (2, 1, 160, 16, 33, 17, 80), (4, 2, 64, 16, 300, 65, 700), (3, 1, 64, 16, 20, 0, 70), (2, 2, 32, 64, 24, 600, 640), (4, 4, 32, 16, 50, 257, 650)]


def _every_kernel(qa, k_pool, v_pool, tab, n, H, G_, D, page, scale, window, keep, at, gate=None):
    """The attention of positions ``at`` (a run up to n - 1) by every kernel that takes the sizes: name -> [len(at), H * D]."""
    from tokenmill_amd.hip import ops
    dt = qa.dtype
    m, places = len(at), ints(list(at))
    new = lambda rows=m: torch.full((rows, H * D), math.nan, dtype=dt, device=DEV)     # noqa: E731
    results, which = {}, {}
    g = lambda rows=slice(None): gate[rows] if gate is not None else None     # noqa: E731
    out = new()
    ops.attn_paged_softmax(qa[:m], out, k_pool, v_pool, tab, ints([0] * m), places, H, G_, D, D, scale, window, keep=keep, channel_gate=g())
    results["a token and head alone"] = out
    some = sorted({0, m // 2, m - 1})
    out = new(len(some))
    ops.attn_paged_softmax(qa[:len(some)], out, k_pool, v_pool, tab, ints([0] * len(some)), places[some].contiguous(), H, G_, D, D, scale,
                           window, keep=keep, channel_gate=g(some))
    results["few tokens, keys over wavefronts"] = out
    which["few tokens, keys over wavefronts"] = some
    tiles = torch.tensor([[0, i, min(16, m - i), at[i]] for i in range(0, m, 16)], dtype=torch.int32, device=DEV)
    if ops.attn_prefill_mfma_supported(dt, H, G_, D, page):
        for shared in (False, True):
            out = new()
            ops.attn_prefill_mfma(qa[:m], out, k_pool, v_pool, tab, tiles, H, G_, D, scale, window, shared=shared, keep=keep, channel_gate=g())
            results[f"prompt tiles, shared keys {shared}"] = out
        tabs = tab.expand(m, -1).contiguous()
        for split in (False, True):
            out = new()
            ops.attn_decode_mfma(qa[:m], out, k_pool, v_pool, tabs, ints([p + 1 for p in at]), H, G_, D, scale, window, n, split=split, keep=keep,
                                 channel_gate=g())
            results[f"single tokens, split {split}"] = out
    if ops.attn_prefill_f32_supported(dt, H, G_, D, page):
        out = new()
        ops.attn_prefill_f32(qa[:m], out, k_pool, v_pool, tab, tiles, H, G_, D, scale, window, keep=keep, channel_gate=g())
        results["prompt tiles in 32-bit"] = out
    return {k: (v.float().cpu(), which.get(k, range(m))) for k, v in results.items()}


@pytest.mark.parametrize("dt", DTS)
@pytest.mark.parametrize("H,G_,D,page,window,keep,n", MASKS)
def test_every_edge_of_the_window_and_of_the_kept_tokens_shows(dt, H, G_, D, page, window, keep, n):
    """Values with one channel set to one (position j sets channel j % D) and scores that are all zero: a token's result is,
    channel by channel, how many of the positions it sees set that channel, over their number. A position too many or too few at any
    edge, in every kernel that runs such an attention, changes it by more than the bound. Then the last tokens once more with
    the pages that nobody may see given away: what stands in their entries' place is full of NaN."""
    torch.manual_seed(n + D)
    pages = n // page + 3
    k_pool = torch.zeros((pages, page, G_, D), dtype=dt, device=DEV)
    v_flat = torch.zeros((pages, page, G_, D), dtype=dt)
    table = (torch.randperm(pages - 1)[: -(-n // page)] + 1).to(torch.int32)           # pages in no order; page 0 is somebody else's
    for j in range(n):
        v_flat[int(table[j // page]), j % page, :, j % D] = 1.0
    v_pool = v_flat.permute(0, 2, 3, 1).contiguous().to(DEV)
    qa = torch.zeros((n, H * D), dtype=dt, device=DEV)
    k_pool[0], v_pool[0] = math.nan, math.nan
    seen = P.visible(n, window, keep)
    want = (seen.float() @ torch.eye(D)[torch.arange(n) % D])[:, None, :] / seen.sum(-1).float()[:, None, None]
    first = max(n - 37, 0)
    gone = [i for i in range(len(table)) if i >= -(-keep // page) and (i + 1) * page <= max(0, first - window + 1)]
    given = table.clone()
    given[gone] = 0
    assert gone or n - window - keep < 2 * page + 37
    for tab, at in ((table, range(n)), (given, range(first, n))):
        for how, (got, which) in _every_kernel(qa, k_pool, v_pool, tab.view(1, -1).to(DEV), n, H, G_, D, page, 0.3, window, keep, list(at)).items():
            got = got.view(len(which), H, D)
            for i, p in enumerate(which):
                w = want[at[p]]
                err = (got[i] - w).abs().max()
                assert err <= (F32_REL if dt == torch.float32 else 2.0 ** -7) * float(w.max()), f"{how}: position {at[p]}: {float(err):.3e}"


@pytest.mark.parametrize("dt", DTS)
@pytest.mark.parametrize("D", [32, 64, 20, 128])
def test_far_keys_at_the_edges_of_what_is_kept(dt, D):
    """One key stands out for every query, by a score of 24 against scores near zero: where it is seen the result is its value, where
    it is not the result is something else altogether. The key is put at the last kept place, just behind it, at a window's
    oldest place and just before it, in every kernel; queries, other keys and values are random."""
    H, G_, page, window, keep, n = 4, 2, 16, 50, 19, 400
    pages = n // page + 2
    g = torch.Generator().manual_seed(D)
    k = torch.randn(n, G_, D, generator=g) * 0.1
    v = q(torch.randn(n, G_, D, generator=g), dt)
    qa = torch.randn(n, H, D, generator=g) * 0.1
    qa[:, :, 0] = 4.0
    table = torch.randperm(pages, generator=g)[: n // page].to(torch.int32)
    at = list(range(200, n))
    for far in (0, keep - 1, keep, 250 - window, 251 - window, 320):
        kk = k.clone()
        kk[:, :, 0], kk[far, :, 0] = 0.0, 12.0
        kk = q(kk, dt)
        k_flat, v_flat = torch.zeros((pages * page, G_, D), dtype=dt), torch.zeros((pages * page, G_, D), dtype=dt)
        slots = table.long()[torch.arange(n) // page] * page + torch.arange(n) % page
        k_flat[slots], v_flat[slots] = kk.to(dt), v.to(dt)
        k_pool = k_flat.view(pages, page, G_, D).to(DEV)
        v_pool = v_flat.view(pages, page, G_, D).permute(0, 2, 3, 1).contiguous().to(DEV)
        spread = lambda x: x.repeat_interleave(H // G_, 1)     # noqa: E731
        want = P.kept_window_attention(q(qa, dt), spread(kk), spread(v), 0.5, window, keep)
        for how, (got, which) in _every_kernel(qa[200:].reshape(-1, H * D).to(dt).to(DEV), k_pool, v_pool, table.view(1, -1).to(DEV), n, H, G_, D,
                                               page, 0.5, window, keep, at).items():
            if "few" in how:
                continue                                   # (its rows of q are the first ones)
            close(got.view(-1, H, D), want[200:], dt, f"key {far}, {how}", bf16=2.0 ** -6)


@pytest.mark.parametrize("dt", DTS)
@pytest.mark.parametrize("H,G_,D", [(4, 2, 32), (6, 1, 64), (3, 3, 20), (2, 1, 128), (2, 2, 160)])
def test_a_gate_per_channel_in_every_kernel(dt, H, G_, D):
    """The gate's rows are a view into wider rows; wide open, shut, and in between."""
    n, page, window, keep = 90, 16, 30, 3
    g = torch.Generator().manual_seed(D)
    k, v, qa = (q(torch.randn(n, h, D, generator=g), dt) for h in (G_, G_, H))
    gate = q(torch.randn(n, 8 + H * D, generator=g) * 3, dt)
    gate[5, 8:10], gate[6, 8:10] = 200.0, -200.0
    pages = n // page + 1
    pool = [torch.zeros((pages * page, G_, D), dtype=dt) for _ in range(2)]
    pool[0][:n], pool[1][:n] = k.to(dt), v.to(dt)
    k_pool = pool[0].view(pages, page, G_, D).to(DEV)
    v_pool = pool[1].view(pages, page, G_, D).permute(0, 2, 3, 1).contiguous().to(DEV)
    spread = lambda x: x.repeat_interleave(H // G_, 1)     # noqa: E731
    want = P.kept_window_attention(qa, spread(k), spread(v), 0.2, window, keep).reshape(n, -1) * torch.sigmoid(gate[:, 8:])
    for how, (got, which) in _every_kernel(qa.reshape(n, -1).to(dt).to(DEV), k_pool, v_pool, ints([list(range(pages))]), n, H, G_, D, page, 0.2, window,
                                           keep, list(range(n)), gate.to(dt).to(DEV)[:, 8:]).items():
        if "few" not in how:                               # (its rows of q are the first ones)
            close(got, want, dt, how, bf16=2.0 ** -6)


ATTENTIONS = [(6, 2, 20, 12, 4, 9, 3), (4, 2, 32, 32, 3, 24, 5), (8, 1, 64, 64, 2, 40, 18), (5, 1, 96, 96, 5, 1, 35), (2, 2, 128, 128, 4, 70, 1),
              (3, 1, 64, 64, 3, None, 0), (3, 3, 16, 16, 1, 33, 20), (4, 1, 24, 40, 3, 17, 1), (3, 1, 36, 30, 7, 21, 2)]


@pytest.mark.parametrize("dt", DTS)
@pytest.mark.parametrize("H,G_,D,Dv,taps,window,keep", ATTENTIONS)
def test_gated_attention_whole_in_portions_token_by_token_and_beside_another(dt, H, G_, D, Dv, taps, window, keep):
    """Biases, convolutions with their state, the norms over the whole projection, the mask, the gate per channel and the biased
    output projection together; in 16-token pages and in pages of 8 where the kernels take them."""
    from tokenmill_amd.parts import SoftmaxAttention
    attn = SoftmaxAttention(64, H, G_, D, Dv, 1.1 / math.sqrt(D), whole_norm_eps=1e-5, qkv_bias=True, window=window, keep_first=keep, taps=taps,
                            channel_gate=True, o_bias=True)
    g = torch.Generator().manual_seed(D)
    conv = {n + ".conv": torch.randn(s, taps, generator=g) * 0.7 for n, s in (("q", H * D), ("k", G_ * D), ("v", G_ * Dv))}
    w = _weights(attn, dt, 0.25, H * 3 + D, **conv)
    m = {"heads": H, "kv_heads": G_, "dim": D, "vdim": Dv, "conv": taps, "scale": 1.1 / math.sqrt(D)}
    if window is not None:
        m["mask"] = {"size": window, "keep_first": keep}
    T = 150
    torch.manual_seed(D)
    x = q(torch.randn(T, 64), dt)
    want = q(P.gated_attention(x, m, w, "a.", 1e-5, dt), dt)
    other = q(torch.randn(60, 64) * 2, dt)
    for page in (16, 8):
        pools, manager, runner = _alone(attn, dt, page=page, pages=80)
        assert len(pools.states) == (1 if taps > 1 else 0)
        for cuts in CUTS(T):
            close(_run_cuts(attn, pools, manager, runner, x, cuts, dt), want, dt, f"cuts {cuts[:4]}..", bf16=2.0 ** -6)
            for t in pools.states.values():                # whoever comes next into a slot finds zeros by the runner, not by luck
                t.fill_(math.nan)
            close(_run_cuts(attn, pools, manager, runner, x, cuts, dt, beside=other), want, dt, f"beside another, cuts {cuts[:4]}..", bf16=2.0 ** -6)
        assert manager.num_free_pages == manager.num_pages


@pytest.mark.parametrize("dt", DTS)
@pytest.mark.parametrize("rot,interleaved,per_head", [(8, False, False), (20, True, False), (0, False, True), (12, False, True)])
def test_a_convolution_with_rotations_and_norms_head_by_head(dt, rot, interleaved, per_head):
    """The other things the convolution's kernel may be asked for: rotated heads, norms head by head with shared weights."""
    from tokenmill_amd.hip import ops
    from tokenmill_amd.parts import RotaryEmbedding
    H, G_, D, Dv, taps, page, T, eps = 3, 1, 20, 12, 3, 4, 9, 1e-5
    torch.manual_seed(rot)
    C = (H + G_) * D + G_ * Dv
    proj, conv_w = q(torch.randn(T, C) * 2, dt), q(torch.randn(C, taps), dt)
    q_w, k_w = (torch.rand(D if per_head else n * D) + 0.5 for n in (H, G_))
    table = RotaryEmbedding(D, 100.0, 64, rotary_dim=rot, exact=True) if rot else None
    if rot:
        table.build_tables("cpu")
    places = torch.arange(T) + 11
    u = P.short_conv(proj, conv_w)

    def turned(x, w):
        x = P.rms(x, w, eps) if per_head else (P.rms(x.reshape(T, -1), w, eps)).view(x.shape)
        if not rot:
            return x
        c, s = table.cos[places][:, None], table.sin[places][:, None]
        a, b = (x[..., 0:rot:2], x[..., 1:rot:2]) if interleaved else (x[..., :rot // 2], x[..., rot // 2:rot])
        y = x.clone()
        for cols, val in zip((slice(0, rot, 2), slice(1, rot, 2)) if interleaved else (slice(0, rot // 2), slice(rot // 2, rot)), (a * c - b * s, b * c + a * s)):
            y[..., cols] = val
        return y
    slots = torch.randperm(16)[:T].to(torch.int32)
    k_pool = torch.zeros((4, page, G_, D), dtype=dt, device=DEV)
    v_pool = torch.zeros((4, G_, Dv, page), dtype=dt, device=DEV)
    q_out = torch.empty((T, H * D), dtype=dt, device=DEV)
    state = torch.zeros((2, taps - 1, C), dtype=dt, device=DEV)
    cos, sin = (table.cos.to(DEV), table.sin.to(DEV)) if rot else (None, None)
    ops.conv_norm_rope_store(proj.to(dt).to(DEV), conv_w.to(dt).to(DEV), state, ints([0, T]), ints([1]), ints([0] * T), 1, 0, q_out, H, G_, D, Dv,
                             q_w.to(DEV), k_w.to(DEV), eps, cos, sin, interleaved, places.to(torch.int32).to(DEV), slots.to(DEV), k_pool, v_pool,
                             per_head=per_head)
    s = slots.long()
    close(q_out.float().cpu().view(T, H, D), q(turned(u[:, :H * D].view(T, H, D), q_w), dt), dt, "q", bf16=2.0 ** -7)
    close(k_pool.float().cpu().view(-1, G_, D)[s], q(turned(u[:, H * D:(H + G_) * D].view(T, G_, D), k_w), dt), dt, "k", bf16=2.0 ** -7)
    close(v_pool.float().cpu().permute(0, 3, 1, 2).reshape(-1, G_, Dv)[s], q(u[:, (H + G_) * D:].view(T, G_, Dv), dt), dt, "v", bf16=2.0 ** -7)
    assert torch.equal(state[1].float().cpu(), proj[-(taps - 1):]) and float(state[0].abs().max()) == 0.0


@pytest.mark.parametrize("dt", DTS)
def test_a_key_inside_and_outside_of_what_is_seen_decides_through_the_mixer(dt):
    """One token's key stands out for every query: at the last kept place it decides results hundreds of tokens later, one place
    on only until the window has passed it; in a prompt and token by token."""
    from tokenmill_amd.parts import SoftmaxAttention
    H, G_, D, window, keep = 4, 2, 32, 21, 6
    attn = SoftmaxAttention(64, H, G_, D, D, 0.25, whole_norm_eps=1e-5, qkv_bias=True, window=window, keep_first=keep, taps=2, channel_gate=True,
                            o_bias=True)
    k_w = torch.randn(G_ * D, 64, generator=torch.Generator().manual_seed(3)) * 0.05
    q_w = torch.randn(H * D, 64, generator=torch.Generator().manual_seed(4)) * 0.01
    k_w[::D, 0] = 3.0                                      # channel 0 of the input reaches channel 0 of every key head
    q_w[::D, 1] = 2.0                                      # channel 1, set in every row, makes every query ask for it
    last = {n + ".conv": torch.tensor([[0.05, 1.0]]).repeat(s * D, 1) for n, s in (("q", H), ("k", G_), ("v", G_))}
    w = _weights(attn, dt, 0.25, 5, q=q_w, k=k_w, **last, **{"k.b": torch.zeros(G_ * D), "q.b": torch.zeros(H * D)})
    m = {"heads": H, "kv_heads": G_, "dim": D, "vdim": D, "scale": 0.25, "mask": {"size": window, "keep_first": keep}}
    T = 120
    for far in (keep - 1, keep, 40):
        torch.manual_seed(6)
        x = torch.randn(T, 64)
        x[:, 0], x[:, 1] = 0.0, 2.0
        x[far, 0] = 4.0
        x = q(x, dt)
        want = q(P.gated_attention(x, m, w, "a.", 1e-5, dt), dt)
        hidden = q(P.gated_attention(x, dict(m, mask={"size": window, "keep_first": 0}), w, "a.", 1e-5, dt), dt)
        if far < keep:
            assert float((want[-20:] - hidden[-20:]).norm()) > 0.5 * float(want[-20:].norm()), "the kept key does not stand out"
        pools, manager, runner = _alone(attn, dt, page=16)
        for cuts in ([T], [far, 1, window - 2, 1, 1, 1, T - far - window - 2], [1] * T):
            close(_run_cuts(attn, pools, manager, runner, x, cuts, dt), want, dt, f"key {far}, cuts {cuts[:4]}..", bf16=2.0 ** -6)


# ----------------------------------------------------------------------------------------------- the recurrence

@pytest.mark.parametrize("dt", DTS)
@pytest.mark.parametrize("H,D,Dv", [(3, 20, 12), (2, 64, 48), (1, 160, 24), (4, 128, 64), (2, 48, 160), (2, 32, 300)])
def test_lightning_attention_whole_in_portions_token_by_token_and_beside_another(dt, H, D, Dv):
    from tokenmill_amd.parts import Retention
    decay = [0.999, 0.9, 0.5, 1.0][:H]
    mixer = Retention(64, H, D, Dv, decay, 1e-5, silu=True, k_scale=1.0, whole_norm=True, sigmoid_gate=True)
    w = _weights(mixer, dt, 0.25, H * 5 + D)
    m = {"heads": H, "dim": D, "vdim": Dv, "decay": decay}
    T = 300                                                # whole: chunks or (keys of 160) segments; in pieces, scans and chunks
    assert T >= 2 * mixer.SEGMENT and mixer.CHUNKS_FROM <= 40
    torch.manual_seed(D)
    x = q(torch.randn(T, 64), dt)
    want = q(P.lightning(x, m, w, "a.", 1e-5, dt), dt)
    pools, manager, runner = _alone(mixer, dt)
    assert len(pools.states) == 1 and pools.states[0].dtype == torch.float32
    other = q(torch.randn(60, 64) * 2, dt)
    for cuts in CUTS(T):
        close(_run_cuts(mixer, pools, manager, runner, x, cuts, dt), want, dt, f"cuts {cuts[:4]}..", bf16=2.0 ** -5)
        for t in pools.states.values():
            t.fill_(math.nan)
        close(_run_cuts(mixer, pools, manager, runner, x, cuts, dt, beside=other), want, dt, f"beside another, cuts {cuts[:4]}..", bf16=2.0 ** -5)


@pytest.mark.parametrize("dt", DTS)
@pytest.mark.parametrize("H,D,Dv", [(3, 20, 12), (2, 64, 70), (1, 160, 24), (4, 128, 256), (2, 30, 600)])
def test_a_single_token_of_silu_projections_in_one_launch(dt, H, D, Dv):
    from tokenmill_amd.hip import ops
    g = torch.Generator().manual_seed(D + Dv)
    n = 5
    proj = torch.randn(n, H * (2 * D + Dv), generator=g).to(dt).to(DEV)
    slots = ints([4, 0, 6, 1, 3])
    decay = torch.tensor([0.999, 0.9, 0.5, 0.97][:H]).repeat_interleave(D)[None].contiguous().to(DEV)
    state = torch.randn(n + 2, H, D, Dv, generator=g).to(DEV)
    s1, s2 = state.clone(), state.clone()
    rows, want, got = (torch.full((n, k), math.nan, device=DEV) for k in (ops.retention_row_width(H, D, Dv), H * Dv, H * Dv))
    ops.retention_prepare(proj, None, None, ints([0] * n), rows, H, D, Dv, 0.5, silu=True)
    f = proj.float().cpu()
    plain = P.silu(f)
    plain[:, H * D:2 * H * D] *= 0.5
    close(rows[:, :H * (2 * D + Dv)].cpu(), plain, torch.float32, "prepared rows")
    ops.gla_scan(rows, 0, H * D, 2 * H * D, decay, want, s1, ints(list(range(n + 1))), slots, n, H, D, Dv, 1.0)
    ops.retention_step(proj, None, None, ints([0] * n), decay, s2, slots, None, H, D, Dv, 0.5, 1e-5, silu=True, o=got)
    close(got.cpu(), want.cpu(), torch.float32, "result")
    close(s2.cpu(), s1.cpu(), torch.float32, "state")


# ----------------------------------------------------------------------------------------------- experts

def test_router_of_sigmoid_scores():
    from tokenmill_amd.hip import ops
    torch.manual_seed(0)
    for E, top, T in ((7, 2, 33), (3, 3, 5), (16, 4, 64), (130, 6, 9), (1, 1, 4), (64, 64, 3), (300, 5, 7)):
        z = torch.randn(T, E + 2) * 2
        chosen, w = ops.moe_router(z.to(DEV)[:, :E + 2], E, top, sigmoid=True)
        want_c, want_w = P.route(z[:, :E], torch.eye(E), top, torch.float32)
        assert torch.equal(chosen.cpu().long(), want_c), f"choices of {top} among {E}"
        close(w.cpu(), want_w, torch.float32, "weights")
    chosen, w = ops.moe_router(torch.full((2, 6), 0.0).to(DEV), 6, 3, sigmoid=True)       # equal scores: the lower index first
    assert chosen.cpu().tolist() == [[0, 1, 2]] * 2 and torch.equal(w.cpu(), torch.full((2, 3), 0.5))
    chosen, w = ops.moe_router(torch.tensor([[-90.0, 90.0, -3.0]]).to(DEV), 3, 3, sigmoid=True)
    assert chosen.cpu().tolist() == [[1, 2, 0]] and torch.isfinite(w).all()


@pytest.mark.parametrize("dt", DTS)
@pytest.mark.parametrize("width,ff,experts,top,limit,shared,T", [(88, 40, 5, 2, 0.6, (24, 1.5), 77), (88, 16, 3, 3, 3.0, None, 9), (88, 32, 7, 1, 0.4, (48, 0.3), 1),
                                                                   (128, 48, 4, 1, 1.0, (32, 7.0), 300), (128, 24, 6, 4, 0.2, None, 130),
                                                                   (72, 20, 9, 2, 1.0, (20, 1.0), 600), (100, 12, 2, 2, 0.9, (36, 0.5), 2)])
def test_experts_on_weighted_inputs(dt, width, ff, experts, top, limit, shared, T):
    """Sigmoid router, experts with clamped gates whose weight multiplies their input, the gated shared expert: the part against
    the plain sum, at tile sizes of 32, 64 and 128 rows; a row alone gives what it has in the batch."""
    from types import SimpleNamespace
    from tokenmill_amd.parts import RoutedExperts
    torch.manual_seed(width + T)
    part = RoutedExperts(width, ff, experts, top, correction=False, activation="clamped_glu", limit=limit, scoring="sigmoid", weigh_input=True,
                         shared_ff=shared[0] if shared else None, shared_limit=shared[1] if shared else None)
    w = {name: q(torch.randn(spec.shape) * (0.15 if name.endswith(("router", "sg")) else 0.2), dt) for name, spec in part.tensor_specs("m.").items()}
    part.load({k: v.to(dt).to(DEV) for k, v in w.items()}, "m.")
    part.prepare(True)
    x = q(torch.randn(T, width), dt)
    mlp = {"expert": {"limit": limit}, "router": {"experts": experts, "top": top}}
    if shared:
        mlp["shared"] = {"ff": shared[0], "limit": shared[1]}
    step = SimpleNamespace(num_seqs=1)
    got = part.forward(x.to(dt).to(DEV), step).float().cpu()
    want = P.feed_forward(x, mlp, w, "m.", dt)
    _, weights = P.route(x, w["m.router"], top, dt)
    other = P.feed_forward(x * 1.0, dict(mlp, expert={"limit": 1e9}), w, "m.", dt)
    assert float(weights.max() - weights.min()) > 0.05 or T < 3
    assert float((other - want).abs().max()) > 0.05 * float(want.abs().max()), "the limit does not show"
    # a choice that is a near-tie in the router's scores may fall the other way: such rows are left out (few)
    c = torch.sigmoid(P.linear(x, w["m.router"], None, dt)).topk(min(top + 1, experts)).values
    sure = torch.ones(T, dtype=torch.bool) if top == experts else (c[:, top - 1] - c[:, top]) > 1e-4
    assert int(sure.sum()) >= T * 0.9
    close(got[sure], want[sure], dt, "experts", bf16=2.0 ** -6)
    i = int(sure.nonzero()[len(sure.nonzero()) // 2])
    one = part.forward(x[i:i + 1].to(dt).to(DEV), step).float().cpu()
    close(one[0], got[i], dt, "a row alone against the row in the batch", bf16=2.0 ** -7)


# ----------------------------------------------------------------------------------------------- whole models

@pytest.fixture(scope="module")
def models(tmp_path_factory):
    """name -> (folder, config, plain weights)."""
    from safetensors.torch import load_file, save_file
    from tokenmill_amd.weights.random_init import write_random_model
    out = {}
    for name, (cfg, seed, std, norm_std) in CASES.items():
        d = tmp_path_factory.mktemp(f"sanazen{name}")
        write_random_model(cfg, d, seed=seed, std=std, norm_std=norm_std)
        w = lively(cfg, load_file(str(d / "model.safetensors")), seed)
        save_file(w, str(d / "model.safetensors"))
        out[name] = (d, cfg, w)
    return out


_plain_cache: dict = {}


def plain_logits(models, name, ids, dt):
    key = (str(models[name][0]), tuple(ids), dt)
    if key not in _plain_cache:
        _, cfg, w = models[name]
        _plain_cache[key] = P.forward(ids, cfg, w, dt)
    return _plain_cache[key]


def check_rows(models, name, got, reqs, dt, what):
    """float32: 5e-5 of the largest logit. bfloat16: the model's floor is the largest distance of the plain bfloat16 run from the
    plain float32 run over the requests at hand, and the engine may be twice as far from the plain bfloat16 run (both differ from
    the 32-bit run by the same roundings, falling differently); one row in a hundred up to four times further: where a recurrence's
    read-out is next to nothing, the norm behind it blows the roundings of the layers before up for that one token, in the plain
    run as in the engine."""
    assert got, "no rows"
    if dt == torch.float32:
        for (rid, p), row in sorted(got.items()):
            want = plain_logits(models, name, reqs[rid], dt)
            err, bound = float((row - want[p]).abs().max()), 2.5 * F32_REL * float(want.abs().max())
            assert torch.isfinite(row).all() and err <= bound, f"{what}: request {rid} position {p}: {err:.3e} > {bound:.3e}"
        return
    floor = max(float((plain_logits(models, name, ids, dt) - plain_logits(models, name, ids, torch.float32)).abs().max()) for ids in reqs.values())
    over = 0
    for (rid, p), row in sorted(got.items()):
        want = plain_logits(models, name, reqs[rid], dt)
        bound = max(2.0 * floor, 2.0 ** -7 * float(want.abs().max()))
        err = float((row - want[p]).abs().max())
        assert torch.isfinite(row).all() and err <= 4 * bound, f"{what}: request {rid} position {p}: {err:.3e} > 4 * {bound:.3e}"
        over += err > bound
    assert over <= max(1, len(got) // 100), f"{what}: {over} of {len(got)} rows beyond twice the model's floor"


def make_requests(name, lengths, seed):
    vocab = CASES[name][0]["vocab"]
    return {f"r{i}": random_ids(n, vocab, seed * 100 + i) for i, n in enumerate(lengths)}


@pytest.mark.parametrize("dtype_name", ["float32", "bfloat16"])
@pytest.mark.parametrize("name,page", [("A", 16), ("B", 16), ("B", 8), ("C", 4), ("A", 64), ("C", 16)])
def test_whole_decode_portions_mixed(models, name, page, dtype_name):
    from tokenmill_amd.replay import ReplaySession
    from test_gpu_replay import assert_all_given_back, mixed, poison_freed_pages, portions, prefill_then_decode, run_trace, whole
    dt = {"float32": torch.float32, "bfloat16": torch.bfloat16}[dtype_name]
    s = ReplaySession(models[name][0], dtype_name, 4 * 128, max_requests=4, page_size=page)
    poison_freed_pages(s)
    poison_freed_slots(s)
    lengths = [1, 9, 26, 53, 120]
    reqs = make_requests(name, lengths, 1)
    got = run_trace(s, whole(reqs))
    assert len(got) == sum(lengths)
    check_rows(models, name, got, reqs, dt, "whole")
    assert_all_given_back(s)
    check_rows(models, name, run_trace(s, prefill_then_decode(reqs, tail=60)), reqs, dt, "prefill + decode")
    assert_all_given_back(s)
    steps = portions({k: v for k, v in reqs.items() if len(v) >= 2})
    assert min(len(e["tokens"]) for st in steps for e in st["entries"]) == 2
    check_rows(models, name, run_trace(s, steps), reqs, dt, "portions")
    assert_all_given_back(s)
    many = make_requests(name, [37, 64, 21, 90, 48, 33, 75, 18, 59, 44, 96, 27, 70, 52, 85, 40, 113, 66], 2)
    steps = mixed(many, seed=5)
    assert max(len(st["entries"]) for st in steps) == 4
    got = run_trace(s, steps)
    assert len(got) == sum(len(v) for v in many.values())
    check_rows(models, name, got, many, dt, "mixed")
    assert_all_given_back(s)


@pytest.mark.parametrize("dtype_name", ["float32", "bfloat16"])
def test_a_token_far_back_decides_the_logits_through_the_recurrence(models, dtype_name):
    """Weights made so that it shows. Hidden channel 0 is zero in every embedding row but one token's; the first layer's recurrence
    reads it into one key channel of a head that hardly forgets and asks for that channel by the constant channel 2 (either sign
    of it: two key channels). Hundreds of tokens later, far behind every window and not among the kept tokens, the logits follow
    the plain implementation's only if the state carries the ONE token, through prompts, portions and decoded tokens."""
    from safetensors.torch import save_file
    from tokenmill_amd.replay import ReplaySession
    from test_gpu_replay import portions, prefill_then_decode, run_trace, whole
    dt = {"float32": torch.float32, "bfloat16": torch.bfloat16}[dtype_name]
    d, cfg, w = models["A"]
    w2 = {k: v.clone() for k, v in w.items()}
    far_id, right = 7, cfg["layers"][0]["mixer"]["right"]
    D = right["dim"]
    emb = w["embed"].float().clone()
    emb[:, 0] = 0.0
    emb[far_id, 0] = 8.0
    qw, kw = w["l0.mix.right.q"].float().clone() * 0.1, w["l0.mix.right.k"].float().clone() * 0.1
    for i, sign in ((0, 1.0), (1, -1.0)):                  # head 1 (decay 0.995), its first two channels
        qw[D + i] = 0.0
        qw[D + i, 2] = 4.0 * sign
        kw[D + i] = 0.0
        kw[D + i, 0] = 6.0
    w2["embed"], w2["l0.mix.right.q"], w2["l0.mix.right.k"] = (t.to(torch.bfloat16) for t in (emb, qw, kw))
    folder = d.parent / f"sanazen_far_{dtype_name}"
    folder.mkdir(exist_ok=True)
    (folder / "config.json").write_text(json.dumps(cfg))
    save_file(w2, str(folder / "model.safetensors"))
    ids = [t if t != far_id else far_id + 1 for t in random_ids(420, cfg["vocab"], 9)]
    ids[45] = far_id
    local = {"A": (folder, cfg, w2)}
    with_far = P.forward(ids, cfg, w2, torch.float32)
    swapped = list(ids)
    swapped[45] = far_id + 1
    without = P.forward(swapped, cfg, w2, torch.float32)
    moved = float((with_far[-40:] - without[-40:]).abs().max()) / float(with_far.abs().max())
    assert moved > 0.02, f"the far token moves the last logits by {moved:.3g} of their size only: the test would not show a lost state"
    s = ReplaySession(folder, dtype_name, 448, max_requests=4, page_size=16)
    for steps, what in ((whole({"a": ids}), "whole"), (prefill_then_decode({"a": ids}, tail=48), "decoded"), (portions({"a": ids}), "portions")):
        check_rows(local, "A", run_trace(s, steps), {"a": ids}, dt, f"far token, {what}")


@pytest.mark.parametrize("dtype_name", ["float32", "bfloat16"])
def test_long_decoding_over_many_page_borders(models, dtype_name):
    """One token at a time from the third token on: every page border and every window is passed by decoded tokens and the
    convolutions' and the recurrences' states are carried over 250 steps, two requests beside each other that start at different
    times."""
    from tokenmill_amd.replay import ReplaySession
    from test_gpu_replay import assert_all_given_back, poison_freed_pages, run_trace
    dt = {"float32": torch.float32, "bfloat16": torch.bfloat16}[dtype_name]
    s = ReplaySession(models["A"][0], dtype_name, 512, max_requests=4, page_size=8)
    poison_freed_pages(s)
    n, m = 260, 150
    a, b = random_ids(n, 211, 77), random_ids(m, 211, 78)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:3], "want": [0, 1, 2]}], "end": []}]
    for p in range(3, n):
        entries = [{"id": "a", "tokens": [a[p]], "want": [0]}]
        if p == 60:
            entries.append({"id": "b", "tokens": b[:2], "want": [0, 1]})
        elif 60 < p < 60 + m - 1:
            entries.append({"id": "b", "tokens": [b[p - 59]], "want": [0]})
        ends = (["a"] if p == n - 1 else []) + (["b"] if p == 60 + m - 2 else [])
        steps.append({"step": p - 2, "entries": entries, "end": ends})
    got = run_trace(s, steps)
    assert len(got) == n + m
    check_rows(models, "A", got, {"a": a, "b": b}, dt, "long decoding")
    assert_all_given_back(s)


@pytest.mark.parametrize("dtype_name", ["float32", "bfloat16"])
def test_a_request_alone_and_in_a_batch_and_pages_given_back_behind_the_window(models, dtype_name):
    """The same request alone, and beside three others of unequal lengths in a pool that is too small for all of them without the
    pages that fall behind the windows; its logits differ by rounding at most, and the pages of kept tokens stay."""
    from tokenmill_amd.cache.manager import RELEASED
    from tokenmill_amd.replay import ReplaySession
    from test_gpu_replay import assert_all_given_back, poison_freed_pages, run_trace
    dt = {"float32": torch.float32, "bfloat16": torch.bfloat16}[dtype_name]
    reqs = make_requests("B", [200, 31, 90, 64], 7)
    rows = {}
    for who in (["r0"], list(reqs)):
        s = ReplaySession(models["B"][0], dtype_name, 320, max_requests=4, page_size=16)
        poison_freed_pages(s)
        free = s.manager.num_free_pages
        steps, at = [], {r: 0 for r in who}
        while any(at[r] < len(reqs[r]) for r in who):
            entries, ends = [], []
            for i, r in enumerate(who):
                n = min((1, 17, 2, 40)[(len(steps) + i) % 4] if r != "r0" else (40, 1, 23, 2)[len(steps) % 4], len(reqs[r]) - at[r])
                if n:
                    entries.append({"id": r, "tokens": reqs[r][at[r]:at[r] + n], "want": list(range(n))})
                    at[r] += n
                    if at[r] == len(reqs[r]):
                        ends.append(r)
            steps.append({"step": len(steps), "entries": entries, "end": ends})
        got = run_trace(s, steps[:-1])
        table = [[i for i, p in enumerate(t) if p == RELEASED] for t in s.manager.live["r0"].tables]
        # windows of 24 and 64 beside 5 and 18 kept tokens: pages 0, and 0 and 1, are held; the next ones are gone
        assert all(t for t in table) and min(table[0]) == 1 and min(table[1]) == 2
        got.update(run_trace(s, steps[-1:]))
        check_rows(models, "B", got, reqs, dt, f"{len(who)} requests")
        rows[len(who)] = got
        assert s.manager.num_free_pages == free
        assert_all_given_back(s)
    scale = max(float(r.abs().max()) for r in rows[1].values())
    worst = max(float((rows[1]["r0", p] - rows[4]["r0", p]).abs().max()) for p in range(200))
    assert worst <= (2.5 * F32_REL if dt == torch.float32 else 2.0 ** -4) * scale, f"alone against in a batch: {worst:.3e} of {scale:.3g}"


def test_greedy_generation_through_the_engine_and_its_graphs(models):
    """The engine's own entry point: scheduler, chunked prefill, sampling, HIP graphs for the decode steps, decode steps
    queued ahead. Every token is the plain implementation's first choice at its place (or a near-tie with it), and all
    modes agree."""
    from tokenmill_amd import EngineConfig, LLMEngine, SamplingParams
    d, cfg, w = models["A"]
    prompts = [random_ids(n, 211, 500 + i) for i, n in enumerate([12, 3, 30, 7, 21, 16, 45, 25, 5, 18])]
    params = [SamplingParams(max_tokens=8 + 5 * (i % 4), ignore_eos=True) for i in range(len(prompts))]
    outs = {}
    for mode in ("eager", "graphs", "chunked", "ahead"):
        eng = LLMEngine(EngineConfig(model=str(d), dtype="float32", block_size=8, num_blocks=48, max_model_len=96,
                                     max_num_seqs=4, max_num_batched_tokens=32 if mode == "chunked" else 64, watermark=0.0,
                                     hip_graphs=mode != "eager", enable_chunked_prefill=mode == "chunked",
                                     pipeline_decode=mode == "ahead"))
        kinds = [type(p).__name__ for p in eng.runner.program.foreign_parts]
        assert kinds.count("ParallelMixer") == 3 and kinds.count("TokenEmbedding") == 1 and kinds.count("OutputHead") == 1
        outs[mode] = eng.generate(prompts, params)
        if mode in ("graphs", "ahead"):
            assert eng.runner.graphs.replays > 10
        assert (eng.stats["steps_ahead"] > 5) == (mode == "ahead")
        assert eng.cache.num_free_pages == eng.cache.num_pages
    tokens = {m: [list(o) for o in outs[m]] for m in outs}
    assert tokens["eager"] == tokens["graphs"] == tokens["chunked"] == tokens["ahead"]
    exempt = 0
    for prompt, toks in zip(prompts, tokens["eager"]):
        rows = P.forward(prompt + toks[:-1], cfg, w, torch.float32)[len(prompt) - 1:]
        for row, tok in zip(rows, toks):
            best = int(row.argmax())
            if tok != best:
                assert float(row[best] - row[tok]) <= 4 * F32_REL * float(row.abs().max()), "a token that is no near-tie"
                exempt += 1
    assert exempt <= 2


def test_command_line_generates_with_a_random_sanazen_model(tmp_path):
    import subprocess
    import sys
    from conftest import ROOT
    (tmp_path / "config.json").write_text(json.dumps(B))
    r = subprocess.run([sys.executable, "-m", "tokenmill_amd.generate", "--random", str(tmp_path / "config.json"), "--prompt-ids",
                        "5,9,33,2;7,7", "--max-tokens", "6", "--max-model-len", "64", "--ignore-eos"], capture_output=True, text=True, cwd=ROOT, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    lines = [json.loads(ln) for ln in r.stdout.splitlines() if ln.startswith("{")]
    assert [len(ln["output_ids"]) for ln in lines] == [6, 6] and all(0 <= t < 150 for ln in lines for t in ln["output_ids"])
