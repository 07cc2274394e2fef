"""Kasovik on the GPU against the plain implementation (``tests/plain/kasovik_plain.py``): every mechanism alone, then whole
models through the replay session and the engine: whole prompts, prefill + decoding, portions down to two tokens, mixed
batches with pages and state slots used again, window edges and sinks that show, far tokens through both recurrences, the
first tokens, long decoding, greedy generation through the scheduler."""
from __future__ import annotations

import json
import math

import pytest
import torch

from conftest import random_ids
from kasovik_cases import A, B, CASES, lively
from plain import kasovik_plain as P
from test_gpu_luzevik import CUTS, _alone, _run_cuts, close, ints, poison_freed_slots, q
from tolerances import F32_REL

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DTS = [torch.float32, torch.bfloat16]


def _weights(part, dt, std, seed, **fixed):
    """Random weights of a part drawn over its declared tensors (on the CPU and in the part); ``fixed``: name -> tensor."""
    g = torch.Generator().manual_seed(seed)
    w = {}
    for name, spec in part.tensor_specs("a.").items():
        shape = spec.drawn_shape()
        t = torch.rand(shape, generator=g) + 0.5 if spec.init == "ones" else torch.randn(shape, generator=g) * std
        w[name] = q(fixed.get(name[2:], t), dt)
    part.load({k: v.to(dt).to(DEV) for k, v in w.items()}, "a.")
    part.prepare(True)
    return w


# ----------------------------------------------------------------------------------------------- small kernels

@pytest.mark.parametrize("dt", DTS)
def test_rows_of_pairs_whole_in_portions_and_beside_another_request(dt):
    """The pair's row at every place of a sequence: the first token, inside a portion, a portion's first token (the token before
    comes from the request's slot), single tokens; two requests beside each other; multipliers whose products need 64 bits."""
    from tokenmill_amd.cache import CacheManager
    from tokenmill_amd.cache.pool import CachePools
    from tokenmill_amd.engine.runner import ModelRunner, StepEntry
    from tokenmill_amd.parts import Retention, TokenEmbedding
    from tokenmill_amd.parts.embedding import PairRows
    from test_gpu_parts import OneLayer
    torch.manual_seed(1)
    vocab, width = 70000, 12
    for buckets, mul_prev, mul_cur, scale in ((19, 2147483647, 2147480009, 1.5), (1, 3, 5, 1.0), (64, 64, 1, 0.25)):
        emb = TokenEmbedding(vocab, width, name="embed", scale=scale, pairs=PairRows(buckets, width, mul_prev, mul_cur, name="bigram"))
        t = {"embed": torch.randn(vocab, width), "bigram": torch.randn(buckets + 1, width)}
        t = {k: q(v, dt) for k, v in t.items()}
        emb.load({k: v.to(dt).to(DEV) for k, v in t.items()}, "")
        assert emb.emit(None) is None and set(emb.tensor_specs("")) == {"embed", "bigram"}
        cfg = {"embedding": {"scale": scale, "bigram": {"buckets": buckets, "mul_prev": mul_prev, "mul_cur": mul_cur}}}
        model = OneLayer(Retention(12, 1, 4, 4, [0.5], 1e-5))
        specs = model.cache_specs()
        model.cache_specs = lambda: specs + [emb.cache_spec()]
        pools = CachePools(model, 8, 8, 3, dt, DEV)
        manager = CacheManager(pools.group_specs, 8, 8, 3)

        class Shell:
            device = torch.device(DEV)
            head = type("H", (), {"vocab": vocab})()

            def program(self, views, tune=None):
                return None
        runner = ModelRunner(Shell(), pools, 64)
        reqs = {"a": random_ids(31, vocab, 3), "b": random_ids(31, vocab, 4)}
        reqs["a"][7] = reqs["a"][8] = vocab - 1
        want = {r: P.embed(torch.tensor(v), cfg, t) for r, v in reqs.items()}
        for t_ in pools.states.values():
            t_.fill_(77)
        for cuts in ({"a": [31], "b": [2, 29]}, {"a": [1, 1, 2, 5, 1, 21], "b": [4, 1, 1, 1, 1, 23]}):
            held = {r: manager.allocate(r, 31) for r in reqs}
            at = {r: 0 for r in reqs}
            for i in range(max(len(c) for c in cuts.values())):
                entries, names = [], []
                for r, c in cuts.items():
                    if i < len(c):
                        entries.append(StepEntry(held[r], at[r], reqs[r][at[r]:at[r] + c[i]], []))
                        names.append((r, at[r], c[i]))
                        at[r] += c[i]
                ctx, _ = runner.prepare(entries)
                got = emb.forward_step(ctx, pools.views[-1]).cpu()
                row = 0
                for single in (False, True):               # portions first, single tokens behind them
                    for r, lo, n in names:
                        if (n == 1) == single:
                            close(got[row:row + n], want[r][lo:lo + n], torch.float32, f"{r} {lo}..{lo + n}")
                            row += n
            for r in held.values():
                manager.free(r)


@pytest.mark.parametrize("dt", DTS)
@pytest.mark.parametrize("W", [72, 88, 1000, 1026, 4096, 5000])
def test_several_results_added_at_once_and_normed(dt, W):
    from tokenmill_amd.parts import GroupRMSNorm, WeightedAdd
    torch.manual_seed(W)
    T, eps = 7, 1e-5
    x = torch.randn(T, W) * 3
    ys = [q(torch.randn(T, W) * s, dt) for s in (1.0, 4.0, 0.02, 1.5)]
    x[3] *= 1e-4
    for y in ys:
        y[3] *= 1e-4                                       # a row so small that eps matters
    ys = [q(y, dt) for y in ys]
    scales = [0.7, -1.25, 1.0, 0.3]
    w = q(torch.rand(W) + 0.5, dt)
    dev = [y.to(dt).to(DEV) for y in ys]
    for n in (1, 2, 3, 4):
        want = x + sum(s * y for s, y in zip(scales[:n], ys))
        for wide in (False, True):                         # the weight in the model's type, or in 32-bit
            norm = GroupRMSNorm(W, eps, name="w")
            norm.load({"w": w.to(DEV) if wide else w.to(dt).to(DEV)}, "")
            way = WeightedAdd(scales[0], list(zip(dev[1:n], scales[1:n])))
            resid = x.clone().to(DEV)
            out = norm.add_norm(resid, dev[0], dt, delta_norm=way)
            close(resid.cpu(), want, torch.float32, f"the sum of {n}")
            close(out.float().cpu(), q(P.rms(want, w, eps), dt), dt, f"the norm of the sum of {n}", bf16=2.0 ** -8)
            resid = x.clone().to(DEV)
            rows = ints([5, 0, 3])
            some = norm.add_norm(resid, dev[0], dt, rows=rows, delta_norm=way)
            close(some.float().cpu(), q(P.rms(want, w, eps), dt)[[5, 0, 3]], dt, f"wanted rows, {n}", bf16=2.0 ** -8)
            assert torch.equal(resid.cpu(), x), "wanted rows leave the stream as it is"
        resid = x.clone().to(DEV)
        way.add_normed(resid, dev[0])
        close(resid.cpu(), want, torch.float32, f"the add alone, {n}")


@pytest.mark.parametrize("dt", DTS)
@pytest.mark.parametrize("ff,limit", [(52, 0.8), (56, 7.0), (2816, 1.5)])
def test_clamped_gate(dt, ff, limit):
    from tokenmill_amd.hip import ops
    from tokenmill_amd.parts import GatedFeedForward
    torch.manual_seed(ff)
    gu = q(torch.randn(9, 2 * ff) * 3, dt)
    gu[0, 0], gu[0, ff] = limit, -limit
    gu[1, 0], gu[1, 1], gu[1, ff], gu[1, ff + 1] = 200.0, -200.0, 200.0, -200.0
    gu = q(gu, dt)
    out = torch.empty((9, ff), dtype=dt, device=DEV)
    ops.clamped_glu(gu.to(dt).to(DEV), out, limit, 1.702)
    close(out.float().cpu(), q(P.clamped_glu(gu[:, :ff], gu[:, ff:], limit), dt), dt, "clamped gate", bf16=2.0 ** -8)
    if ff > 100:
        return
    part = GatedFeedForward(64, ff, "clamped_glu", bias=True, limit=limit)
    w = _weights(part, dt, 0.3, ff)
    for n in (1, 5, 70):
        x = q(torch.randn(n, 64), dt)
        want = P.feed_forward(x, {"limit": limit}, {k[2:]: v for k, v in w.items()}, "", dt)
        close(part.forward(x.to(dt).to(DEV)).float().cpu(), q(want, dt), dt, f"feed-forward, {n} rows", bf16=2.0 ** -6)


# ----------------------------------------------------------------------------------------------- window attention

@pytest.mark.parametrize("dt", DTS)
@pytest.mark.parametrize("H,G_,D", [(6, 2, 20), (4, 1, 64), (5, 5, 32), (3, 1, 128)])
def test_unit_norm_head_by_head_and_values_that_are_the_keys(dt, H, G_, D):
    from tokenmill_amd.hip import ops
    torch.manual_seed(D)
    T, page, eps = 9, 4, 1e-5
    proj = torch.randn(T, H * D + G_ * D) * 2
    proj[3, :D] *= 1e-4                                    # heads so small that eps matters
    proj[4, H * D:H * D + D] *= 1e-4
    slots = torch.randperm(T + 5)[:T].to(torch.int32)
    k_pool = torch.zeros((4, page, G_, D), dtype=dt, device=DEV)
    v_pool = torch.zeros((4, G_, D, page), dtype=dt, device=DEV)
    q_out = torch.empty((T, H * D), dtype=dt, device=DEV)
    ops.whole_norm_rope_store(proj.to(DEV), q_out, H, G_, D, D, None, None, eps, None, None, False, None, slots.to(DEV), k_pool, v_pool,
                              per_head=True, unit=True, v_is_k=True)
    raw = proj[:, H * D:].view(T, G_, D)
    close(q_out.float().cpu().view(T, H, D), q(P.unit(proj[:, :H * D].view(T, H, D), eps), dt), dt, "q", bf16=2.0 ** -8)
    close(k_pool.float().cpu().view(-1, G_, D)[slots.long()], q(P.unit(raw, eps), dt), dt, "cached k", bf16=2.0 ** -8)
    assert torch.equal(v_pool.float().cpu().permute(0, 3, 1, 2).reshape(-1, G_, D)[slots.long()], q(raw, dt)), "a value is the key as projected"


@pytest.mark.parametrize("dt", DTS)
@pytest.mark.parametrize("H,G_,D,page,window,n", [(6, 2, 64, 16, 40, 150), (4, 1, 32, 16, 1, 60), (8, 8, 128, 16, 100, 330), (5, 1, 96, 32, 64, 150),
                                                  (3, 3, 20, 8, 9, 60), (2, 1, 160, 16, 33, 80), (4, 2, 64, 16, 300, 700)])
def test_a_sink_counts_once_and_every_window_edge_shows(dt, H, G_, D, page, window, n):
    """Values with one channel set to one (position j sets channel j % D) and scores that are all zero: a token's result is,
    channel by channel, how many of the positions it sees set that channel, over their number plus exp(sink) of the head. A sink
    left out, counted twice (once a wavefront or chunk) or scaled, and a position too many or too few at either edge of the
    window, in every kernel that runs such an attention, change it by more than the bound."""
    from tokenmill_amd.hip import ops
    torch.manual_seed(n + D)
    pages = n // page + 2
    k_pool = torch.zeros((pages, page, G_, D), dtype=dt, device=DEV)
    v_flat = torch.zeros((pages, page, G_, D), dtype=dt)
    table = torch.randperm(pages)[: -(-n // page)].to(torch.int32)                   # pages in no order
    for j in range(n):
        v_flat[int(table[j // page]), j % page, :, j % D] = 1.0
    v_pool = v_flat.permute(0, 2, 3, 1).contiguous().to(DEV)
    sink = (torch.arange(H).float() % 7) - 3.0                                       # exp(sink) from 0.05 to 20
    qa = torch.zeros((n, H * D), dtype=dt, device=DEV)
    tab, places = table.view(1, -1).to(DEV), ints(list(range(n)))
    scale = 0.3
    seqs = ints([0] * n)
    results = {}
    out = torch.full((n, H * D), math.nan, dtype=dt, device=DEV)
    ops.attn_paged_softmax(qa, out, k_pool, v_pool, tab, seqs, places, H, G_, D, D, scale, window, sink=sink.to(DEV))
    results["a wavefront a token and head"] = out.float().cpu()
    few = torch.full((3, H * D), math.nan, dtype=dt, device=DEV)
    ops.attn_paged_softmax(qa[:3], few, k_pool, v_pool, tab, seqs, ints([0, n // 2, n - 1]), H, G_, D, D, scale, window, sink=sink.to(DEV))
    results["few tokens, keys over wavefronts"] = few.float().cpu()
    at = {"few tokens, keys over wavefronts": [0, n // 2, n - 1]}
    tiles = torch.tensor([[0, a, min(16, n - a), a] for a in range(0, n, 16)], dtype=torch.int32, device=DEV)
    if dt == torch.bfloat16 and ops.attn_prefill_mfma_supported(dt, H, G_, D, page):
        for shared in (False, True):
            out = torch.full((n, H * D), math.nan, dtype=dt, device=DEV)
            ops.attn_prefill_mfma(qa, out, k_pool, v_pool, tab, tiles, H, G_, D, scale, window, shared=shared, sink=sink.to(DEV))
            results[f"prompt tiles, shared keys {shared}"] = out.float().cpu()
        tabs = tab.expand(n, -1).contiguous()
        for split in (False, True):
            out = torch.full((n, H * D), math.nan, dtype=dt, device=DEV)
            ops.attn_decode_mfma(qa, out, k_pool, v_pool, tabs, ints(list(range(1, n + 1))), H, G_, D, scale, window, n, split=split,
                                 sink=sink.to(DEV))
            results[f"single tokens, split {split}"] = out.float().cpu()
    if dt == torch.float32 and ops.attn_prefill_f32_supported(dt, H, G_, D, page):
        out = torch.full((n, H * D), math.nan, dtype=dt, device=DEV)
        ops.attn_prefill_f32(qa, out, k_pool, v_pool, tab, tiles, H, G_, D, scale, window, sink=sink.to(DEV))
        results["prompt tiles in 32-bit"] = out.float().cpu()
    pos = torch.arange(n)
    seen = ((pos[:, None] - pos[None, :]) >= 0) & ((pos[:, None] - pos[None, :]) < window)
    counts = seen.float() @ torch.eye(D)[pos % D]                                    # [n, D]
    want = counts[:, None, :] / (seen.sum(-1).float()[:, None, None] + torch.exp(sink)[None, :, None])
    for how, got in results.items():
        which = at.get(how, list(range(n)))
        got = got.view(len(which), H, D)
        for i, p in enumerate(which):
            err = (got[i] - want[p]).abs().max()
            assert err <= (F32_REL if dt == torch.float32 else 2.0 ** -7) * float(want[p].max()), f"{how}: position {p}: {float(err):.3e}"


@pytest.mark.parametrize("dt", DTS)
@pytest.mark.parametrize("H,G_,D,window,page", [(6, 2, 20, 9, 8), (4, 2, 32, 24, 16), (8, 1, 64, 40, 16), (5, 1, 96, 1, 16), (2, 2, 128, 70, 16),
                                                (3, 1, 64, None, 16)])
def test_window_attention_whole_in_portions_and_token_by_token(dt, H, G_, D, window, page):
    from tokenmill_amd.parts import SoftmaxAttention
    attn = SoftmaxAttention(64, H, G_, D, D, 0.9 / math.sqrt(D), window=window, head_norm_eps=1e-5, norm_weights=False, sink=True,
                            keys_are_values=True)
    w = _weights(attn, dt, 0.25, H * 3 + D, sink=torch.randn(H, generator=torch.Generator().manual_seed(D)))
    m = {"heads": H, "kv_heads": G_, "dim": D, "scale": 0.9 / math.sqrt(D), "mask": {"size": window} if window else None}
    T = 150
    torch.manual_seed(D)
    x = q(torch.randn(T, 64), dt)
    want = q(P.key_value_attention(x, m, w, "a.", 1e-5, dt), dt)
    pools, manager, runner = _alone(attn, dt, page=page, pages=80)
    for cuts in CUTS(T):
        close(_run_cuts(attn, pools, manager, runner, x, cuts, dt), want, dt, f"cuts {cuts[:4]}..", bf16=2.0 ** -6)
    assert manager.num_free_pages == manager.num_pages


@pytest.mark.parametrize("dt", DTS)
def test_a_key_at_the_edge_of_the_window_decides_just_inside_and_not_just_outside(dt):
    """One token's key stands out for every query (a score of several units against scores near zero): the last token that sees
    it and the first that does not differ by far, and both follow the plain implementation, in a prompt and token by token."""
    from tokenmill_amd.parts import SoftmaxAttention
    H, G_, D, window, page, far = 4, 2, 32, 21, 16, 30
    attn = SoftmaxAttention(64, H, G_, D, D, 0.25, window=window, head_norm_eps=1e-5, norm_weights=False, sink=True, keys_are_values=True)
    k_w = torch.randn(G_ * D, 64, generator=torch.Generator().manual_seed(3)) * 0.05
    q_w = torch.randn(H * D, 64, generator=torch.Generator().manual_seed(4)) * 0.01
    k_w[::D, 0] = 3.0                                      # channel 0 of the input reaches channel 0 of every key head
    q_w[::D, 1] = 2.0                                      # channel 1, set in every row, makes every query ask for it
    w = _weights(attn, dt, 0.25, 5, q=q_w, k=k_w, sink=torch.zeros(H))
    m = {"heads": H, "kv_heads": G_, "dim": D, "scale": 0.25, "mask": {"size": window}}
    T = 80
    torch.manual_seed(6)
    x = torch.randn(T, 64)
    x[:, 0], x[:, 1] = 0.0, 2.0
    x[far, 0] = 4.0
    x = q(x, dt)
    want = q(P.key_value_attention(x, m, w, "a.", 1e-5, dt), dt)
    inside, outside = want[far + window - 1], want[far + window]
    assert float(inside.norm()) > 1.5 * float(outside.norm()), "the key does not stand out: the test would not show a wrong edge"
    pools, manager, runner = _alone(attn, dt, page=page)
    for cuts in ([T], [far, 1, window - 2, 1, 1, 1, T - far - window - 2], [1] * T):
        got = _run_cuts(attn, pools, manager, runner, x, cuts, dt)
        for p in (far, far + 1, far + window - 2, far + window - 1, far + window, far + window + 1):
            close(got[p], want[p], dt, f"cuts {cuts[:4]}.. position {p - far} behind the key", bf16=2.0 ** -6)


# ----------------------------------------------------------------------------------------------- the recurrences

@pytest.mark.parametrize("dt", DTS)
@pytest.mark.parametrize("H,D,Dv,rot", [(3, 20, 12, 8), (2, 64, 32, 64), (1, 160, 24, 0), (4, 128, 64, 32), (2, 48, 70, 48)])
def test_retention_whole_in_portions_token_by_token_and_beside_another(dt, H, D, Dv, rot):
    from tokenmill_amd.parts import Retention, RotaryEmbedding
    decay = [0.999, 0.9, 0.5, 0.97][:H]
    rotary = RotaryEmbedding(D, 3e3, 640, rotary_dim=rot, exact=True) if rot else None
    mixer = Retention(64, H, D, Dv, decay, 1e-5, rotary=rotary)
    w = _weights(mixer, dt, 0.25, H * 5 + D)
    m = {"heads": H, "dim": D, "vdim": Dv, "decay": decay, "rot": {"base": 3e3, "dims": rot} if rot else None}
    T = 300                                                # whole: chunks or (keys of 160) segments; in pieces, scans and chunks
    assert T >= 2 * mixer.SEGMENT and mixer.CHUNKS_FROM <= 40
    torch.manual_seed(D)
    x = q(torch.randn(T, 64), dt)
    want = q(P.retention(x, m, w, "a.", 1e-5, torch.arange(T), dt), dt)
    pools, manager, runner = _alone(mixer, dt)
    assert len(pools.states) == 1 and pools.states[0].dtype == torch.float32
    other = q(torch.randn(60, 64) * 2, dt)
    for cuts in CUTS(T):
        close(_run_cuts(mixer, pools, manager, runner, x, cuts, dt), want, dt, f"cuts {cuts[:4]}..", bf16=2.0 ** -6)
        for t in pools.states.values():                    # whoever comes next into a slot finds zeros by the runner, not by luck
            t.fill_(math.nan)
        close(_run_cuts(mixer, pools, manager, runner, x, cuts, dt, beside=other), want, dt, f"beside another, cuts {cuts[:4]}..", bf16=2.0 ** -6)


def test_a_retention_remembers_one_token_among_hundreds():
    """Keys that are zero but for one token's, queries that ask for it: hundreds of tokens later the result points at its value
    with the weight its head's decay leaves, whole (segments) and cut."""
    from tokenmill_amd.hip import ops
    H, D, Dv, T, far = 2, 32, 8, 400, 17
    rows = torch.zeros(T, ops.retention_row_width(H, D, Dv))
    v = torch.randn(T, H, Dv)
    rows[:, 0], rows[:, D] = 1.0, 2.0                      # both heads' queries ask for key channel 0
    rows[far, H * D], rows[far, H * D + D] = 4.0, 8.0
    rows[:, 2 * H * D:2 * H * D + H * Dv] = v.reshape(T, -1)
    decay = torch.tensor([[1023.0 / 1024.0, 0.99]]).repeat_interleave(D, dim=1).to(DEV)
    for cuts in ([0, T], [0, 18, 19, 150, T]):
        state = torch.zeros((2, H, D, Dv), dtype=torch.float32, device=DEV)
        got = []
        for lo, hi in zip(cuts, cuts[1:]):
            o = torch.empty((hi - lo, H * Dv), dtype=torch.float32, device=DEV)
            ops.gla_scan(rows[lo:hi].to(DEV), 0, H * D, 2 * H * D, decay, o, state, ints([0, hi - lo]), ints([1]), 1, H, D, Dv, 1.0)
            got.append(o.cpu())
        got = torch.cat(got).view(T, H, Dv)
        assert float(got[:far].abs().max()) == 0.0 and float(state[0].abs().max()) == 0.0
        for t in (far, far + 1, 200, T - 1):
            close(got[t, 0], 4.0 * v[far, 0] * (1023.0 / 1024.0) ** (t - far), torch.float32, f"head 0, token {t}")
            close(got[t, 1], 16.0 * v[far, 1] * 0.99 ** (t - far), torch.float32, f"head 1, token {t}")


@pytest.mark.parametrize("dt", DTS)
@pytest.mark.parametrize("H,G_,D,Dv,taps,ranks", [(4, 2, 12, 20, 4, (5, 7)), (2, 2, 64, 48, 2, (16, 16)), (6, 3, 32, 16, 3, (24, 8)),
                                                  (2, 1, 160, 24, 5, (9, 33)), (3, 1, 20, 12, 1, (1, 2)), (4, 4, 128, 64, 4, (128, 64))])
def test_delta_rule_with_a_decay_per_channel_whole_in_portions_token_by_token_and_beside_another(dt, H, G_, D, Dv, taps, ranks):
    from tokenmill_amd.parts import GatedDeltaRule
    mixer = GatedDeltaRule(64, H, G_, D, Dv, taps, 1e-5, channel_decay=True, narrow_gate=True)
    g = torch.Generator().manual_seed(D)
    narrow = {"a1": (ranks[0], 64), "a2": (H * D, ranks[0]), "g1": (ranks[1], 64), "g2": (H * Dv, ranks[1])}
    fixed = {k: torch.randn(s, generator=g) * 0.3 for k, s in narrow.items()}
    fixed["A_log"] = torch.rand(H, generator=g) * 5 - 5    # decays from a few tokens to hundreds
    w = _weights(mixer, dt, 0.25, H * 7 + D, **fixed)
    m = {"heads": H, "kv_heads": G_, "dim": D, "vdim": Dv, "conv": taps}
    T = 300                                                # whole: chunks or (keys of 160) segments; in pieces, scans and chunks
    assert T >= 2 * mixer.SEGMENT > T - 113 and mixer.CHUNKS_FROM <= 40
    torch.manual_seed(D)
    x = q(torch.randn(T, 64), dt)
    want = q(P.delta_rule(x, m, w, "a.", 1e-5, dt), dt)
    pools, manager, runner = _alone(mixer, dt)
    assert len(pools.states) == (2 if taps > 1 else 1) and pools.states[0].dtype == torch.float32
    other = q(torch.randn(60, 64) * 2, dt)
    for cuts in CUTS(T):
        close(_run_cuts(mixer, pools, manager, runner, x, cuts, dt), want, dt, f"cuts {cuts[:4]}..", bf16=2.0 ** -5)
        for t in pools.states.values():
            t.fill_(math.nan)
        close(_run_cuts(mixer, pools, manager, runner, x, cuts, dt, beside=other), want, dt, f"beside another, cuts {cuts[:4]}..", bf16=2.0 ** -5)


@pytest.mark.parametrize("D", [8, 64, 130])
def test_channels_fade_by_their_own_decays(D):
    """The scan alone, on rows made by hand: unit keys, beta = 1. A query for key channel c, tokens later, returns the value last
    written there times that channel's decay for each token since; writing replaces."""
    from tokenmill_amd.hip import ops
    H, G_, Dv, T = 2, 1, 6, 300
    C = 2 * G_ * D + H * Dv
    g = torch.linspace(0.9, 1.0, H * D).view(H, D)
    for ask in (0, 3, 7):
        rows = torch.zeros(T, ops.delta_row_width(H, G_, D, Dv, True))
        v = torch.randn(T, H, Dv)
        for t in range(T):
            rows[t, D + (t % 8)] = 1.0                     # key t % 8
            rows[t, ask] = 1.0
            rows[t, C + 2 * H] = 1.0 if t % 8 == ask else 0.0      # k . q
        rows[:, 2 * D:C] = v.reshape(T, -1)
        rows[:, C:C + H] = 1.0
        rows[:, C + H:C + 2 * H] = math.nan                # the places of a decay per head are not looked at
        rows[:, C + 2 * H + G_:C + 2 * H + G_ + H * D] = g.reshape(-1)
        o = torch.empty((T, H * Dv), dtype=torch.float32, device=DEV)
        state = torch.zeros((2, H, D, Dv), dtype=torch.float32, device=DEV)
        ops.delta_scan(rows.to(DEV), o, state, ints([0, T]), ints([1]), 1, H, G_, D, Dv, per_channel=True)
        got = o.cpu().view(T, H, Dv)
        for t in (ask, ask + 1, ask + 7, ask + 8, 299):
            last = t - (t - ask) % 8
            for h in range(H):
                close(got[t, h], v[last, h] * g[h, ask] ** (t - last), torch.float32, f"channel {ask}, head {h}, token {t}")
        assert float(state[0].abs().max()) == 0.0


def _delta_rows(T, H, G_, D, Dv, per_channel, g, decays):
    """Rows as the recurrence takes them, made by hand: unit keys (some of them equal to the one before), decays drawn from
    ``decays``."""
    from tokenmill_amd.hip import ops
    C = 2 * G_ * D + H * Dv
    rows = torch.zeros(T, ops.delta_row_width(H, G_, D, Dv, per_channel))
    qk = torch.randn(2, T, G_, D, generator=g)
    qk[1, 3::7] = qk[1, 2:-1:7][:qk[1, 3::7].shape[0]]
    qk = qk / qk.norm(dim=-1, keepdim=True)
    rows[:, :G_ * D], rows[:, G_ * D:2 * G_ * D] = qk[0].reshape(T, -1), qk[1].reshape(T, -1)
    rows[:, 2 * G_ * D:C] = torch.randn(T, H * Dv, generator=g)
    rows[:, C:C + H] = torch.rand(T, H, generator=g)
    rows[::5, C:C + H] = 1.0
    pool = torch.tensor(decays)
    if per_channel:
        rows[:, C + 2 * H + G_:C + 2 * H + G_ + H * D] = pool[torch.randint(0, len(pool), (T, H * D), generator=g)]
    else:
        rows[:, C + H:C + 2 * H] = pool[torch.randint(0, len(pool), (T, H), generator=g)]
    rows[:, C + 2 * H:C + 2 * H + G_] = (qk[0] * qk[1]).sum(-1)
    return rows


LENGTHS = [1, 64, 200, 65, 33, 128, 17]


def _chunk_table(lengths):
    cu, first, row = [0], [0], 0
    for n in lengths:
        for lo in range(0, n, 64):
            row += min(64, n - lo)
            cu.append(row)
        first.append(len(cu) - 1)
    return ints(cu), ints(first), len(cu) - 1


@pytest.mark.parametrize("per_channel", [True, False])
@pytest.mark.parametrize("H,G_,D,Dv", [(2, 1, 8, 6), (4, 2, 64, 48), (2, 2, 100, 130), (3, 1, 128, 16), (8, 4, 128, 128)])
def test_delta_rule_in_chunks_is_the_scan(H, G_, D, Dv, per_channel):
    """Portions of ragged lengths from states that are not zero: the chunks' products give the scan's results and states; with
    decays that hardly forget, that forget at once, that underflow when they are multiplied, and that are zero."""
    from tokenmill_amd.hip import ops
    g = torch.Generator().manual_seed(D + Dv)
    T, S = sum(LENGTHS), len(LENGTHS)
    for decays in ([0.999, 0.9, 1.0], [0.5, 1e-6, 1e-30, 0.0, 1.0], [0.02, 0.05]):
        rows = _delta_rows(T, H, G_, D, Dv, per_channel, g, decays).to(DEV)
        start = torch.randn(S + 1, H, D, Dv, generator=g).to(DEV)
        slots = torch.randperm(S, generator=g).to(torch.int32).to(DEV)
        want_o, got_o = torch.empty((T, H * Dv), device=DEV), torch.full((T, H * Dv), math.nan, device=DEV)
        want_s, got_s = start.clone(), start.clone()
        ops.delta_scan(rows, want_o, want_s, ints([sum(LENGTHS[:i]) for i in range(S + 1)]), slots, S, H, G_, D, Dv, per_channel=per_channel)
        cu, first, n = _chunk_table(LENGTHS)
        ops.delta_chunk_scan(rows, got_o, got_s, cu, first, n, slots, S, H, G_, D, Dv, per_channel)
        close(got_o.cpu(), want_o.cpu(), torch.float32, f"results, decays {decays}")
        close(got_s.cpu(), want_s.cpu(), torch.float32, f"states, decays {decays}")
        assert torch.equal(got_s[S], start[S]), "a slot of nobody's"


@pytest.mark.parametrize("H,D,Dv", [(1, 8, 6), (3, 64, 40), (2, 100, 130), (4, 128, 256)])
def test_retention_in_chunks_is_the_scan(H, D, Dv):
    from tokenmill_amd.hip import ops
    g = torch.Generator().manual_seed(D + Dv)
    T, S = sum(LENGTHS), len(LENGTHS)
    rows = (torch.randn(T, ops.retention_row_width(H, D, Dv), generator=g) * 0.3).to(DEV)
    decay = torch.tensor([0.9990234375, 0.5, 1.0, 0.03][:H]).repeat_interleave(D)[None].contiguous().to(DEV)
    start = torch.randn(S + 1, H, D, Dv, generator=g).to(DEV)
    slots = torch.randperm(S, generator=g).to(torch.int32).to(DEV)
    want_o, got_o = torch.empty((T, H * Dv), device=DEV), torch.full((T, H * Dv), math.nan, device=DEV)
    want_s, got_s = start.clone(), start.clone()
    ops.gla_scan(rows, 0, H * D, 2 * H * D, decay, want_o, want_s, ints([sum(LENGTHS[:i]) for i in range(S + 1)]), slots, S, H, D, Dv, 1.0)
    cu, first, n = _chunk_table(LENGTHS)
    ops.retention_chunk_scan(rows, decay, got_o, got_s, cu, first, n, slots, S, H, D, Dv)
    close(got_o.cpu(), want_o.cpu(), torch.float32, "results")
    close(got_s.cpu(), want_s.cpu(), torch.float32, "states")
    assert torch.equal(got_s[S], start[S]), "a slot of nobody's"


@pytest.mark.parametrize("dt", DTS)
@pytest.mark.parametrize("channel", [True, False])
@pytest.mark.parametrize("H,G_,D,Dv,taps", [(4, 2, 12, 20, 4), (2, 2, 64, 48, 2), (6, 3, 128, 128, 3), (2, 1, 160, 24, 5), (3, 1, 20, 12, 1), (16, 2, 32, 70, 7)])
def test_a_single_token_in_one_launch_is_the_same_token_step_by_step(dt, channel, H, G_, D, Dv, taps):
    """Convolution, norms, decays, recurrence, convolution state and gate as one kernel against the kernels one by one."""
    from tokenmill_amd.hip import ops
    assert ops.delta_step_takes(H, G_, D, Dv)
    g = torch.Generator().manual_seed(D + Dv)
    n, C = 5, 2 * G_ * D + H * Dv
    rnd = lambda *shape: torch.randn(*shape, generator=g)      # noqa: E731
    proj, gate = rnd(n, C + 3).to(dt).to(DEV), rnd(n, H * Dv + 1).to(dt).to(DEV)
    conv_w = (rnd(C, taps) * 0.5).to(dt).to(DEV)
    conv_state = rnd(n + 2, taps - 1, C).to(dt).to(DEV) if taps > 1 else None
    ba, z = rnd(n, 2 * H).to(DEV), rnd(n, H * D).to(DEV) if channel else None
    a_log, dt_bias, norm_w = (rnd(H) - 1).to(DEV), rnd(H * D if channel else H).to(DEV), (torch.rand(Dv, generator=g) + 0.5).to(DEV)
    state = rnd(n + 2, H, D, Dv).to(DEV)
    slots = ints([4, 0, 6, 1, 3])
    cu, seqs = ints(list(range(n + 1))), ints(list(range(n)))
    s1, c1 = state.clone(), conv_state.clone() if taps > 1 else None
    rows = torch.empty((n, ops.delta_row_width(H, G_, D, Dv, channel)), device=DEV)
    o, want = torch.empty((n, H * Dv), device=DEV), torch.empty((n, H * Dv), dtype=dt, device=DEV)
    ops.delta_prepare(proj, conv_w, c1, ba, a_log, dt_bias, cu, slots, seqs, n, rows, H, G_, D, Dv, 1e-6, z=z)
    if taps > 1:
        ops.delta_conv_state(proj, C, c1, cu, slots, n)
    ops.delta_scan(rows, o, s1, cu, slots, n, H, G_, D, Dv, per_channel=channel)
    ops.gla_out_gate(o, gate, norm_w, want, H, Dv, 1e-5, sigmoid=channel)
    s2, c2, got = state.clone(), conv_state.clone() if taps > 1 else None, torch.full((n, H * Dv), math.nan, dtype=dt, device=DEV)
    ops.delta_step(proj, conv_w, c2, ba, z, a_log, dt_bias, gate, norm_w, s2, slots, got, H, G_, D, Dv, 1e-6, 1e-5, channel)
    close(got.float().cpu(), want.float().cpu(), dt, "result", bf16=2.0 ** -7)
    close(s2.cpu(), s1.cpu(), torch.float32, "state")
    assert taps == 1 or torch.equal(c2, c1), "convolution state"


@pytest.mark.parametrize("dt", DTS)
@pytest.mark.parametrize("H,D,Dv,rot", [(3, 20, 12, 8), (2, 64, 70, 64), (1, 160, 24, 0), (4, 128, 256, 32), (2, 30, 600, 30)])
def test_a_single_token_of_a_retention_in_one_launch(dt, H, D, Dv, rot):
    from tokenmill_amd.hip import ops
    from tokenmill_amd.parts import RotaryEmbedding
    g = torch.Generator().manual_seed(D + Dv)
    n = 5
    proj = torch.randn(n, 2 * H * (D + Dv), generator=g).to(dt).to(DEV)
    table = None
    if rot:
        table = RotaryEmbedding(D, 1e4, 300, rotary_dim=rot, exact=True)
        table.build_tables(DEV)
    cos, sin = (table.cos, table.sin) if rot else (None, None)
    places, slots = ints([0, 7, 299, 64, 1]), ints([4, 0, 6, 1, 3])
    decay = torch.tensor([0.999, 0.9, 0.5, 0.97][:H]).repeat_interleave(D)[None].contiguous().to(DEV)
    state = torch.randn(n + 2, H, D, Dv, generator=g).to(DEV)
    s1, s2 = state.clone(), state.clone()
    rows, o = torch.empty((n, ops.retention_row_width(H, D, Dv)), device=DEV), torch.empty((n, H * Dv), device=DEV)
    want, got = torch.empty((n, H * Dv), dtype=dt, device=DEV), torch.full((n, H * Dv), math.nan, dtype=dt, device=DEV)
    ops.retention_prepare(proj, cos, sin, places, rows, H, D, Dv, D ** -0.5)
    ops.gla_scan(rows, 0, H * D, 2 * H * D, decay, o, s1, ints(list(range(n + 1))), slots, n, H, D, Dv, 1.0)
    ops.gla_out_gate(o, proj[:, H * (2 * D + Dv):], None, want, H, Dv, 1e-5)
    ops.retention_step(proj, cos, sin, places, decay, s2, slots, got, H, D, Dv, D ** -0.5, 1e-5)
    close(got.float().cpu(), want.float().cpu(), dt, "result", bf16=2.0 ** -7)
    close(s2.cpu(), s1.cpu(), torch.float32, "state")


@pytest.mark.parametrize("dt", DTS)
def test_two_mixers_added_with_constant_weights(dt):
    from tokenmill_amd.parts import ParallelMixer, Retention
    left, right = Retention(64, 2, 16, 16, [0.9, 0.8], 1e-5), Retention(64, 1, 32, 8, [0.7], 1e-5)
    right.cache_spec = lambda: None                        # the state of one mixer a layer
    left_only = ParallelMixer(64, left, right, scales=(0.7, -1.3))
    assert not [k for k in left_only.tensor_specs("") if "out" in k]
    a, b = q(torch.randn(5, 64), dt).to(dt).to(DEV), q(torch.randn(5, 64), dt).to(dt).to(DEV)
    left_only._both = lambda x, step, cache: (a, b)
    parts = left_only.forward_parts(a, None, None)
    assert [s for _, s in parts] == [0.7, -1.3] and parts[0][0] is a and parts[1][0] is b
    close(left_only.forward(a, None, None).float().cpu(), q(0.7 * a.float().cpu() - 1.3 * b.float().cpu(), dt), dt, "their sum", bf16=2.0 ** -8)


# ----------------------------------------------------------------------------------------------- whole models

@pytest.fixture(scope="module")
def models(tmp_path_factory):
    """name -> (folder, config, plain weights)."""
    from safetensors.torch import load_file, save_file
    from tokenmill_amd.weights.random_init import write_random_model
    out = {}
    for name, (cfg, seed, std, norm_std) in CASES.items():
        d = tmp_path_factory.mktemp(f"kasovik{name}")
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
    """float32: 5e-5 of the largest logit, every row. bfloat16: the model's floor is the largest distance of the plain bfloat16
    run from the plain float32 run over the requests at hand, and the engine may be twice as far from the plain bfloat16 run
    (both differ from the 32-bit run by the same roundings, falling differently). One row in a hundred may be up to four times
    further: where a recurrence's read-out is next to nothing, the norms behind it blow the roundings of the layers before up
    for that one token, in the plain run as in the engine."""
    assert got, "no rows"
    if dt == torch.float32:
        for (rid, p), row in sorted(got.items()):
            want = plain_logits(models, name, reqs[rid], dt)
            err = float((row - want[p]).abs().max())
            bound = 2.5 * F32_REL * float(want.abs().max())
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
    layers = CASES[name][0]["layers"]
    assert len(s.pools.views) == len(layers) + 1 and s.pools.views[-1].state.dtype == torch.int32
    poison_freed_pages(s)
    slots, pools, release = s.manager.slots, s.pools, s.manager.slots.release

    def poisoned(slot):
        for t in pools.states.values():
            t[slot].fill_(math.nan if t.is_floating_point() else 5)
        return release(slot)
    slots.release = poisoned
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
def test_a_token_far_back_decides_the_logits_through_a_recurrence(models, dtype_name):
    """Weights made so that it shows. Hidden channel 0 is zero in every embedding row but one token's, channel 1 is the same
    constant in all; the first layer's key projection reads channel 0 into one key channel of a head that hardly forgets, and
    its query projection reads channel 1 there. Hundreds of tokens later every query still points at the ONE token, and the
    logits follow the plain implementation's only if the state carries it, through prompts, portions and decoded tokens."""
    from safetensors.torch import save_file
    from tokenmill_amd.replay import ReplaySession
    from test_gpu_replay import portions, prefill_then_decode, run_trace, whole
    dt = {"float32": torch.float32, "bfloat16": torch.bfloat16}[dtype_name]
    d, cfg, w = models["A"]
    w2 = {k: v.clone() for k, v in w.items()}
    far_id, m = 7, cfg["layers"][0]["mixer"]
    D = m["dim"]
    emb, big = w["embed"].float().clone(), w["bigram"].float().clone()
    emb[:, 0], emb[:, 1], big[:, 0], big[:, 1] = 0.0, 1.0, 0.0, 0.0
    emb[far_id, 0] = 8.0
    qw, kw = w["l0.mix.q"].float().clone() * 0.1, w["l0.mix.k"].float().clone() * 0.02
    at = D + D - 1                                         # head 1 (decay 0.995), a channel behind the rotated ones
    qw[at] = 0.0
    qw[at, 1] = 6.0
    kw[at] = 0.0
    kw[at, 0] = 6.0
    w2["embed"], w2["bigram"], w2["l0.mix.q"], w2["l0.mix.k"] = (t.to(torch.bfloat16) for t in (emb, big, qw, kw))
    folder = d.parent / f"kasovik_far_{dtype_name}"
    folder.mkdir(exist_ok=True)
    (folder / "config.json").write_text(json.dumps(cfg))
    save_file(w2, str(folder / "model.safetensors"))
    ids = [t if t != far_id else far_id + 1 for t in random_ids(420, cfg["vocab"], 9)]
    ids[5] = far_id
    local = {"A": (folder, cfg, w2)}
    with_far = P.forward(ids, cfg, w2, torch.float32)
    swapped = list(ids)
    swapped[5] = far_id + 1
    without = P.forward(swapped, cfg, w2, torch.float32)
    moved = float((with_far[-40:] - without[-40:]).abs().max()) / float(with_far.abs().max())
    assert moved > 0.02, f"the far token moves the last logits by {moved:.3g} of their size only: the test would not show a lost state"
    s = ReplaySession(folder, dtype_name, 448, max_requests=4, page_size=16)
    for steps, what in ((whole({"a": ids}), "whole"), (prefill_then_decode({"a": ids}, tail=48), "decoded"), (portions({"a": ids}), "portions")):
        check_rows(local, "A", run_trace(s, steps), {"a": ids}, dt, f"far token, {what}")


@pytest.mark.parametrize("dtype_name", ["float32", "bfloat16"])
def test_long_decoding_over_many_page_borders(models, dtype_name):
    """One token at a time from the third token on: every page border and every window is passed by decoded tokens and both
    recurrences' states are carried over 250 steps, two requests beside each other that start at different times."""
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
    pages that fall behind the windows; its logits differ by rounding at most."""
    from tokenmill_amd.replay import ReplaySession
    from test_gpu_replay import assert_all_given_back, run_trace
    dt = {"float32": torch.float32, "bfloat16": torch.bfloat16}[dtype_name]
    reqs = make_requests("B", [200, 31, 90, 64], 7)
    rows = {}
    for who in (["r0"], list(reqs)):
        s = ReplaySession(models["B"][0], dtype_name, 512, max_requests=4, page_size=16)
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
        got = run_trace(s, steps)
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
        assert kinds.count("Retention") == 2 and kinds.count("ParallelMixer") == 3 and kinds.count("TokenEmbedding") == 1
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


def test_command_line_generates_with_a_random_kasovik_model(tmp_path):
    import subprocess
    import sys
    from conftest import ROOT
    (tmp_path / "config.json").write_text(json.dumps(B))
    r = subprocess.run([sys.executable, "-m", "tokenmill_amd.generate", "--random", str(tmp_path / "config.json"), "--prompt-ids",
                        "5,9,33,2;7,7", "--max-tokens", "6", "--max-model-len", "64", "--ignore-eos"], capture_output=True, text=True, cwd=ROOT, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    lines = [json.loads(ln) for ln in r.stdout.splitlines() if ln.startswith("{")]
    assert [len(ln["output_ids"]) for ln in lines] == [6, 6] and all(0 <= t < 150 for ln in lines for t in ln["output_ids"])
