"""Kasovik without a GPU: configuration, tensor declarations, what the layers ask of the cache manager, and the plain
implementation's mechanisms pinned against special cases that reduce to something known."""
from __future__ import annotations

import copy
import math

import pytest
import torch

from kasovik_cases import A, B, C, lively
from plain import kasovik_plain as P


def _random_model(cfg, seed, std=0.1, norm_std=0.1):
    from tokenmill_amd.config.model_config import KasovikConfig
    from tokenmill_amd.models.kasovik import build_kasovik
    from tokenmill_amd.weights.random_init import random_tensors
    return lively(cfg, dict(random_tensors(build_kasovik(KasovikConfig.from_dict(cfg), 64).tensor_specs(), seed=seed, std=std, norm_std=norm_std)), seed)


# ----------------------------------------------------------------------------------------------- configuration

def test_config_reads_every_size_and_constant():
    from tokenmill_amd.config.model_config import KasovikConfig
    from tokenmill_amd.config.registry import architecture_name, get_architecture
    assert architecture_name(A) == "Kasovik" and get_architecture("Kasovik").name == "Kasovik"
    cfg = KasovikConfig.from_dict(A)
    assert (cfg.vocab_size, cfg.hidden_size, cfg.norm_eps, cfg.embedding_scale, cfg.max_position_embeddings) == (211, 88, 3e-5, 2.5, None)
    assert (cfg.pair_buckets, cfg.pair_mul_prev, cfg.pair_mul_cur) == (37, 19, 3)
    assert [l.type for l in cfg.layers] == ["retention", "parallel", "parallel", "retention", "parallel"]
    assert [l.weights_of for l in cfg.layers] == [None, None, 1, 0, None]
    assert cfg.layers[0].mlp == {"ff": 56, "limit": 1.2} and cfg.layers[1].mlp is None
    assert cfg.layers[1].mixer["left"]["mask"] == {"size": 9} and cfg.layers[4].mixer["right"]["conv"] == 1
    limited = dict(copy.deepcopy(C), max_positions=77)
    assert KasovikConfig.from_dict(limited).max_position_embeddings == 77
    chained = copy.deepcopy(C)
    chained["layers"][3]["weights_of"] = 1                 # layer 1 itself runs layer 0's tensors
    assert KasovikConfig.from_dict(chained).layers[3].weights_of == 0


@pytest.mark.parametrize("edit,match", [
    (lambda c: c.pop("norm"), "norm"),
    (lambda c: c.pop("width"), "width"),
    (lambda c: c["embedding"].pop("bigram"), "bigram"),
    (lambda c: c["embedding"]["bigram"].pop("mul_prev"), "mul_prev"),
    (lambda c: c["embedding"]["bigram"].update(buckets=0), "buckets"),
    (lambda c: c["embedding"]["bigram"].update(mul_cur=1 << 31), "mul_cur"),
    (lambda c: c["layers"][0].update(type="attention"), "type"),
    (lambda c: c["layers"][0]["mixer"].pop("decay"), "decay"),
    (lambda c: c["layers"][0]["mixer"].update(heads=2), "decays"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=22), "rot.dims"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7), "rot.dims"),
    (lambda c: c["layers"][1]["mixer"].pop("right"), "left' and 'right"),
    (lambda c: c["layers"][1]["mixer"].pop("left_scale"), "left_scale"),
    (lambda c: c["layers"][1]["mixer"]["left"].update(kv_heads=4), "kv_heads"),
    (lambda c: c["layers"][1]["mixer"]["left"].update(vdim=24), "vdim"),
    (lambda c: c["layers"][1]["mixer"]["left"]["mask"].update(size=0), "mask.size"),
    (lambda c: c["layers"][1]["mixer"]["right"].update(kv_heads=3), "kv_heads"),
    (lambda c: c["layers"][1]["mixer"]["right"].update(conv=0), "conv"),
    (lambda c: c["layers"][2].update(weights_of=2), "weights_of"),
    (lambda c: c["layers"][2].update(weights_of=0), "equal"),
    (lambda c: c["layers"][4]["mlp"].pop("limit"), "limit"),
    (lambda c: c["layers"][4]["mlp"].update(limit=0.0), "limit"),
    (lambda c: c["layers"][4]["mlp"].update(kind="moe"), "kind"),
])
def test_config_refuses_what_the_model_cannot_be(edit, match):
    from tokenmill_amd.config import ConfigError
    from tokenmill_amd.config.model_config import KasovikConfig
    raw = copy.deepcopy(A)
    edit(raw)
    with pytest.raises(ConfigError, match=match):
        KasovikConfig.from_dict(raw)


def test_tensor_names_shapes_and_caches():
    from tokenmill_amd.config.model_config import KasovikConfig
    from tokenmill_amd.models.kasovik import build_kasovik
    from tokenmill_amd.parts import KVCacheSpec, LayerCacheSpec, StateSpec
    model = build_kasovik(KasovikConfig.from_dict(A), 64)
    specs = {k: tuple(v.drawn_shape()) for k, v in model.tensor_specs().items()}
    assert specs["embed"] == (211, 88) and specs["bigram"] == (38, 88) and specs["final.norm"] == (88,) and "head" not in specs
    assert specs["l0.norm1"] == (88,) and "l0.norm2" not in specs
    assert specs["l0.mix.q"] == (60, 88) and specs["l0.mix.v"] == (36, 88) and specs["l0.mix.g"] == (36, 88) and specs["l0.mix.o"] == (88, 36)
    assert specs["l0.mlp.gate"] == (56, 88) and specs["l0.mlp.gate.b"] == (56,) and specs["l0.mlp.down.b"] == (88,)
    assert specs["l1.mix.left.q"] == (120, 88) and specs["l1.mix.left.k"] == (40, 88) and specs["l1.mix.left.sink"] == (6,)
    assert "l1.mix.left.v" not in specs and "l1.mix.left.q.norm" not in specs and "l1.mix.left.q.b" not in specs and "l1.mix.left.out" not in specs
    assert specs["l1.mix.right.q"] == (24, 88) and specs["l1.mix.right.v.conv"] == (80, 4) and specs["l1.mix.right.b"] == (4, 88)
    assert specs["l1.mix.right.A_log"] == (4,) and specs["l1.mix.right.dt_bias"] == (48,) and specs["l1.mix.right.norm"] == (20,)
    assert specs["l1.mix.right.a1"][1] == 88 and specs["l1.mix.right.a2"][0] == 48 and specs["l1.mix.right.g2"][0] == 80
    assert "l1.mix.right.a" not in specs and "l1.mix.right.g" not in specs and "l1.mlp.gate" not in specs
    assert not [k for k in specs if k.startswith(("l2.", "l3."))] and specs["l4.mlp.up"] == (30, 88)        # layers 2 and 3 have no tensors of their own
    assert len(model.layers) == 3 and [c.layer for c in model.run] == [0, 1, 1, 0, 2] and all(c.cache_of is None for c in model.run)
    caches = model.cache_specs()
    assert len(caches) == 6 and caches[5] == StateSpec((1,), torch.int32)              # the last: the embedding's token before
    assert caches[0] == StateSpec((3, 20, 12), torch.float32) and caches[3] == caches[0]
    assert isinstance(caches[1], LayerCacheSpec) and caches[1].kv == KVCacheSpec(2, 20, 9, v_head_dim=20) and caches[2] == caches[1]
    assert [tuple(s.shape) for s in caches[1].state] == [(4, 12, 20), (3, 128)] and caches[1].state[0].dtype == torch.float32
    assert len(caches[4].state) == 1 and caches[4].kv.window == 33                     # one tap: no rows to carry


def test_every_run_of_a_layer_has_a_cache_of_its_own():
    from tokenmill_amd.cache.pool import CachePools
    from tokenmill_amd.config.model_config import KasovikConfig
    from tokenmill_amd.models.kasovik import build_kasovik
    pools = CachePools(build_kasovik(KasovikConfig.from_dict(A), 64), 5, 4, 3, torch.bfloat16, "cpu")
    a, b = pools.views[1], pools.views[2]
    assert a.k.data_ptr() != b.k.data_ptr() and a.group == b.group and a.state[0].data_ptr() != b.state[0].data_ptr()
    assert pools.views[0].state.data_ptr() != pools.views[3].state.data_ptr()
    assert len(pools.views) == 6 and pools.views[5].state.dtype == torch.int32 and tuple(pools.views[5].state.shape) == (4, 1)
    pools.views[5].state.fill_(9)
    pools.reset_state_slot(1)
    assert pools.views[5].state[:, 0].tolist() == [9, 0, 9, 9]


def test_narrow_widths_come_from_the_tensors_and_must_agree():
    from tokenmill_amd.parts import GatedDeltaRule
    part = GatedDeltaRule(24, 2, 1, 8, 6, 2, 1e-5, channel_decay=True, narrow_gate=True)
    shapes = {"q": (8, 24), "k": (8, 24), "v": (12, 24), "b": (2, 24), "o": (24, 12), "a1": (5, 24), "a2": (16, 5), "g1": (7, 24), "g2": (12, 7),
              "q.conv": (8, 2), "k.conv": (8, 2), "v.conv": (12, 2), "A_log": (2,), "dt_bias": (16,), "norm": (6,)}
    t = {f"p.{k}": torch.randn(s) for k, s in shapes.items()}
    assert set(part.tensor_specs("p.")) == set(t)
    part.load(t, "p.")
    assert part.proj.out_features == 8 + 8 + 12 + 5 + 7 and part.gate_at == 33 and part.decay2.in_features == 5 and part.gate2.in_features == 7
    bad = dict(t, **{"p.a2": torch.randn(16, 6)})
    with pytest.raises(ValueError, match="disagree"):
        GatedDeltaRule(24, 2, 1, 8, 6, 2, 1e-5, channel_decay=True, narrow_gate=True).load(bad, "p.")


def test_parts_refuse_what_they_cannot_be():
    from tokenmill_amd.parts import GatedFeedForward, ParallelMixer, Retention, RotaryEmbedding, SoftmaxAttention, TokenEmbedding
    from tokenmill_amd.parts.embedding import LearnedPositions, PairRows
    with pytest.raises(ValueError, match="decays"):
        Retention(16, 2, 8, 8, [0.5], 1e-5)
    with pytest.raises(ValueError, match="apart"):
        Retention(16, 1, 8, 8, [0.5], 1e-5, rotary=RotaryEmbedding(8, 1e4, 8, interleaved=True))
    with pytest.raises(ValueError, match="keys' size"):
        SoftmaxAttention(16, 2, 1, 8, 12, 1.0, keys_are_values=True)
    with pytest.raises(ValueError, match="limit"):
        GatedFeedForward(16, 8, "clamped_glu")
    with pytest.raises(ValueError, match="limit"):
        GatedFeedForward(16, 8, "silu", limit=1.0)
    with pytest.raises(ValueError, match="either"):
        ParallelMixer(16, Retention(16, 1, 8, 8, [0.5], 1e-5), Retention(16, 1, 8, 8, [0.5], 1e-5))
    with pytest.raises(ValueError, match="pairs"):
        TokenEmbedding(5, 4, places=LearnedPositions(8, 4), pairs=PairRows(3, 4, 1, 1))


def test_random_weights_round_trip(tmp_path):
    from safetensors.torch import load_file
    from tokenmill_amd.weights.random_init import write_random_model
    write_random_model(B, tmp_path, seed=3)
    w = load_file(str(tmp_path / "model.safetensors"))
    assert w["l0.mix.right.q.conv"].shape == (128, 2) and w["l2.mix.left.sink"].shape == (6,) and w["bigram"].shape == (65, 128)
    assert torch.isfinite(P.forward([3, 1, 4, 1, 5, 9, 2, 6], B, w)).all()


# ----------------------------------------------------------------------------------------------- the plain mechanisms

def test_rows_of_pairs_depend_on_both_tokens_and_their_order():
    t = {"embed": torch.zeros(211, 38), "bigram": torch.eye(38)}
    rows = P.embed(torch.tensor([4, 9, 4, 9]), A, t).argmax(-1).tolist()
    assert rows == [37, (4 * 19 + 9 * 3) % 37, (9 * 19 + 4 * 3) % 37, (4 * 19 + 9 * 3) % 37]
    t["embed"] = torch.ones(211, 38)
    assert torch.equal(P.embed(torch.tensor([4]), A, t), 2.5 + torch.eye(38)[37:])     # the row of the pair is not scaled


def test_a_retention_is_the_decayed_sum_over_all_tokens():
    torch.manual_seed(0)
    T, H, D, Dv = 9, 2, 4, 3
    q, k, v = torch.randn(T, H, D), torch.randn(T, H, D), torch.randn(T, H, Dv)
    decay = torch.tensor([0.5, 0.9])
    o = P.retention_scan(q, k, v, decay)
    for t in (0, 3, 8):
        for h in range(H):
            want = sum(decay[h] ** (t - j) * (q[t, h] @ k[j, h]) * v[j, h] for j in range(t + 1))
            assert torch.allclose(o[t, h], want, atol=1e-5)


def test_window_and_sink():
    T, D = 7, 3
    qk = torch.zeros(T, 2, D)                              # every score is zero
    v = torch.arange(T, dtype=torch.float32)[:, None, None].expand(T, 2, 1)
    sink = torch.tensor([0.0, math.log(3.0)])
    out = P.window_attention(qk, qk, v, 5.0, 3, sink)
    for p in range(T):
        seen = range(max(0, p - 2), p + 1)                 # itself and the two before it
        assert math.isclose(float(out[p, 0, 0]), sum(seen) / (len(seen) + 1), rel_tol=1e-6)
        assert math.isclose(float(out[p, 1, 0]), sum(seen) / (len(seen) + 3), rel_tol=1e-6)
    every = P.window_attention(qk, qk, v, 5.0, None, sink)
    assert math.isclose(float(every[6, 0, 0]), 21 / 8, rel_tol=1e-6)


def test_values_are_the_keys_before_their_norm():
    m = {"heads": 1, "kv_heads": 1, "dim": 4, "vdim": 4, "scale": 1.0, "mask": {"size": 1}}
    t = {"q": torch.eye(4), "k": 3.0 * torch.eye(4), "sink": torch.full((1,), -100.0), "o": torch.eye(4)}
    h = torch.tensor([[1.0, 2.0, -1.0, 0.5]])
    assert torch.allclose(P.key_value_attention(h, m, t, "", 1e-6, torch.float32), 3.0 * h)      # one key: its value, as projected
    t["sink"] = torch.zeros(1)
    score = float((P.unit(h, 1e-6) * P.unit(3 * h, 1e-6)).sum())
    assert math.isclose(score, 4.0, rel_tol=1e-5)                                                # unit RMS vectors of four channels
    assert torch.allclose(P.key_value_attention(h, m, t, "", 1e-6, torch.float32), 3.0 * h / (1 + math.exp(-score)), rtol=1e-5)


def test_the_delta_rule_decays_channel_by_channel_before_it_reads():
    T, D, Dv = 3, 2, 2
    e = torch.eye(2)
    k = torch.stack([e[0], e[1], e[1]]).view(T, 1, D)
    q = torch.stack([e[0], e[0], e[0] + e[1]]).view(T, 1, D)
    v = torch.tensor([[1.0, 2.0], [3.0, 4.0], [5.0, 6.0]]).view(T, 1, Dv)
    g = torch.tensor([0.5, 0.25]).expand(T, 1, 2)
    o = P.delta_scan(q, k, v, g, torch.ones(T, 1))
    assert torch.allclose(o[0, 0], v[0, 0])                                           # the read-out sees the token's own write
    assert torch.allclose(o[1, 0], 0.5 * v[0, 0])                                     # channel 0 fades by its own decay
    assert torch.allclose(o[2, 0], 0.25 * v[0, 0] + v[2, 0])                          # channel 1 was replaced, not added to
    half = P.delta_scan(q, k, v, g, torch.full((T, 1), 0.5))
    s1 = 0.5 * v[1, 0]
    assert torch.allclose(half[2, 0], 0.25 * 0.5 * v[0, 0] + 0.25 * s1 + 0.5 * (v[2, 0] - 0.25 * s1))   # the correction is taken on the decayed state


def test_decays_lie_between_zero_and_one_and_follow_their_head():
    z = torch.zeros(1, 4)
    g = P.channel_decay(z, torch.tensor([0.0, math.log(2.0)]), torch.tensor([0.0, 50.0, 0.0, -50.0]), 2)[0]
    assert math.isclose(float(g[0, 0]), 0.5, rel_tol=1e-6) and math.isclose(float(g[1, 0]), 0.25, rel_tol=1e-6)
    assert float(g[0, 1]) < 1e-20 and math.isclose(float(g[1, 1]), 1.0, rel_tol=1e-6)


def test_clamped_gate():
    g, u = torch.tensor([0.0, 3.0, -9.0, 1.0]), torch.tensor([5.0, -5.0, 0.0, 0.5])
    y = P.clamped_glu(g, u, 2.0)
    sig = lambda x: 1 / (1 + math.exp(-1.702 * x))     # noqa: E731
    want = [0.0, 2.0 * sig(2.0) * (-2.0 + 1), -9.0 * sig(-9.0), 1.0 * sig(1.0) * 1.5]      # the gate has no lower limit
    assert torch.allclose(y, torch.tensor(want), atol=1e-6)


def test_both_sublayers_read_the_same_norm():
    w = _random_model(A, 5)
    shut = {k: (torch.zeros_like(v) if k.endswith((".o", ".down", ".down.b")) else v) for k, v in w.items()}
    ids = torch.tensor([4, 9, 2])
    x = P.embed(ids, A, w)
    head = lambda v: P.rms(v, w["final.norm"], 3e-5) @ w["embed"].float().T      # noqa: E731
    assert torch.allclose(P.forward(ids, A, shut), head(x), atol=1e-5)
    one = dict(shut, **{k: w[k] for k in ("l0.mix.o", "l0.mlp.down", "l0.mlp.down.b")})
    cfg = dict(A, layers=A["layers"][:1])
    h = P.rms(x, w["l0.norm1"], 3e-5)
    add = P.retention(h, A["layers"][0]["mixer"], w, "l0.mix.", 3e-5, torch.arange(3), torch.float32) + \
        P.feed_forward(h, A["layers"][0]["mlp"], w, "l0.mlp.", torch.float32)
    assert torch.allclose(P.forward(ids, cfg, one), head(x + add), atol=1e-5)


@pytest.mark.parametrize("cfg", [A, B, C])
def test_a_later_token_never_changes_an_earlier_row(cfg):
    w = _random_model(cfg, 6)
    ids = torch.tensor([3, 1, 4, 1, 5, 9, 2, 6, 5, 3, 5, 8])
    whole = P.forward(ids, cfg, w)
    assert torch.allclose(P.forward(ids[:7], cfg, w), whole[:7], atol=2e-5)
