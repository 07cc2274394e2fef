"""Sanazen without a GPU: configuration, tensor declarations, what the layers ask of the cache manager, kept pages, and the plain
implementation's mechanisms pinned against special cases that reduce to something known."""
from __future__ import annotations

import copy
import math

import pytest
import torch

from plain import sanazen_plain as P
from sanazen_cases import A, B, C, lively


def _model(cfg):
    from tokenmill_amd.config.model_config import SanazenConfig
    from tokenmill_amd.models.sanazen import build_sanazen
    return build_sanazen(SanazenConfig.from_dict(cfg), 64)


def _random_weights(cfg, seed, std=0.1, norm_std=0.1):
    from tokenmill_amd.weights.random_init import random_tensors
    return lively(cfg, dict(random_tensors(_model(cfg).tensor_specs(), seed=seed, std=std, norm_std=norm_std)), seed)


# ----------------------------------------------------------------------------------------------- configuration

def test_config_reads_every_size_and_constant():
    from tokenmill_amd.config.model_config import SanazenConfig
    from tokenmill_amd.config.registry import architecture_name, get_architecture
    assert architecture_name(A) == "Sanazen" and get_architecture("Sanazen").name == "Sanazen"
    cfg = SanazenConfig.from_dict(A)
    assert (cfg.vocab_size, cfg.hidden_size, cfg.norm_eps, cfg.embedding_scale, cfg.max_position_embeddings) == (211, 88, 3e-5, 2.5, None)
    assert (cfg.logit_scale, cfg.logit_softcap) == (0.7, 5.0)
    assert cfg.layers[0].mlp == {"ff": 28, "limit": 1.2, "experts": 7, "top": 3, "shared": {"ff": 20, "limit": 0.8}} and cfg.layers[1].mlp is None
    assert cfg.layers[0].mixer["left"]["mask"] == {"size": 9, "keep_first": 3} and cfg.layers[2].mixer["right"]["decay"] == [0.97]
    cfg = SanazenConfig.from_dict(dict(copy.deepcopy(B), max_positions=77))
    assert cfg.max_position_embeddings == 77 and cfg.logit_softcap is None and cfg.layers[1].mlp["shared"] is None


@pytest.mark.parametrize("edit,match", [
    (lambda c: c.pop("norm"), "norm"),
    (lambda c: c.pop("width"), "width"),
    (lambda c: c["embedding"].pop("scale"), "scale"),
    (lambda c: c["norm"].update(eps=0.0), "eps"),
    (lambda c: c.update(logit_softcap=-1.0), "softcap"),
    (lambda c: c["layers"][0].update(type="attention"), "type"),
    (lambda c: c["layers"][0]["mixer"].pop("right"), "left' and 'right"),
    (lambda c: c["layers"][0]["mixer"].pop("left_scale"), "left_scale"),
    (lambda c: c["layers"][0]["mixer"]["left"].pop("conv"), "conv"),
    (lambda c: c["layers"][0]["mixer"]["left"].update(conv=0), "conv"),
    (lambda c: c["layers"][0]["mixer"]["left"].update(kv_heads=4), "kv_heads"),
    (lambda c: c["layers"][0]["mixer"]["left"]["mask"].update(size=0), "mask.size"),
    (lambda c: c["layers"][0]["mixer"]["left"]["mask"].update(keep_first=-1), "keep_first"),
    (lambda c: c["layers"][0]["mixer"]["right"].pop("decay"), "decay"),
    (lambda c: c["layers"][0]["mixer"]["right"].update(heads=2), "decays"),
    (lambda c: c["layers"][0]["mixer"]["right"].update(dim=0), "right.dim"),
    (lambda c: c["layers"][0]["mlp"].update(kind="dense"), "kind"),
    (lambda c: c["layers"][0]["mlp"]["expert"].pop("limit"), "limit"),
    (lambda c: c["layers"][0]["mlp"]["shared"].pop("limit"), "shared expert"),
    (lambda c: c["layers"][0]["mlp"]["shared"].update(limit=0.0), "limit"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=8), "experts"),
])
def test_config_refuses_what_the_model_cannot_be(edit, match):
    from tokenmill_amd.config import ConfigError
    from tokenmill_amd.config.model_config import SanazenConfig
    raw = copy.deepcopy(A)
    edit(raw)
    with pytest.raises(ConfigError, match=match):
        SanazenConfig.from_dict(raw)


def test_tensor_names_shapes_and_caches():
    from tokenmill_amd.parts import KVCacheSpec, LayerCacheSpec
    model = _model(A)
    specs = {k: tuple(v.drawn_shape()) for k, v in model.tensor_specs().items()}
    assert specs["embed"] == (211, 88) and specs["head"] == (211, 88) and specs["final.norm"] == (88,)
    assert specs["l0.norm1"] == (88,) and specs["l0.norm2"] == (88,) and "l1.norm2" not in specs and model.ignorable == ("l1.norm2",)
    left = {k[12:]: v for k, v in specs.items() if k.startswith("l0.mix.left.")}
    assert left == {"q": (120, 88), "q.b": (120,), "q.norm": (120,), "q.conv": (120, 4), "k": (40, 88), "k.b": (40,), "k.norm": (40,),
                    "k.conv": (40, 4), "v": (24, 88), "v.b": (24,), "v.conv": (24, 4), "g": (72, 88), "o": (88, 72), "o.b": (88,)}
    right = {k[13:]: v for k, v in specs.items() if k.startswith("l0.mix.right.")}
    assert right == {"q": (60, 88), "k": (60, 88), "v": (36, 88), "g": (36, 88), "o": (88, 36), "norm": (36,)}
    mlp = {k[7:]: v for k, v in specs.items() if k.startswith("l0.mlp.") and not k.startswith("l0.mlp.e")}
    assert mlp == {"router": (7, 88), "shared.gate": (20, 88), "shared.up": (20, 88), "shared.down": (88, 20), "shared.sg": (1, 88)}
    assert specs["l0.mlp.e6.gate"] == (28, 88) and specs["l0.mlp.e6.down"] == (88, 28) and "l0.mlp.e7.up" not in specs
    assert not [k for k in specs if k.startswith("l1.mlp")]
    caches = model.cache_specs()
    assert isinstance(caches[0], LayerCacheSpec) and caches[0].kv == KVCacheSpec(2, 20, 9, v_head_dim=12, keep=3)
    assert [(tuple(s.shape), s.dtype) for s in caches[0].state] == [((3, 184), None), ((3, 20, 12), torch.float32)]
    assert (tuple(caches[1].state.shape), caches[1].kv.keep) == ((2, 12, 30), 20)         # one tap: no rows to carry, the recurrence's state alone


def test_each_side_of_a_parallel_mixer_is_handed_its_own_state():
    from tokenmill_amd.cache.pool import CachePools
    from tokenmill_amd.parts import KVCacheView, ParallelMixer, Retention, StateView
    pools = CachePools(_model(A), 5, 4, 3, torch.bfloat16, "cpu")
    mixer = _model(A).layers[0].mixer
    view = pools.views[0]
    left, right = mixer._cache_for(0, view), mixer._cache_for(1, view)
    assert isinstance(left, KVCacheView) and left.k is view.k and left.state is view.state[0] and tuple(left.state.shape) == (4, 3, 184)
    assert isinstance(right, StateView) and right.state is view.state[1] and right.state.dtype == torch.float32
    one_tap = _model(A).layers[1].mixer
    assert one_tap._cache_for(0, pools.views[1]).k is pools.views[1].k and one_tap._cache_for(1, pools.views[1]).state is pools.views[1].state
    both = ParallelMixer(8, Retention(8, 1, 4, 4, [0.5], 1e-5), Retention(8, 2, 4, 6, [0.5, 0.9], 1e-5), scales=(1.0, 1.0))
    states = StateView(("a", "b"))
    assert both._cache_for(0, states).state == "a" and both._cache_for(1, states).state == "b"
    pools.reset_state_slot(1)


def test_pages_of_kept_tokens_stay_when_the_window_has_passed():
    from tokenmill_amd.cache import CacheManager
    from tokenmill_amd.cache.manager import RELEASED
    from tokenmill_amd.parts import KVCacheSpec
    for keep, kept_pages in ((0, 0), (1, 1), (4, 1), (5, 2), (9, 3)):
        m = CacheManager([KVCacheSpec(1, 4, 8, keep=keep)], 12, 4, 2)
        rc = m.allocate("a", 1)
        for n in range(2, 41):
            m.append(rc, n)
            m.release_behind_window(rc, n)
            first = max(0, n - 8 + 1) // 4                                                # the page of the oldest key of the next window
            held = [i for i, p in enumerate(rc.tables[0]) if p != RELEASED]
            assert held == [i for i in range(-(-n // 4)) if i < kept_pages or i >= first], (keep, n)
            m.check_invariants()
        m.free(rc)
        m.check_invariants()
        assert m.num_free_pages == 12


def test_parts_refuse_what_they_cannot_be():
    from tokenmill_amd.parts import OutputHead, PositionWaves, RoutedExperts, SharedNormBlock, SoftmaxAttention, TokenEmbedding
    from tokenmill_amd.parts.embedding import LearnedPositions
    with pytest.raises(ValueError, match="taps"):
        SoftmaxAttention(16, 2, 1, 8, 8, 1.0, taps=17)
    with pytest.raises(ValueError, match="taps"):
        SoftmaxAttention(16, 2, 1, 8, 8, 1.0, taps=2, keys_are_values=True)
    with pytest.raises(ValueError, match="kept"):
        SoftmaxAttention(16, 2, 1, 8, 8, 1.0, keep_first=2)
    with pytest.raises(ValueError, match="per channel"):
        SoftmaxAttention(16, 2, 1, 8, 8, 1.0, channel_gate=True)
    with pytest.raises(ValueError, match="limits"):
        RoutedExperts(16, 8, 4, 1, correction=False, activation="clamped_glu")
    with pytest.raises(ValueError, match="limits"):
        RoutedExperts(16, 8, 4, 1, correction=False, activation="clamped_glu", limit=1.0, shared_ff=4)
    with pytest.raises(ValueError, match="input"):
        RoutedExperts(16, 8, 4, 1, correction=False, activation="swiglu", weigh_input=True)
    with pytest.raises(ValueError, match="waves"):
        TokenEmbedding(5, 4, places=LearnedPositions(8, 4), waves=PositionWaves(4))
    with pytest.raises(ValueError, match="cap"):
        OutputHead(4, 5, None, cap=0.0)
    with pytest.raises(ValueError, match="feed-forward"):
        SharedNormBlock(None, None, None, norm_fed=object())


def test_biases_of_some_of_the_stacked_matrices():
    from tokenmill_amd.parts import Linear
    lin = Linear(4, [3, 2, 1], ["a", "b", "c"], bias=[True, False, True], suffixes=("", ".b"))
    assert set(lin.tensor_specs("")) == {"a", "a.b", "b", "c", "c.b"}
    lin.load({"a": torch.ones(3, 4), "b": torch.ones(2, 4), "c": torch.ones(1, 4), "a.b": torch.tensor([1.0, 2.0, 3.0]), "c.b": torch.tensor([9.0])}, "")
    assert lin.bias.tolist() == [1.0, 2.0, 3.0, 0.0, 0.0, 9.0]


def test_random_weights_round_trip(tmp_path):
    from safetensors.torch import load_file
    from tokenmill_amd.weights.random_init import write_random_model
    write_random_model(B, tmp_path, seed=3)
    w = load_file(str(tmp_path / "model.safetensors"))
    assert w["l0.mix.left.q.conv"].shape == (128, 2) and w["l1.mix.right.norm"].shape == (320,) and "l1.mlp.shared.gate" not in w
    assert torch.isfinite(P.forward([3, 1, 4, 1, 5, 9, 2, 6], B, w)).all()


# ----------------------------------------------------------------------------------------------- the plain mechanisms

def test_waves_of_the_position():
    w = P.position_waves(torch.tensor([0, 1, 50]), 6)
    assert w[0].tolist() == [0.0, 1.0] * 3
    for i in range(3):
        a = 50 * 10000.0 ** (-2 * i / 6)
        assert math.isclose(float(w[2, 2 * i]), math.sin(a), abs_tol=1e-5) and math.isclose(float(w[2, 2 * i + 1]), math.cos(a), abs_tol=1e-5)
    assert P.position_waves(torch.tensor([2]), 3).shape == (1, 3)
    cfg = {"embedding": {"scale": 3.0}, "width": 4}
    assert torch.equal(P.embed(torch.tensor([1]), torch.tensor([0]), cfg, {"embed": torch.ones(2, 4)})[0], torch.tensor([3.0, 4.0, 3.0, 4.0]))


def test_what_a_token_sees():
    seen = P.visible(8, 3, 2)
    assert [torch.nonzero(r).flatten().tolist() for r in seen] == [[0], [0, 1], [0, 1, 2], [0, 1, 2, 3], [0, 1, 2, 3, 4], [0, 1, 3, 4, 5], [0, 1, 4, 5, 6],
                                                                  [0, 1, 5, 6, 7]]
    assert torch.equal(P.visible(6, None, 0), torch.ones(6, 6).tril().bool())
    assert P.visible(4, 1, 0).equal(torch.eye(4).bool()) and P.visible(4, 1, 9).equal(torch.ones(4, 4).tril().bool())


def test_attention_over_equal_scores_averages_what_is_seen():
    T = 9
    z = torch.zeros(T, 2, 3)
    v = torch.arange(T, dtype=torch.float32)[:, None, None].expand(T, 2, 1)
    out = P.kept_window_attention(z, z, v, 5.0, 3, 1)
    for p in range(T):
        seen = sorted({0, *range(max(0, p - 2), p + 1)})
        assert math.isclose(float(out[p, 0, 0]), sum(seen) / len(seen), rel_tol=1e-6)


def test_the_convolution_reads_projected_rows_with_their_bias_and_zeros_before_the_first():
    w = torch.tensor([[10.0, 1.0]])
    assert P.short_conv(torch.tensor([[1.0], [2.0], [3.0]]), w).flatten().tolist() == [1.0, 12.0, 23.0]
    m = {"heads": 1, "kv_heads": 1, "dim": 1, "vdim": 1, "scale": 1.0, "mask": {"size": 1, "keep_first": 0}}
    t = {k: torch.zeros(1, 1) for k in ("q", "k", "g")}
    t |= {"v": torch.ones(1, 1), "o": torch.ones(1, 1), "o.b": torch.zeros(1), "q.b": torch.zeros(1), "k.b": torch.zeros(1), "v.b": torch.full((1,), 4.0),
          "q.norm": torch.ones(1), "k.norm": torch.ones(1), "q.conv": w, "k.conv": w, "v.conv": w}
    out = P.gated_attention(torch.tensor([[1.0], [2.0]]), m, t, "", 1e-6, torch.float32)
    assert torch.allclose(out.flatten(), 0.5 * torch.tensor([5.0, 6.0 + 10.0 * 5.0]))      # the gate is sigmoid(0); the value alone is seen


def test_q_and_k_are_normed_over_all_heads_at_once():
    m = {"heads": 2, "kv_heads": 2, "dim": 2, "vdim": 1, "scale": 1.0}
    eye = torch.eye(4)
    t = {"q": eye, "k": eye, "v": torch.tensor([[1.0, 0, 0, 0], [0, 1.0, 0, 0]]), "g": torch.zeros(2, 4), "o": torch.eye(2), "o.b": torch.zeros(2)}
    t |= {n + ".b": torch.zeros(t[n].shape[0]) for n in "qkv"} | {n + ".conv": torch.ones(t[n].shape[0], 1) for n in "qkv"}
    t |= {"q.norm": torch.ones(4), "k.norm": torch.ones(4)}
    h = torch.tensor([[3.0, 0.0, 0.0, 1.0], [0.0, 2.0, 2.0, 2.0]])
    n = [math.sqrt(10 / 4), math.sqrt(12 / 4)]
    s = [[0.0, 4 / n[1] ** 2], [2 / (n[1] * n[0]), 8 / n[1] ** 2]]                        # the second token's scores, head by head
    out = P.gated_attention(h, m, t, "", 1e-9, torch.float32)
    for head, v in ((0, (3.0, 0.0)), (1, (0.0, 2.0))):
        p = torch.softmax(torch.tensor(s[head]), 0)
        assert math.isclose(float(out[1, head]), 0.5 * float(p[0] * v[0] + p[1] * v[1]), rel_tol=1e-5)


def test_lightning_attention_is_the_decayed_sum_normed_over_all_heads():
    torch.manual_seed(0)
    T, H, D, Dv = 7, 2, 4, 3
    m = {"heads": H, "dim": D, "vdim": Dv, "decay": [0.5, 0.9]}
    t = {n: torch.randn(s, 5) for n, s in (("q", H * D), ("k", H * D), ("v", H * Dv), ("g", H * Dv))} | {"o": torch.eye(H * Dv), "norm": torch.rand(H * Dv)}
    h = torch.randn(T, 5)
    q, k, v = (P.silu(h @ t[n].T).view(T, H, -1) for n in "qkv")
    i = T - 1
    o = torch.cat([sum(m["decay"][g] ** (i - j) * (q[i, g] @ k[j, g]) * v[j, g] for j in range(T)) for g in range(H)])
    want = o / torch.sqrt((o * o).mean() + 1e-6) * t["norm"] * torch.sigmoid(h[i] @ t["g"].T)
    assert torch.allclose(P.lightning(h, m, t, "", 1e-6, torch.float32)[i], want, atol=1e-5)


def test_the_router_weighs_the_experts_input_and_is_not_renormalized():
    t = {"router": torch.tensor([[1.0, 0.0], [-1.0, 0.0], [0.5, 0.0]])}
    h = torch.tensor([[2.0, 0.0], [-2.0, 0.0]])
    chosen, weights = P.route(h, t["router"], 2, torch.float32)
    assert chosen.tolist() == [[0, 2], [1, 2]]
    sig = lambda z: 1 / (1 + math.exp(-z))     # noqa: E731
    assert torch.allclose(weights, torch.tensor([[sig(2.0), sig(1.0)], [sig(2.0), sig(-1.0)]]))
    for e in range(3):
        t |= {f"e{e}.gate": torch.eye(2), f"e{e}.up": torch.zeros(2, 2), f"e{e}.down": torch.eye(2)}
    mlp = {"expert": {"limit": 1.5}, "router": {"top": 2}}
    act = lambda z: min(z, 1.5) * sig(1.702 * min(z, 1.5))     # noqa: E731
    out = P.feed_forward(h, mlp, t, "", torch.float32)
    assert math.isclose(float(out[0, 0]), act(sig(2.0) * 2.0) + act(sig(1.0) * 2.0), rel_tol=1e-6)
    t |= {"shared.gate": torch.eye(2), "shared.up": torch.eye(2), "shared.down": torch.eye(2), "shared.sg": torch.tensor([[0.5, 0.0]])}
    more = P.feed_forward(h, dict(mlp, shared={"limit": 0.25}), t, "", torch.float32)
    assert math.isclose(float(more[0, 0] - out[0, 0]), sig(1.0) * 0.25 * sig(1.702 * 0.25) * 1.25, rel_tol=1e-5)


def test_clamped_gate():
    g, u = torch.tensor([0.0, 3.0, -9.0, 1.0]), torch.tensor([5.0, -5.0, 0.0, 0.5])
    sig = lambda x: 1 / (1 + math.exp(-1.702 * x))     # noqa: E731
    want = [0.0, 2.0 * sig(2.0) * (-2.0 + 1), -9.0 * sig(-9.0), 1.0 * sig(1.0) * 1.5]      # the gate has no lower limit
    assert torch.allclose(P.clamped_glu(g, u, 2.0), torch.tensor(want), atol=1e-6)


def test_logits_are_scaled_and_then_capped():
    h, t = torch.eye(2), {"head": torch.tensor([[4.0, 0.0], [0.0, -40.0]])}
    got = P.logits_of(h, {"logit_scale": 0.5, "logit_softcap": 10.0}, t, torch.float32)
    assert torch.allclose(got.diagonal(), torch.tensor([10 * math.tanh(0.2), -10 * math.tanh(2.0)]))
    assert torch.equal(P.logits_of(h, {}, t, torch.float32), t["head"].T)


def test_the_sublayers_read_two_norms_of_one_stream():
    w = _random_weights(A, 5)
    ids = torch.tensor([4, 9, 2])
    cfg = dict(A, layers=A["layers"][:1])
    x = P.embed(ids, torch.arange(3), cfg, w)
    add = P.mixer(P.rms(x, w["l0.norm1"], 3e-5), A["layers"][0]["mixer"], w, "l0.mix.", 3e-5, torch.float32) + \
        P.feed_forward(P.rms(x, w["l0.norm2"], 3e-5), A["layers"][0]["mlp"], w, "l0.mlp.", torch.float32)
    want = P.logits_of(P.rms(x + add, w["final.norm"], 3e-5), cfg, w, torch.float32)
    assert torch.allclose(P.forward(ids, cfg, w), want, atol=1e-5)


@pytest.mark.parametrize("cfg", [A, B, C])
def test_a_later_token_never_changes_an_earlier_row(cfg):
    w = _random_weights(cfg, 6)
    ids = torch.tensor([3, 1, 4, 1, 5, 9, 2, 6, 5, 3, 5, 8])
    whole = P.forward(ids, cfg, w)
    assert torch.allclose(P.forward(ids[:7], cfg, w), whole[:7], atol=2e-5)


@pytest.mark.parametrize("cfg", [A, B, C])
def test_no_choice_of_experts_is_a_close_call(cfg):
    """The weights the whole-model tests use: the router's outputs at the border of the choice are far apart at every token, and both
    signs of the channel they follow are in use."""
    w = _random_weights(cfg, 7)
    g = torch.Generator().manual_seed(1)
    ids = torch.randint(0, cfg["vocab"], (60,), generator=g)
    streams: list = []
    P.forward(ids, cfg, w, torch.float32, streams)
    streams = [P.embed(ids, torch.arange(60), cfg, w), *streams]
    for i, layer in enumerate(cfg["layers"]):
        if layer["mlp"] is None:
            continue
        r = layer["mlp"]["router"]
        z = P.rms(streams[i], w[f"l{i}.norm2"], cfg["norm"]["eps"]) @ w[f"l{i}.mlp.router"].float().T
        top = z.topk(min(r["top"] + 1, r["experts"])).values
        if r["top"] < r["experts"]:
            assert float((top[:, r["top"] - 1] - top[:, r["top"]]).min()) > 0.05
            assert len({tuple(sorted(c)) for c in z.topk(r["top"]).indices.tolist()}) > 1
