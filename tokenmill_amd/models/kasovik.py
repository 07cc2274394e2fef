"""The Kasovik decoder assembled from parts.

    x = embed[token] * scale + pairs[bucket(previous token, token)]
    every layer:  h = N(x);   x += mixer(h) + ff(h)            (one norm for both; without ff where the layer has none)
    logits = embed . Nf(x)

with N(v) = v / sqrt(mean(v^2) + eps) * w. A layer's mixer is, by its ``type``,
  * ``retention``: a recurrence with one fixed decay per head, rotated queries and keys and a silu gate;
  * ``parallel``: softmax attention inside a sliding window (values that are the keys, q and k normed head by head without
    weights, no positions, a sink per head) beside a gated delta rule with a decay per key channel behind short convolutions and
    a sigmoid gate; the two results are added with constant weights.
The feed-forward is dense with a clamped gate and biases. A layer with ``weights_of: j`` runs layer j's tensors with a cache and
state of its own.
Tensor names: ``embed``, ``bigram``, ``l<i>.norm1``, ``l<i>.mix.<name>`` (``.conv`` for a convolution, ``left.`` / ``right.`` in a
parallel mixer), ``l<i>.mlp.<name>`` (+ ``.b`` for a bias), ``final.norm``.
"""
from __future__ import annotations

from tokenmill_amd.config.model_config import KasovikConfig, KasovikLayer
from tokenmill_amd.config.registry import register_architecture
from tokenmill_amd.models.decoder import DecoderModel, LayerCall
from tokenmill_amd.parts import (GatedDeltaRule, GatedFeedForward, GroupRMSNorm, OutputHead, PairRows, ParallelMixer, Retention,
                                 RotaryEmbedding, SharedNormBlock, SoftmaxAttention, TokenEmbedding)

DEFAULT_POSITIONS = 8192        # positions the rotation tables reach when neither the engine nor config.json says


def _mixer(cfg: KasovikConfig, layer: KasovikLayer, n_pos: int, tables: dict):
    m = layer.mixer
    hidden, eps = cfg.hidden_size, cfg.norm_eps
    if layer.type == "retention":
        rot = m.get("rot") or {}
        dims, rotary = int(rot.get("dims", 0)), None
        if dims:
            key = (int(m["dim"]), float(rot["base"]), dims)
            if key not in tables:           # layers with the same rotation share one table
                tables[key] = RotaryEmbedding(key[0], key[1], n_pos, rotary_dim=dims, exact=True)
            rotary = tables[key]
        return Retention(hidden, int(m["heads"]), int(m["dim"]), int(m["vdim"]), m["decay"], eps, rotary=rotary)
    left, right = m["left"], m["right"]
    window = (left.get("mask") or {}).get("size")
    attention = SoftmaxAttention(hidden, int(left["heads"]), int(left["kv_heads"]), int(left["dim"]), int(left["vdim"]), float(left["scale"]),
                                 window=int(window) if window is not None else None, head_norm_eps=eps, norm_weights=False, sink=True,
                                 keys_are_values=True)
    recurrence = GatedDeltaRule(hidden, int(right["heads"]), int(right["kv_heads"]), int(right["dim"]), int(right["vdim"]),
                                int(right["conv"]), eps, channel_decay=True, narrow_gate=True)
    return ParallelMixer(hidden, attention, recurrence, scales=(float(m["left_scale"]), float(m["right_scale"])))


def build_kasovik(cfg: KasovikConfig, max_positions: int | None = None) -> DecoderModel:
    n_pos = max_positions or cfg.max_position_embeddings or DEFAULT_POSITIONS
    if cfg.max_position_embeddings:
        n_pos = min(n_pos, cfg.max_position_embeddings)
    hidden = cfg.hidden_size
    pairs = PairRows(cfg.pair_buckets, hidden, cfg.pair_mul_prev, cfg.pair_mul_cur, name="bigram")
    embedding = TokenEmbedding(cfg.vocab_size, hidden, name="embed", scale=cfg.embedding_scale, pairs=pairs)
    tables: dict = {}
    layers, numbers, index, run = [], [], {}, []
    for i, layer in enumerate(cfg.layers):
        if layer.weights_of is None:
            ffn = None
            if layer.mlp is not None:
                ffn = GatedFeedForward(hidden, layer.mlp["ff"], "clamped_glu", bias=True, limit=layer.mlp["limit"])
            index[i] = len(layers)
            layers.append(SharedNormBlock(GroupRMSNorm(hidden, cfg.norm_eps, name=""), _mixer(cfg, layer, n_pos, tables), ffn))
            numbers.append(i)
        run.append(LayerCall(index[i if layer.weights_of is None else layer.weights_of]))
    head = OutputHead(hidden, cfg.vocab_size, tied_to=embedding, name="head")
    return DecoderModel(cfg, embedding, layers, GroupRMSNorm(hidden, cfg.norm_eps, name=""), head, run=run,
                        names=("", "l{i}.", "final.norm", ""), layer_numbers=numbers)


register_architecture(KasovikConfig.architecture, KasovikConfig.from_dict, build_kasovik, replace=True)
