"""The Ralitar decoder as a ``ModelSpec``: a token embedding plus a row of a hashed table of
token pairs; blocks whose norms stand behind the sublayers (``x += norm(f(x))``), three of them a
layer: a mixer, a gated GELU unit where the layer has one, and the layer's own token input (a
thin gated projection of x against the layer's part of a second embedding table); a final norm
and a head of its own.  A block's mixer is a gated linear recurrence per channel, the gated delta
rule with a decay per key channel, or softmax attention inside chunks of positions (biased
projections, a norm over the whole rows of queries and of keys, rotation of neighbouring dims
with stretched frequencies, capped scores, keys that serve as values, a gate per channel).  Every
part is one of the package's registered kinds with this model's sizes and constants as
parameters; tensor names are the checkpoint's (``embed``, ``bigram``, ``side.embed``,
``l<i>.norm1``, ``l<i>.mix. ...``, ``l<i>.mlp. ...``, ``l<i>.side. ...``, ``final.norm``,
``head``)."""
from __future__ import annotations

from ..config.errors import ConfigError
from ..config.ralitar import ARCHITECTURE, RalitarConfig, RalitarLayer
from ..parts.base import PartSpec
from ..registry import Architecture, register_architecture
from .spec import LayerSpec, ModelSpec

RECURRENCE_POWER = 8.0      # the design fixes the factor in the recurrence's log decay


def _mixer(cfg: RalitarConfig, layer: RalitarLayer, index: int) -> PartSpec:
    W, m = cfg.width, layer.mixer
    if layer.type == "rglru":
        return PartSpec("rglru", {"hidden_size": W, "width": m.width, "blocks": m.blocks,
                                  "conv": m.conv, "power": RECURRENCE_POWER})
    if layer.type == "channel_delta":
        if m.decay_rank is None or m.gate_rank is None:
            raise ConfigError(f"config.json layers[{index}] mixer: the ranks of the decay's and the "
                              "gate's projections are known neither from a checkpoint nor from "
                              "'decay_rank' and 'gate_rank'")
        return PartSpec("channel_delta", {
            "hidden_size": W, "num_heads": m.heads, "num_kv_heads": m.kv_heads,
            "head_dim": m.dim, "value_dim": m.vdim, "conv": m.conv, "decay_rank": m.decay_rank,
            "gate_rank": m.gate_rank, "eps": cfg.norm_eps})
    position = PartSpec("none")
    if m.rot_dims:
        scaling = None
        if m.rot_scaling is not None:
            s = m.rot_scaling
            scaling = {"rope_type": "llama3", "factor": s.factor, "low_freq_factor": s.low,
                       "high_freq_factor": s.high, "original_max_position_embeddings": s.original}
        position = PartSpec("rope", {"rot_dim": m.rot_dims, "theta": m.rot_base,
                                     "scaling": scaling, "precise": True, "interleaved": True})
    return PartSpec("attention", {
        "hidden_size": W, "num_heads": m.heads, "num_kv_heads": m.kv_heads, "head_dim": m.dim,
        "value_dim": m.dim, "scale": m.scale, "window": None, "chunk": m.chunk,
        "position": position, "softcap": m.softcap or None, "bias": ".b",
        "qk_norm": {"q": "q.norm", "k": "k.norm", "eps": cfg.norm_eps, "whole": True},
        "keys_as_values": True, "channel_gate": "g",
        "names": {"q": "q", "k": "k", "o": "o"}})


def ralitar_spec(cfg: RalitarConfig) -> ModelSpec:
    W = cfg.width
    norm = PartSpec("rmsnorm", {"size": W, "eps": cfg.norm_eps, "weight_name": ""})
    layers, optional = [], []
    for i, layer in enumerate(cfg.layers):
        ff = side = None
        if layer.ff is not None:
            ff = PartSpec("gated_mlp", {"hidden_size": W, "intermediate_size": layer.ff,
                                        "activation": "gelu_tanh",
                                        "names": {"gate": "gate", "up": "up", "down": "down"}})
        else:
            optional.append(f"l{i}.norm2")
        if cfg.side_dim:
            side = PartSpec("token_side", {"hidden_size": W, "vocab_size": cfg.vocab,
                                           "dim": cfg.side_dim, "index": i,
                                           "parts": len(cfg.layers), "table": "side.embed"})
        layers.append(LayerSpec(PartSpec("postnorm", {
            "mixer": _mixer(cfg, layer, i), "feed_forward": ff, "side": side,
            "mixer_norm": norm, "ffn_norm": norm, "side_norm": norm,
            "names": {"mixer": "mix", "mixer_norm": "norm1", "feed_forward": "mlp",
                      "ffn_norm": "norm2", "side": "side", "side_norm": "side.norm"}}), f"l{i}"))
    embedding = {"vocab_size": cfg.vocab, "hidden_size": W, "weight_name": ""}
    if cfg.bigram is not None:
        b = cfg.bigram
        embedding["bigram"] = {"name": "bigram", "buckets": b.buckets, "mul_prev": b.mul_prev,
                               "mul_cur": b.mul_cur}
    return ModelSpec(
        hidden_size=W,
        vocab_size=cfg.vocab,
        embedding=PartSpec("token", embedding),
        embedding_prefix="embed",
        layers=layers,
        final_norm=norm,
        final_norm_prefix="final.norm",
        head=PartSpec("linear", {"vocab_size": cfg.vocab, "hidden_size": W, "tied_to": None,
                                 "weight_name": ""}),
        head_prefix="head",
        optional_tensors=tuple(optional),
    )


register_architecture(Architecture(
    name=ARCHITECTURE,
    parse_config=RalitarConfig.from_dict,
    build_spec=ralitar_spec,
    config_to_dict=lambda cfg: cfg.to_dict(),
    complete_config=lambda cfg, shapes: cfg.with_tensor_shapes(shapes),
))
