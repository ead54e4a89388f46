"""The Pozelix decoder as a ``ModelSpec``: a token embedding, blocks with norms in front of their
sublayers and behind them, a final norm and a head of its own.  A stretch of the layers may run
several times in a row: the run order names those layers once per pass (every run then has a cache
of its own), and in front of each pass's first layer stands a junction that makes the stream a
linear map of itself and of the embedding output.  A block's mixer is attention over a cached
latent (queries from a latent of their own, a rotated key part of neighbouring pairs with stretched
frequencies) or grouped attention under a sliding window (queries and keys normed behind their
rotation, a gate per head); its feed-forward, when it has one, is a SwiGLU unit or a mixture of
such units beside identity experts.  Every part is one of the package's registered kinds with this
model's sizes and constants as parameters; tensor names are the checkpoint's (``embed``,
``loop.in``, ``l<i>.norm1``, ``l<i>.norm1b``, ``l<i>.mix. ...``, ``l<i>.norm2``, ``l<i>.norm2b``,
``l<i>.mlp. ...``, ``final.norm``, ``head``)."""
from __future__ import annotations

from typing import Optional

from ..config.pozelix import ARCHITECTURE, DenseMlp, PozelixConfig, PozelixLayer, Rotation
from ..parts.base import PartSpec
from ..registry import Architecture, register_architecture
from .spec import JunctionSpec, LayerSpec, ModelSpec, RunEntry


def _position(rot: Optional[Rotation], interleaved: bool) -> PartSpec:
    if rot is None or rot.dims == 0:
        return PartSpec("none")
    scaling = None
    if rot.scaling is not None:
        s = rot.scaling
        scaling = {"rope_type": "yarn", "factor": s.factor, "original": s.original,
                   "fast": s.fast, "slow": s.slow}
    return PartSpec("rope", {"rot_dim": rot.dims, "theta": rot.base, "scaling": scaling,
                             "precise": True, "interleaved": interleaved})


def _mixer(cfg: PozelixConfig, layer: PozelixLayer) -> PartSpec:
    W, m = cfg.width, layer.mixer
    if layer.type == "latent_attention":
        return PartSpec("latent_attention", {
            "hidden_size": W, "num_heads": m.heads, "head_dim": m.dim, "rot_dim": m.rot_dim,
            "value_dim": m.vdim, "q_rank": m.q_rank, "kv_rank": m.kv_rank, "scale": m.scale,
            "eps": cfg.norm_eps, "window": None, "position": _position(m.rot, True)})
    return PartSpec("attention", {
        "hidden_size": W, "num_heads": m.heads, "num_kv_heads": m.kv_heads, "head_dim": m.dim,
        "value_dim": m.vdim, "scale": m.scale, "window": m.window,
        "position": _position(m.rot, False),
        "qk_norm": {"eps": cfg.norm_eps, "behind_rotation": True}, "gate": "g",
        "names": {n: n for n in "qkvo"}})


def _feed_forward(cfg: PozelixConfig, layer: PozelixLayer) -> Optional[PartSpec]:
    W, p = cfg.width, layer.mlp
    if p is None:
        return None
    if isinstance(p, DenseMlp):
        return PartSpec("swiglu", {"hidden_size": W, "intermediate_size": p.ff,
                                   "names": {n: n for n in ("gate", "up", "down")}})
    return PartSpec("routed_swiglu", {
        "hidden_size": W, "expert_size": p.expert_ff, "experts": p.experts,
        "identity": p.identity, "top": p.top, "groups": 1, "keep": 1, "scores": "softmax",
        "group_score": "max", "scale": 1.0})


def pozelix_spec(cfg: PozelixConfig) -> ModelSpec:
    W, n = cfg.width, len(cfg.layers)
    norm = PartSpec("rmsnorm", {"size": W, "eps": cfg.norm_eps, "weight_name": ""})
    layers, optional = [], []
    for i, layer in enumerate(cfg.layers):
        ff = _feed_forward(cfg, layer)
        if ff is None:
            optional += [f"l{i}.norm2", f"l{i}.norm2b"]
        layers.append(LayerSpec(PartSpec("sandwich", {
            "mixer": _mixer(cfg, layer), "feed_forward": ff, "mixer_norm": norm,
            "mixer_post": norm, "ffn_norm": norm, "ffn_post": norm,
            "names": {"mixer": "mix", "mixer_norm": "norm1", "mixer_post": "norm1b",
                      "feed_forward": "mlp", "ffn_norm": "norm2", "ffn_post": "norm2b"}}),
            f"l{i}"))
    runs = [RunEntry(i) for i in range(n)]
    junctions = []
    if cfg.loop is not None:
        a, b = cfg.loop.start, cfg.loop.stop
        junctions = [JunctionSpec(PartSpec("embedding_rejoin", {"hidden_size": W}), "loop.in")]
        one_pass = [RunEntry(i, junction=0 if i == a else None) for i in range(a, b)]
        runs = runs[:a] + one_pass * cfg.loop.times + runs[b:]
    return ModelSpec(
        hidden_size=W,
        vocab_size=cfg.vocab,
        embedding=PartSpec("token", {"vocab_size": cfg.vocab, "hidden_size": W,
                                     "weight_name": ""}),
        embedding_prefix="embed",
        layers=layers,
        run_order=runs,
        junctions=junctions,
        final_norm=norm,
        final_norm_prefix="final.norm",
        head=PartSpec("linear", {"vocab_size": cfg.vocab, "hidden_size": W, "tied_to": None,
                                 "weight_name": ""}),
        head_prefix="head",
        optional_tensors=tuple(optional),
    )


register_architecture(Architecture(
    name=ARCHITECTURE,
    parse_config=PozelixConfig.from_dict,
    build_spec=pozelix_spec,
    config_to_dict=lambda cfg: cfg.to_dict(),
))
