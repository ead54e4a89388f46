"""Typed configuration of the Ralitar decoder, read from its ``config.json``.

The file names the design under ``architecture`` and gives every size and every constant that
may differ between two models of it: vocabulary, width, the table of token pairs that joins the
embedding (``embedding.bigram``; absent: none), the norms' epsilon, the width of the per-layer
token input (``token_side``; absent: none) and a list of layers.  A layer's ``type`` names its
mixer: ``rglru`` (a gated linear recurrence per channel), ``channel_delta`` (the gated delta rule
with a decay per key channel) or ``attention`` (softmax attention inside chunks, whose values are
its keys).  Its ``mlp`` is null or ``dense`` (a gated unit with the tanh form of GELU).  The ranks
of the low-rank projections of ``channel_delta`` are the tensors' (``with_tensor_shapes``); a
configuration that is to get random weights names them as ``decay_rank`` and ``gate_rank`` in the
layer's ``mixer``.

The parser refuses what the engine would compute wrongly, with the key's name."""
from __future__ import annotations

from dataclasses import dataclass, replace
from typing import Any, Dict, Mapping, Optional, Sequence, Tuple, Union

from .errors import ConfigError
from .gipotar import _obj, _positive
from .llama import _need, _typed

ARCHITECTURE = "Ralitar"


@dataclass(frozen=True)
class Bigram:
    """Row of the pair table: (previous token * mul_prev + token * mul_cur) mod buckets; row
    ``buckets`` for a sequence's first token."""
    buckets: int
    mul_prev: int
    mul_cur: int

    @classmethod
    def from_dict(cls, d: Dict[str, Any], where: str) -> "Bigram":
        out = cls(*(_need(d, k, int, where) for k in ("buckets", "mul_prev", "mul_cur")))
        _positive(out.buckets, "buckets", where)
        for key, v in (("mul_prev", out.mul_prev), ("mul_cur", out.mul_cur)):
            if not 0 <= v < 1 << 31:
                raise ConfigError(f"{where}: '{key}' {v} must be in [0, 2^31)")
        return out

    def to_dict(self) -> Dict[str, Any]:
        return {"buckets": self.buckets, "mul_cur": self.mul_cur, "mul_prev": self.mul_prev}


@dataclass(frozen=True)
class RotScaling:
    factor: float
    low: float
    high: float
    original: float

    @classmethod
    def from_dict(cls, d: Dict[str, Any], where: str) -> "RotScaling":
        out = cls(*(_need(d, k, float, where) for k in ("factor", "low", "high", "original")))
        if not (out.factor > 0 and out.low > 0 and out.high > out.low and out.original > 0):
            raise ConfigError(f"{where}: 'factor', 'low' and 'original' must be positive and "
                              "'high' above 'low'")
        return out

    def to_dict(self) -> Dict[str, Any]:
        return {"factor": self.factor, "high": self.high, "low": self.low,
                "original": self.original}


@dataclass(frozen=True)
class AttentionMixer:
    heads: int
    kv_heads: int
    dim: int
    scale: float
    chunk: Optional[int] = None         # a query sees keys of its own chunk of so many positions
    softcap: float = 0.0                # 0: no cap
    rot_dims: int = 0
    rot_base: float = 10000.0
    rot_scaling: Optional[RotScaling] = None

    @classmethod
    def from_dict(cls, d: Dict[str, Any], where: str) -> "AttentionMixer":
        kw: Dict[str, Any] = {k: _positive(_need(d, k, int, where), k, where)
                              for k in ("heads", "kv_heads", "dim")}
        kw["scale"] = _need(d, "scale", float, where)
        if not kw["scale"] > 0:
            raise ConfigError(f"{where}: 'scale' must be positive")
        if d.get("vdim") is not None and _typed(d["vdim"], "vdim", int, where) != kw["dim"]:
            raise ConfigError(f"{where}: 'vdim' {d['vdim']} differs from 'dim' {kw['dim']}: the "
                              "values are the keys")
        if d.get("mask") is not None:
            kw["chunk"] = _positive(_need(_obj(d, "mask", where), "size", int, where + " mask"),
                                    "size", where + " mask")
        if d.get("softcap") is not None:
            kw["softcap"] = _typed(d["softcap"], "softcap", float, where)
            if kw["softcap"] < 0:
                raise ConfigError(f"{where}: 'softcap' must be positive")
        if d.get("rot") is not None:
            rot = _obj(d, "rot", where)
            kw["rot_dims"] = _need(rot, "dims", int, where + " rot")
            kw["rot_base"] = _need(rot, "base", float, where + " rot")
            if rot.get("scaling") is not None:
                kw["rot_scaling"] = RotScaling.from_dict(_obj(rot, "scaling", where + " rot"),
                                                         where + " rot scaling")
        out = cls(**kw)
        if out.heads % out.kv_heads:
            raise ConfigError(f"{where}: 'heads' {out.heads} is not a multiple of 'kv_heads' "
                              f"{out.kv_heads}")
        if out.rot_dims < 0 or out.rot_dims % 2 or out.rot_dims > out.dim:
            raise ConfigError(f"{where} rot: 'dims' {out.rot_dims} must be even and at most "
                              f"'dim' {out.dim}")
        if out.rot_dims and not out.rot_base > 0:
            raise ConfigError(f"{where} rot: 'base' must be positive")
        return out

    def to_dict(self) -> Dict[str, Any]:
        d: Dict[str, Any] = {"dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads,
                             "scale": self.scale, "vdim": self.dim}
        if self.chunk is not None:
            d["mask"] = {"size": self.chunk}
        if self.softcap:
            d["softcap"] = self.softcap
        if self.rot_dims:
            d["rot"] = {"base": self.rot_base, "dims": self.rot_dims}
            if self.rot_scaling is not None:
                d["rot"]["scaling"] = self.rot_scaling.to_dict()
        return d


@dataclass(frozen=True)
class ChannelDeltaMixer:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int
    decay_rank: Optional[int] = None    # rows of the decay's first projection; from the tensors
    gate_rank: Optional[int] = None     # rows of the output gate's; from the tensors

    @classmethod
    def from_dict(cls, d: Dict[str, Any], where: str) -> "ChannelDeltaMixer":
        kw: Dict[str, Any] = {k: _positive(_need(d, k, int, where), k, where)
                              for k in ("heads", "kv_heads", "dim", "vdim", "conv")}
        for k in ("decay_rank", "gate_rank"):
            if d.get(k) is not None:
                kw[k] = _positive(_typed(d[k], k, int, where), k, where)
        out = cls(**kw)
        if out.heads % out.kv_heads:
            raise ConfigError(f"{where}: 'heads' {out.heads} is not a multiple of 'kv_heads' "
                              f"{out.kv_heads}")
        return out

    def to_dict(self) -> Dict[str, Any]:
        d: Dict[str, Any] = {"conv": self.conv, "dim": self.dim, "heads": self.heads,
                             "kv_heads": self.kv_heads, "vdim": self.vdim}
        for k in ("decay_rank", "gate_rank"):
            if getattr(self, k) is not None:
                d[k] = getattr(self, k)
        return d


@dataclass(frozen=True)
class RglruMixer:
    width: int
    blocks: int
    conv: int

    @classmethod
    def from_dict(cls, d: Dict[str, Any], where: str) -> "RglruMixer":
        out = cls(**{k: _positive(_need(d, k, int, where), k, where)
                     for k in ("width", "blocks", "conv")})
        if out.width % out.blocks:
            raise ConfigError(f"{where}: 'width' {out.width} is not a multiple of 'blocks' "
                              f"{out.blocks}")
        return out

    def to_dict(self) -> Dict[str, Any]:
        return {"blocks": self.blocks, "conv": self.conv, "width": self.width}


RalitarMixer = Union[AttentionMixer, ChannelDeltaMixer, RglruMixer]
MIXERS = {"attention": AttentionMixer, "channel_delta": ChannelDeltaMixer, "rglru": RglruMixer}


@dataclass(frozen=True)
class RalitarLayer:
    type: str
    mixer: RalitarMixer
    ff: Optional[int]                   # inner width of the feed-forward, None: there is none

    @classmethod
    def from_dict(cls, d: Any, index: int) -> "RalitarLayer":
        where = f"config.json layers[{index}]"
        if not isinstance(d, dict):
            raise ConfigError(f"{where}: must be an object")
        kind = _need(d, "type", str, where)
        if kind not in MIXERS:
            raise ConfigError(f"{where}: type '{kind}' is not supported (known: "
                              f"{', '.join(repr(m) for m in MIXERS)})")
        mixer = MIXERS[kind].from_dict(_obj(d, "mixer", where), where + " mixer")
        mlp = d.get("mlp")
        if mlp is None:
            return cls(kind, mixer, None)
        mlp = _obj(d, "mlp", where)
        if _need(mlp, "kind", str, where + " mlp") != "dense":
            raise ConfigError(f"{where} mlp: kind '{mlp['kind']}' is not supported (known: 'dense')")
        return cls(kind, mixer, _positive(_need(mlp, "ff", int, where + " mlp"), "ff",
                                          where + " mlp"))

    def to_dict(self) -> Dict[str, Any]:
        return {"mixer": self.mixer.to_dict(), "type": self.type,
                "mlp": None if self.ff is None else {"ff": self.ff, "kind": "dense"}}


@dataclass(frozen=True)
class RalitarConfig:
    vocab: int
    width: int
    norm_eps: float
    bigram: Optional[Bigram]
    side_dim: int                       # 0: no per-layer token input
    layers: Tuple[RalitarLayer, ...]
    architecture: str = ARCHITECTURE

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def max_position_embeddings(self) -> int:
        """No table bounds the positions: the engine's own limit holds."""
        return 1 << 20

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "RalitarConfig":
        where = "config.json"
        layers = d.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError(f"{where}: 'layers' must be a non-empty list")
        bigram = None
        if d.get("embedding") is not None:
            emb = _obj(d, "embedding", where)
            if emb.get("bigram") is not None:
                bigram = Bigram.from_dict(_obj(emb, "bigram", where + " embedding"),
                                          where + " embedding bigram")
        side = 0
        if d.get("token_side") is not None:
            side = _positive(_need(_obj(d, "token_side", where), "dim", int, where + " token_side"),
                             "dim", where + " token_side")
        out = cls(vocab=_positive(_need(d, "vocab", int), "vocab", where),
                  width=_positive(_need(d, "width", int), "width", where),
                  norm_eps=_need(_obj(d, "norm", where), "eps", float, where + " norm"),
                  bigram=bigram, side_dim=side,
                  layers=tuple(RalitarLayer.from_dict(l, i) for i, l in enumerate(layers)))
        if not out.norm_eps > 0:
            raise ConfigError(f"{where} norm: 'eps' must be positive")
        return out

    def to_dict(self) -> Dict[str, Any]:
        d: Dict[str, Any] = {"architecture": self.architecture,
                             "layers": [l.to_dict() for l in self.layers],
                             "norm": {"eps": self.norm_eps}, "vocab": self.vocab,
                             "width": self.width}
        if self.bigram is not None:
            d["embedding"] = {"bigram": self.bigram.to_dict()}
        if self.side_dim:
            d["token_side"] = {"dim": self.side_dim}
        return d

    def with_tensor_shapes(self, shapes: Mapping[str, Sequence[int]]) -> "RalitarConfig":
        """The configuration with the ranks of the low-rank projections filled in (rows of
        ``l<i>.mix.a1`` and ``l<i>.mix.g1``)."""
        layers = []
        for i, layer in enumerate(self.layers):
            if layer.type == "channel_delta":
                found = {}
                for key, name in (("decay_rank", "a1"), ("gate_rank", "g1")):
                    shape = shapes.get(f"l{i}.mix.{name}")
                    if getattr(layer.mixer, key) is None and shape is not None and len(shape) == 2:
                        found[key] = int(shape[0])
                layer = replace(layer, mixer=replace(layer.mixer, **found))
            layers.append(layer)
        return replace(self, layers=tuple(layers))
