"""Typed configuration of the Pozelix decoder, read from its ``config.json``.

The file names the design under ``architecture`` and gives every size and every constant that
may differ between two models of it: vocabulary, width, the norms' epsilon, a list of layers and
the stretch of them that runs several times in a row (``loop``; absent: none).  A layer's ``type``
names its mixer: ``latent_attention`` (queries from one latent, keys and values from another that
is cached, a rotated key part shared by the heads, every earlier key) or ``attention`` (grouped
heads under a sliding window, queries and keys normed behind their rotation, a gate per head).
Its ``mlp`` is null, ``dense`` or ``moe`` (some of whose experts hand their input back).

The parser refuses what the engine would compute wrongly, with the key's name."""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, Optional, Tuple, Union

from .errors import ConfigError
from .gipotar import _obj, _positive
from .llama import _need, _typed

ARCHITECTURE = "Pozelix"


@dataclass(frozen=True)
class RotScaling:
    """Frequencies of slow pairs divided by ``factor``, fast ones kept, a ramp between."""
    factor: float
    original: float
    fast: float
    slow: float

    @classmethod
    def from_dict(cls, d: Dict[str, Any], where: str) -> "RotScaling":
        out = cls(*(_need(d, k, float, where) for k in ("factor", "original", "fast", "slow")))
        if not (out.factor > 0 and out.original > 0 and out.fast > 0 and out.slow > 0):
            raise ConfigError(f"{where}: 'factor', 'original', 'fast' and 'slow' must be positive")
        return out

    def to_dict(self) -> Dict[str, Any]:
        return {"factor": self.factor, "fast": self.fast, "original": self.original,
                "slow": self.slow}


@dataclass(frozen=True)
class Rotation:
    dims: int
    base: float
    scaling: Optional[RotScaling] = None

    @classmethod
    def from_dict(cls, d: Dict[str, Any], where: str, width: int, stretches: bool) -> "Rotation":
        dims, base = _need(d, "dims", int, where), _need(d, "base", float, where)
        if dims < 0 or dims % 2 or dims > width:
            raise ConfigError(f"{where}: 'dims' {dims} must be even and at most {width}")
        if not base > 0 or base == 1.0:
            raise ConfigError(f"{where}: 'base' {base} must be positive and not 1")
        scaling = None
        if d.get("scaling") is not None:
            if not stretches:
                raise ConfigError(f"{where}: 'scaling' is not supported in this mixer")
            scaling = RotScaling.from_dict(_obj(d, "scaling", where), where + " scaling")
        return cls(dims, base, scaling)

    def to_dict(self) -> Dict[str, Any]:
        d: Dict[str, Any] = {"base": self.base, "dims": self.dims}
        if self.scaling is not None:
            d["scaling"] = self.scaling.to_dict()
        return d


def _scale(d: Dict[str, Any], where: str) -> float:
    return _need(d, "scale", float, where)


@dataclass(frozen=True)
class LatentMixer:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    rot: Rotation
    scale: float

    @classmethod
    def from_dict(cls, d: Dict[str, Any], where: str) -> "LatentMixer":
        kw: Dict[str, Any] = {k: _positive(_need(d, k, int, where), k, where) for k in
                              ("heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank")}
        rot = Rotation.from_dict(_obj(d, "rot", where), where + " rot", kw["rot_dim"], True)
        return cls(rot=rot, scale=_scale(d, where), **kw)

    def to_dict(self) -> Dict[str, Any]:
        return {"dim": self.dim, "heads": self.heads, "kv_rank": self.kv_rank,
                "q_rank": self.q_rank, "rot": self.rot.to_dict(), "rot_dim": self.rot_dim,
                "scale": self.scale, "vdim": self.vdim}


@dataclass(frozen=True)
class AttentionMixer:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: Optional[int] = None        # None: every earlier key
    rot: Optional[Rotation] = None      # None: no rotation

    @classmethod
    def from_dict(cls, d: Dict[str, Any], where: str) -> "AttentionMixer":
        kw: Dict[str, Any] = {k: _positive(_need(d, k, int, where), k, where)
                              for k in ("heads", "kv_heads", "dim", "vdim")}
        if kw["heads"] % kw["kv_heads"]:
            raise ConfigError(f"{where}: 'heads' {kw['heads']} is not a multiple of 'kv_heads' "
                              f"{kw['kv_heads']}")
        if d.get("mask") is not None:
            kw["window"] = _positive(_need(_obj(d, "mask", where), "size", int, where + " mask"),
                                     "size", where + " mask")
        if d.get("rot") is not None:
            kw["rot"] = Rotation.from_dict(_obj(d, "rot", where), where + " rot", kw["dim"], False)
        return cls(scale=_scale(d, where), **kw)

    def to_dict(self) -> Dict[str, Any]:
        d: Dict[str, Any] = {"dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads,
                             "scale": self.scale, "vdim": self.vdim}
        if self.window is not None:
            d["mask"] = {"size": self.window}
        if self.rot is not None:
            d["rot"] = self.rot.to_dict()
        return d


@dataclass(frozen=True)
class DenseMlp:
    ff: int

    def to_dict(self) -> Dict[str, Any]:
        return {"ff": self.ff, "kind": "dense"}


@dataclass(frozen=True)
class MoeMlp:
    expert_ff: int
    experts: int                        # those with tensors
    identity: int                       # those that hand back their input
    top: int

    def to_dict(self) -> Dict[str, Any]:
        return {"expert": {"ff": self.expert_ff}, "kind": "moe",
                "router": {"experts": self.experts, "identity": self.identity, "top": self.top}}


def _mlp_from_dict(d: Dict[str, Any], where: str) -> Union[DenseMlp, MoeMlp]:
    kind = _need(d, "kind", str, where)
    if kind == "dense":
        return DenseMlp(_positive(_need(d, "ff", int, where), "ff", where))
    if kind != "moe":
        raise ConfigError(f"{where}: kind '{kind}' is not supported (known: 'dense', 'moe')")
    router = _obj(d, "router", where)
    rw = where + " router"
    identity = 0
    if router.get("identity") is not None:
        identity = _typed(router["identity"], "identity", int, rw)
        if identity < 0:
            raise ConfigError(f"{rw}: 'identity' {identity} must not be negative")
    out = MoeMlp(
        expert_ff=_positive(_need(_obj(d, "expert", where), "ff", int, where + " expert"), "ff",
                            where + " expert"),
        experts=_positive(_need(router, "experts", int, rw), "experts", rw), identity=identity,
        top=_positive(_need(router, "top", int, rw), "top", rw))
    if out.top > out.experts + out.identity:
        raise ConfigError(f"{rw}: 'top' {out.top} exceeds the {out.experts} experts and "
                          f"{out.identity} identity experts")
    return out


MIXERS = {"attention": AttentionMixer, "latent_attention": LatentMixer}


@dataclass(frozen=True)
class PozelixLayer:
    type: str
    mixer: Union[LatentMixer, AttentionMixer]
    mlp: Optional[Union[DenseMlp, MoeMlp]]

    @classmethod
    def from_dict(cls, d: Any, index: int) -> "PozelixLayer":
        where = f"config.json layers[{index}]"
        if not isinstance(d, dict):
            raise ConfigError(f"{where}: must be an object")
        kind = _need(d, "type", str, where)
        if kind not in MIXERS:
            raise ConfigError(f"{where}: type '{kind}' is not supported (known: "
                              f"{', '.join(repr(m) for m in MIXERS)})")
        mixer = MIXERS[kind].from_dict(_obj(d, "mixer", where), where + " mixer")
        mlp = None
        if d.get("mlp") is not None:
            mlp = _mlp_from_dict(_obj(d, "mlp", where), where + " mlp")
        return cls(kind, mixer, mlp)

    def to_dict(self) -> Dict[str, Any]:
        return {"mixer": self.mixer.to_dict(),
                "mlp": None if self.mlp is None else self.mlp.to_dict(), "type": self.type}


@dataclass(frozen=True)
class Loop:
    """Layers ``start`` to ``stop - 1`` run ``times`` times in a row."""
    start: int
    stop: int
    times: int

    @classmethod
    def from_dict(cls, d: Dict[str, Any], layers: int) -> "Loop":
        where = "config.json loop"
        out = cls(*(_need(d, k, int, where) for k in ("start", "stop", "times")))
        if not 0 <= out.start < out.stop <= layers:
            raise ConfigError(f"{where}: 'start' {out.start} and 'stop' {out.stop} name no layers of "
                              f"{layers}")
        _positive(out.times, "times", where)
        return out

    def to_dict(self) -> Dict[str, Any]:
        return {"start": self.start, "stop": self.stop, "times": self.times}


@dataclass(frozen=True)
class PozelixConfig:
    vocab: int
    width: int
    norm_eps: float
    layers: Tuple[PozelixLayer, ...]
    loop: Optional[Loop]
    architecture: str = ARCHITECTURE

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def max_position_embeddings(self) -> int:
        """No table bounds the positions: the engine's own limit holds."""
        return 1 << 20

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "PozelixConfig":
        where = "config.json"
        layers = d.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError(f"{where}: 'layers' must be a non-empty list")
        loop = None
        if d.get("loop") is not None:
            loop = Loop.from_dict(_obj(d, "loop", where), len(layers))
        out = cls(vocab=_positive(_need(d, "vocab", int), "vocab", where),
                  width=_positive(_need(d, "width", int), "width", where),
                  norm_eps=_need(_obj(d, "norm", where), "eps", float, where + " norm"),
                  layers=tuple(PozelixLayer.from_dict(l, i) for i, l in enumerate(layers)),
                  loop=loop)
        if not out.norm_eps > 0:
            raise ConfigError(f"{where} norm: 'eps' must be positive")
        return out

    def to_dict(self) -> Dict[str, Any]:
        d: Dict[str, Any] = {"architecture": self.architecture,
                             "layers": [l.to_dict() for l in self.layers],
                             "norm": {"eps": self.norm_eps}, "vocab": self.vocab,
                             "width": self.width}
        if self.loop is not None:
            d["loop"] = self.loop.to_dict()
        return d
