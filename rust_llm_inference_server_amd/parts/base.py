"""The interfaces of the parts a model is put together from, and one registry per kind.

A model is a list of blocks; a block arranges a *mixer* (the part through which a token sees
earlier tokens), a *feed-forward* and *norms*; a mixer may use a *position encoding*.  Each
part is built from a ``PartSpec`` (a kind name plus a dict of parameters that carries every
size and constant), a weight-name prefix and a ``BuildContext``.  No part knows which model
it is in: what it needs arrives as parameters, per-step data arrives in the ``StepContext``.

The reference builds its layers the same way, with constants passed in:
``RmsNorm::new(weight, eps)`` (crates/model/src/layers.rs:112-118), ``Attention::new(q, k, v,
bias, o, cfg)`` (attention.rs:23-41), ``Mlp::new(gate, up, down)`` (layers.rs:165-167),
``Rope::from_inv_freqs`` (rope.rs:61-78).

Adding a part: subclass the base class of its kind, decorate it with ``@register(kind_name)``
and name it in a model's specification.  The registries are open; a test may register a part
of its own without touching this package.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Callable, Dict, List, Optional, Tuple, Type

import torch

from ..stepplan import HostPlan, StepLengths, StepPlan, StepPlanner  # noqa: F401 (re-exported)


# --------------------------------------------------------------------------- specs
@dataclass(frozen=True)
class TensorSpec:
    """One checkpoint tensor a part reads: its full name, its shape and how random weights
    for it are drawn (``normal``: N(0, std); ``ones_normal``: 1 + N(0, std))."""

    name: str
    shape: Tuple[int, ...]
    init: str = "normal"
    std: float = 0.02


@dataclass
class PartSpec:
    kind: str
    params: Dict[str, Any] = field(default_factory=dict)


PAGE = -1     # in a PageArray's shape: the axis that is as long as a page has positions


@dataclass(frozen=True)
class PageArray:
    """One array a mixer keeps per page: its name and the shape of one page, in which ``PAGE``
    marks the axis of positions.  Keys of 8 heads of 64 are ``("k", (8, PAGE, 64))``; one latent
    vector of 96 numbers per position is ``("latent", (PAGE, 96))``.  ``dtype`` None: the
    model's activation dtype; a mixer that caches something in a precision of its own (float32
    sums in a bfloat16 model, 8-bit codes) names the torch dtype here, and the pools allocate
    and size that array by it."""

    name: str
    shape: Tuple[int, ...]
    dtype: Optional[torch.dtype] = None

    def __post_init__(self):
        if self.shape.count(PAGE) != 1 or any(n <= 0 for n in self.shape if n != PAGE):
            raise ValueError(f"page array '{self.name}': shape {self.shape} needs positive sizes "
                             "and the position axis exactly once")
        if self.dtype is not None and not isinstance(self.dtype, torch.dtype):
            raise ValueError(f"page array '{self.name}': dtype must be a torch dtype or None, "
                             f"got {self.dtype!r}")

    def element_size(self, act_dtype: torch.dtype) -> int:
        """Bytes of one element, in a model whose activations are ``act_dtype``."""
        return torch.empty((), dtype=self.dtype or act_dtype).element_size()

    def bytes_per_token(self, act_dtype: torch.dtype) -> int:
        return self.elements_per_token() * self.element_size(act_dtype)

    def page_shape(self, page_size: int) -> Tuple[int, ...]:
        return tuple(page_size if n == PAGE else n for n in self.shape)

    def elements_per_token(self) -> int:
        n = 1
        for x in self.shape:
            n *= 1 if x == PAGE else x
        return n


@dataclass(frozen=True)
class CacheRequest:
    """What a mixer keeps in pages for every cached position: a kind of its own, given as the
    arrays of one page (each in the activation dtype unless it names its own), for every earlier position (``window``
    None) or for the last ``window`` positions only.  Mixers with equal requests share a page
    group; the pools are allocated from the request, so a mixer that caches something else than
    keys and values names its own arrays.  ``CacheRequest.kv`` is the kind attention uses."""

    arrays: Tuple[PageArray, ...]
    window: Optional[int] = None
    # with a window: the first so many positions of a sequence are kept beside the latest ones
    keep_first: int = 0

    def __post_init__(self):
        names = [a.name for a in self.arrays]
        if not names or len(set(names)) != len(names):
            raise ValueError(f"a cache request needs arrays with distinct names, got {names}")

    @classmethod
    def kv(cls, num_kv_heads: int, head_dim: int, window: Optional[int] = None,
           keep_first: int = 0) -> "CacheRequest":
        """Keys ``[kv head][position][d]`` and values ``[kv head][d][position]`` (values
        transposed inside a page, so that both attention kernels read each as it lies)."""
        return cls((PageArray("k", (num_kv_heads, PAGE, head_dim)),
                    PageArray("v", (num_kv_heads, head_dim, PAGE))), window,
                   int(keep_first) if window else 0)

    def group_key(self) -> Tuple[Any, ...]:
        return (self.arrays, self.window, self.keep_first)

    def elements_per_token(self) -> int:
        return sum(a.elements_per_token() for a in self.arrays)

    def bytes_per_token(self, act_dtype: torch.dtype) -> int:
        """Bytes that one cached position takes in one layer slot of the group."""
        return sum(a.bytes_per_token(act_dtype) for a in self.arrays)


@dataclass
class CacheBinding:
    """Where one run of a mixer keeps its memory of the past.

    ``pages`` maps each array name of the mixer's cache request to this run's slice of its
    group's pool, ``(num_pages, *page shape)``; ``group`` indexes ``StepContext.groups`` (block
    tables and slots of that group).  ``writes`` is false when the run reads the cache another
    run has written in the same step.  ``state`` is the run's slice of the fixed-size
    per-request state buffer, ``(num_slots, state_bytes)`` uint8, or None when the mixer asked
    for none.  ``counters`` is a run of int32 zeros on the device that belongs to the runner
    (and so to its stream): a mixer's kernels may count in it within one launch, the
    workgroups of the decode attention do when they merge partitions, if they leave zeros."""

    group: int = -1
    pages: Dict[str, torch.Tensor] = field(default_factory=dict)
    writes: bool = True
    state: Optional[torch.Tensor] = None
    counters: Optional[torch.Tensor] = None

    @property
    def k_pages(self) -> Optional[torch.Tensor]:
        return self.pages.get("k")

    @property
    def v_pages(self) -> Optional[torch.Tensor]:
        return self.pages.get("v")


@dataclass
class BuildContext:
    """What a part may look at while it is built."""

    device: torch.device
    act_dtype: torch.dtype                      # torch.float32 or torch.bfloat16
    weights: Dict[str, torch.Tensor]            # checkpoint name -> device tensor
    max_positions: int                          # longest sequence the engine will run
    shared: Dict[Any, Any] = field(default_factory=dict)   # e.g. position tables by parameters

    def take(self, name: str) -> torch.Tensor:
        try:
            return self.weights[name]
        except KeyError:
            raise KeyError(f"weight '{name}' was not loaded") from None


# ---------------------------------------------------------------------- registries
_REGISTRIES: Dict[str, Dict[str, Type["Part"]]] = {
    "mixer": {}, "feed_forward": {}, "norm": {}, "position": {}, "block": {},
    "embedding": {}, "head": {}, "junction": {},
}


def register(category: str, kind: str) -> Callable[[Type["Part"]], Type["Part"]]:
    """Class decorator: make ``kind`` buildable as a part of ``category``."""
    if category not in _REGISTRIES:
        raise KeyError(f"unknown part category '{category}' (known: {sorted(_REGISTRIES)})")

    def deco(cls: Type["Part"]) -> Type["Part"]:
        _REGISTRIES[category][kind] = cls
        cls.category = category
        cls.kind = kind
        return cls

    return deco


def lookup(category: str, kind: str) -> Type["Part"]:
    reg = _REGISTRIES[category]
    if kind not in reg:
        raise KeyError(f"no {category} of kind '{kind}' is registered (known: {sorted(reg)})")
    return reg[kind]


def create(category: str, spec: PartSpec, prefix: str, ctx: BuildContext) -> "Part":
    return lookup(category, spec.kind)(spec.params, prefix, ctx)


def tensor_specs(category: str, spec: PartSpec, prefix: str) -> List[TensorSpec]:
    return lookup(category, spec.kind).tensor_specs(spec.params, prefix)


def join(prefix: str, name: str) -> str:
    """``prefix.name``; an empty name is the prefix itself (a part whose one tensor is stored
    under the part's own name)."""
    if not name:
        return prefix
    return f"{prefix}.{name}" if prefix else name


# ---------------------------------------------------------------------- base classes
class Part:
    category = ""
    kind = ""
    # True when the part's forward launches only device work that reads the step's device
    # tensors (no host decision on device data, no synchronisation), so that a decode step may
    # be captured into a HIP graph and replayed with new metadata.  A model's decode steps are
    # captured only when every part of it says so; a new part starts out on the safe side.
    graph_safe = False

    @classmethod
    def tensor_specs(cls, params: Dict[str, Any], prefix: str) -> List[TensorSpec]:
        """The checkpoint tensors this part reads, by full name."""
        return []

    def __init__(self, params: Dict[str, Any], prefix: str, ctx: BuildContext):
        self.params = params
        self.prefix = prefix


class Norm(Part):
    """``forward(stream)`` returns the normalised activations ``(T, H)`` in the activation
    dtype; it first adds the stream's pending delta into the 32-bit residual (one fused pass).
    ``forward_rows(stream, rows)`` does the same for the selected rows only and leaves the
    residual untouched."""

    def forward(self, stream: "ResidualStream") -> torch.Tensor:
        raise NotImplementedError

    def forward_rows(self, stream: "ResidualStream", rows: torch.Tensor) -> torch.Tensor:
        raise NotImplementedError

    def join(self, stream: "ResidualStream", delta: torch.Tensor,
             out_dtype: Optional[torch.dtype]) -> Optional[torch.Tensor]:
        """``x += norm(delta)`` in the 32-bit residual (``delta`` whole, or a stack of float32
        partial sums); returns the new residual in ``out_dtype`` (None: nothing).  For blocks
        whose norms stand behind their sublayers; a norm that has no such kernel has no such
        use."""
        raise NotImplementedError

    def fused_linear(self, stream: "ResidualStream", w: torch.Tensor, out_dtype: torch.dtype,
                     gated: bool, rows: Optional[torch.Tensor]) -> Optional[torch.Tensor]:
        """The norm and the projection behind it in one kernel: ``norm(stream) @ w.T`` (gated:
        ``silu(. @ Wg.T) * (. @ Wu.T)`` for ``w = [Wg; Wu]``), with the effects of ``forward``
        (or ``forward_rows``) on the stream.  None when this norm has no such kernel for these
        operands; the caller then applies the norm and the projection one after the other."""
        return None


class NormedInput:
    """A norm that has not been applied yet, handed to a part that sets ``takes_normed_input``
    in place of the normalised activations, so that the part's first projection can take the
    norm into its kernel.  ``tensor()`` applies the norm now; ``linear(w, ...)`` is the
    projection of the normalised activations."""

    __slots__ = ("norm", "stream", "rows")

    def __init__(self, norm: Norm, stream: "ResidualStream", rows: Optional[torch.Tensor] = None):
        self.norm, self.stream, self.rows = norm, stream, rows

    def tensor(self) -> torch.Tensor:
        if self.rows is None:
            return self.norm.forward(self.stream)
        return self.norm.forward_rows(self.stream, self.rows)

    def linear(self, w: torch.Tensor, out_dtype: torch.dtype, gated: bool = False) -> torch.Tensor:
        y = self.norm.fused_linear(self.stream, w, out_dtype, gated, self.rows)
        if y is None:
            from .. import ops
            x = self.tensor()
            y = ops.linear_swiglu(x, w) if gated else ops.linear(x, w, out_dtype)
        return y


def project(x: Any, w: torch.Tensor, out_dtype: torch.dtype, gated: bool = False) -> torch.Tensor:
    """``x @ w.T`` (or the gated form) for activations ``x`` or a ``NormedInput``."""
    if isinstance(x, NormedInput):
        return x.linear(w, out_dtype, gated)
    from .. import ops
    return ops.linear_swiglu(x, w) if gated else ops.linear(x, w, out_dtype)


def normed(norm: Norm, stream: "ResidualStream", consumer: Part,
           rows: Optional[torch.Tensor] = None) -> Any:
    """What ``consumer`` gets from ``norm``: the norm itself, unapplied, when it asks for that."""
    if getattr(consumer, "takes_normed_input", False):
        return NormedInput(norm, stream, rows)
    return norm.forward(stream) if rows is None else norm.forward_rows(stream, rows)


class PositionEncoding(Part):
    """Built once per distinct parameter set and shared by the mixers that name it."""


class Mixer(Part):
    """``forward(x, step, binding)`` maps activations ``(T, H)`` to ``(T, H)``.  The result goes
    to the residual stream, so it may also be a stack ``(S, T, H)`` of float32 partial sums
    (what ``ops.linear(..., partials=True)`` returns), which the stream adds in order, or the
    last projection not run yet (what ``ops.pending_linear`` returns), which the norm behind
    it may run with the add inside; ``as_tensor`` gives the tensor either way.

    ``cache_request()`` says what the mixer keeps in pages (None: nothing);
    ``state_bytes()`` how many bytes of fixed-size state it keeps per request (0: none).  A
    mixer with state must leave, after a step, the state as it is after the last token the
    step brought for that request.  ``step_planner()`` names the host-side planning its kernels
    need per step (None: the common metadata is enough)."""

    # True when forward takes ``x`` as a NormedInput (and projects it with ``project``).
    takes_normed_input = False

    def cache_request(self) -> Optional[CacheRequest]:
        return None

    def step_planner(self) -> Optional[StepPlanner]:
        return None

    def state_bytes(self) -> int:
        return 0

    def forward(self, x: torch.Tensor, step: Any, binding: CacheBinding) -> torch.Tensor:
        raise NotImplementedError


class FeedForward(Part):
    """``forward(x, step)`` maps activations ``(T, H)`` to ``(T, H)``, row by row (or to a
    stack of float32 partial sums of that, or to a projection that has not run yet, as a mixer
    may)."""

    takes_normed_input = False       # as for a mixer

    def forward(self, x: torch.Tensor, step: Any) -> torch.Tensor:
        raise NotImplementedError


class Block(Part):
    """Arranges a mixer, a feed-forward and their norms around the residual stream."""

    mixer: Mixer

    def forward(self, stream: "ResidualStream", step: Any, binding: CacheBinding) -> None:
        raise NotImplementedError


class Junction(Part):
    """Something that happens to the residual stream between two layer runs.  ``begin(stream)``
    is called once a step, on the embedding output in front of the first layer, and keeps what
    the part wants of it for the step; ``forward(stream, kept)`` gets that back wherever the run
    order names the part."""

    def begin(self, stream: "ResidualStream") -> Any:
        return None

    def forward(self, stream: "ResidualStream", kept: Any) -> None:
        raise NotImplementedError


class Embedding(Part):
    # True when forward also takes the step and the part's binding (``forward(ids, positions,
    # step=..., binding=...)``): a part that looks at earlier tokens or keeps state per request.
    wants_step = False
    # positions the part can place (a table of learned position vectors has so many rows);
    # None: any
    position_rows: Optional[int] = None

    def state_bytes(self) -> int:
        """Bytes of fixed-size state the part keeps per request (as for a mixer)."""
        return 0

    def forward(self, ids: torch.Tensor, positions: Optional[torch.Tensor] = None) -> torch.Tensor:
        """Token ids ``(T)`` int32 (and their absolute positions ``(T)`` int32, for a part that
        adds something per position) -> residual stream ``(T, H)`` float32."""
        raise NotImplementedError


class Head(Part):
    takes_normed_input = False       # as for a mixer

    def forward(self, x: torch.Tensor) -> torch.Tensor:
        """Normalised rows ``(R, H)`` -> logits ``(R, V)`` float32."""
        raise NotImplementedError


def as_tensor(delta: Any) -> torch.Tensor:
    """What a mixer or a feed-forward returned, as one ``(T, H)`` tensor: a projection that has
    not run yet runs now, a stack of partial sums is added up."""
    if not isinstance(delta, torch.Tensor):
        delta = delta.run()
    return delta.sum(0) if delta.dim() == 3 else delta


class LaneSet:
    """Several residual streams side by side (hyper-connections): ``count`` float32 tensors
    ``(T, H)`` that start out equal to the stream they were made from.  A sublayer reads a
    weighted sum of them through its norm (``reading`` names the weights of the next read),
    and its result comes back into all of them at once: ``update(y, mix, back)`` leaves
    ``lanes'[t] = sum_s mix[s, t] lanes[s] + back[t] y`` *pending*, so that the next read does
    the update and the read in one pass (``ops.lanes_step``).  ``total()`` is the plain sum of
    the streams."""

    __slots__ = ("count", "lanes", "pending", "read", "round_parts")

    def __init__(self, x: torch.Tensor, count: int, round_parts: bool):
        self.count = int(count)
        self.lanes = x                 # (T, H) while all streams are equal, then (count, T, H)
        self.pending: Any = None       # (y, mix, back)
        self.read: Optional[torch.Tensor] = None
        self.round_parts = round_parts

    def reading(self, weights: Optional[torch.Tensor]) -> None:
        self.read = weights

    def update(self, y: Any, mix: torch.Tensor, back: torch.Tensor) -> None:
        if self.pending is not None:
            self.settle()
        if not isinstance(y, torch.Tensor):
            y = y.run()
        self.pending = (y, mix, back)

    def settle(self) -> None:
        from .. import ops
        if self.pending is not None:
            self.lanes, _ = ops.lanes_step(self.lanes, self.count, update=self.pending,
                                           round_parts=self.round_parts, want=False)
            self.pending = None

    def normed(self, weight: Optional[torch.Tensor], eps: float, out_dtype: torch.dtype,
               rows: Optional[torch.Tensor] = None) -> torch.Tensor:
        """The pending update, then the read-out through the norm (``weight`` None: as it is,
        float32).  With ``rows`` only those tokens, and the streams stay as they are."""
        from .. import ops
        lanes, out = ops.lanes_step(self.lanes, self.count, update=self.pending, read=self.read,
                                    norm_weight=weight, eps=eps, out_dtype=out_dtype, rows=rows,
                                    round_parts=self.round_parts)
        if rows is None:
            self.lanes, self.pending = lanes, None
        return out

    def total(self) -> torch.Tensor:
        self.reading(None)
        if self.lanes.dim() == 2 and self.pending is None:
            return self.lanes * float(self.count) if self.count != 1 else self.lanes
        return self.normed(None, 0.0, torch.float32)


class ResidualStream:
    """The residual sum, kept in 32-bit, plus a delta that has not been added yet.

    A block's output is left *pending* so that the next norm can add it and normalise in one
    pass over the row; the sum itself is always formed and stored in float32.  A block's output
    joins the sum rounded once to the activation dtype: a delta that arrives as a stack of
    float32 partial sums is added up and, in a bfloat16 model, rounded to bfloat16 first
    (``round_parts``), as a delta that arrives whole in bfloat16 was by its kernel, so that the
    rounding does not depend on which kernel a batch's size chose."""

    __slots__ = ("x", "pending", "pending_scale", "pending_norm", "round_parts", "history",
                 "lanes", "act_dtype")

    def __init__(self, x: torch.Tensor, act_dtype: torch.dtype = torch.float32):
        assert x.dtype == torch.float32
        self.x = x
        # a tensor, or a product that has not run yet (``ops.pending_linear``), which a norm
        # may run with the add and its own multiplies inside
        self.pending: Any = None
        # the multiplier with which the pending delta joins the sum (in float32, by whoever
        # adds it); a norm's fused forms take deltas with multiplier 1 only
        self.pending_scale = 1.0
        # the norm that the pending delta passes on its way into the sum (blocks whose norms
        # stand behind their sublayers); such a delta is folded in by ``rows`` or ``flush``
        self.pending_norm: Optional[Norm] = None
        self.act_dtype = act_dtype
        self.round_parts = act_dtype == torch.bfloat16
        # (slots, T, H) float32: the embedding output and the layers' results so far, for
        # blocks that feed the next layer a mix of them (made by the first such block)
        self.history: Optional[torch.Tensor] = None
        # several streams in place of ``x`` (made by the first block that keeps them); norms
        # read them through ``LaneSet.normed``, ``merge_lanes`` makes ``x`` their sum again
        self.lanes: Optional[LaneSet] = None

    def split_lanes(self, count: int) -> LaneSet:
        """``count`` streams that all start as the residual sum; ``x`` is theirs from now on."""
        if self.lanes is None:
            self.lanes = LaneSet(self.flush(), count, self.round_parts)
        elif self.lanes.count != count:
            raise ValueError(f"the step keeps {self.lanes.count} residual streams, a block "
                             f"asks for {count}")
        return self.lanes

    def merge_lanes(self) -> None:
        """One stream again: the sum of the streams."""
        if self.lanes is not None:
            self.x, self.lanes = self.lanes.total(), None

    def add(self, delta: Any, scale: float = 1.0, norm: Optional[Norm] = None) -> None:
        if self.pending is not None:
            self.flush()
        self.pending = delta
        self.pending_scale = float(scale)
        self.pending_norm = norm

    def rows(self) -> torch.Tensor:
        """The residual itself (a pending delta folded in) in the activation dtype, for
        sublayers without a norm in front."""
        from .. import ops
        norm, self.pending_norm = self.pending_norm, None
        if norm is None:
            self.flush()
            return ops.norm_join(self.x, None, None, 0.0, self.act_dtype)
        return norm.join(self, self.take_raw(), self.act_dtype)

    def take_delta(self) -> Tuple[Optional[torch.Tensor], float]:
        """The pending delta as a tensor with its multiplier; the stream then has none."""
        if self.pending_norm is not None:
            self.flush()
        delta, scale = self.delta(), self.pending_scale
        self.pending, self.pending_scale = None, 1.0
        return delta, scale

    def take_raw(self) -> torch.Tensor:
        """The pending delta as a tensor, in front of the norm it is to pass (the caller applies
        that); the stream then has none."""
        self.pending_norm = None
        delta, self.pending = self.delta(), None
        return delta

    def delta(self) -> Optional[torch.Tensor]:
        """The pending delta as a tensor (a product that has not run yet runs now)."""
        if self.pending_norm is not None:
            self.flush()
        if self.pending is not None and not isinstance(self.pending, torch.Tensor):
            self.pending = self.pending.run()
        return self.pending

    def flush(self) -> torch.Tensor:
        """Fold a pending delta into the residual and return the residual."""
        if self.pending is not None and self.pending_norm is not None:
            norm = self.pending_norm
            norm.join(self, self.take_raw(), None)
        if self.pending is not None:
            from .. import ops
            ops.add_residual(self.x, self.delta(), round_parts=self.round_parts,
                             delta_scale=self.pending_scale)
            self.pending, self.pending_scale = None, 1.0
        return self.x
