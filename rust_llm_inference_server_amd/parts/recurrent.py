"""Mixers that keep a state of fixed size per request, and one that runs two mixers side by
side.

``time_mix`` (RWKV-style): every projection reads its own blend of the token's input and the
previous token's; per head a matrix state S (key channel x value channel) that each token
decays per key channel and writes ``k v^T`` into, read with a bonus for the current token.

``gated_delta``: q, k and v pass a short causal convolution and SiLU, q and k become unit
vectors; per head S decays by one factor, then the token overwrites what its key reads
(``u = beta (v - S^T k)``, ``S += k u^T``) and reads with its query.

Both keep S in float32 in the request's state slot together with the inputs of the last
tokens that the next step's first token needs (one row for the token shift, taps - 1 rows for
the convolution), walk a sequence's tokens in order with whatever else the batch holds, and
leave the state as after the step's last token.  What enters a recurrence (decays, step
sizes, unit norms, the state itself) is float32 in either activation dtype; the projections
that feed it store float32 results.

``selective_scan`` (Mamba): the input passes a short causal convolution and SiLU; a state of N
numbers per channel decays by ``exp(dt A)`` with a step ``dt`` that the token chooses, takes
``dt x B`` and is read with ``C``; the result is gated by ``silu(z)``.

``decay_attention`` (linear attention with a fixed decay per head): q, k and v pass SiLU; per
head ``S <- decay_h S + k v^T`` and the read-out ``S^T q`` includes the token's own key and
value; the heads' read-outs are normalised together, gated by a sigmoid and projected.

``channel_delta``: the gated delta rule with one decay per head and key channel (a low-rank
projection of the token's input), a write that its own token already reads, and a sigmoid gate
(low-rank too) behind the heads' norm.

``rglru`` (a real-gated linear recurrent unit): one number per channel behind a short
convolution decays by ``a = exp(-c r softplus(lam))`` and takes ``sqrt(1 - a^2) i u``, the gates r
and i being block-diagonal products of u; the result meets a GELU branch of the input.

``parallel``: two mixers read the same input, and their outputs meet as a weighted sum in
float32.  Each keeps what it keeps: the pages of the one that asks for a cache, the state
bytes of both, one after the other.
"""
from __future__ import annotations

from typing import Any, Dict, List, Optional

import torch

from .. import ops
from .base import (BuildContext, CacheBinding, CacheRequest, Mixer, NormedInput, PartSpec,
                   TensorSpec, create, join, project, register, tensor_specs)


def _f32(t: torch.Tensor) -> torch.Tensor:
    return t.to(torch.float32).contiguous()


def _state_views(binding: CacheBinding, first: int):
    """The mixer's state area as float32, cut into its first ``first`` floats and the rest."""
    if binding.state is None:
        raise ValueError("this mixer needs a state slot per request; the runner has none")
    st = binding.state.view(torch.float32)
    return st[:, :first], st[:, first:]


def _ran(delta: Any) -> torch.Tensor:
    """A mixer's result as a tensor, whole or as a stack of float32 partial sums; a projection
    that has not run yet runs now."""
    return delta if isinstance(delta, torch.Tensor) else delta.run()


# ------------------------------------------------------------------------------ time mix
@register("mixer", "time_mix")
class TimeMix(Mixer):
    """Parameters: ``hidden_size``, ``num_heads``, ``head_dim`` (keys, values and receptances
    share it), ``decay_rank`` (rows of ``w1``), ``eps`` (of the per-head norm of the read-out).

    Tensors under the prefix: ``mu.r|k|v|g|w`` (W) blend weights; ``r``, ``k``, ``v``, ``g``
    (heads * d, W); ``w1`` (rank, W), ``w2`` (heads * d, rank), ``w0`` (heads * d): the decay
    ``exp(-exp(w2 tanh(w1 x_w) + w0))``; ``u`` (heads, d) the bonus; ``norm`` (heads * d);
    ``o`` (W, heads * d)."""

    graph_safe = True
    MIXES = ("r", "k", "v", "g", "w")

    @classmethod
    def tensor_specs(cls, params: Dict[str, Any], prefix: str) -> List[TensorSpec]:
        W, H, d = params["hidden_size"], params["num_heads"], params["head_dim"]
        rank = params["decay_rank"]
        out = [TensorSpec(join(prefix, f"mu.{m}"), (W,), std=0.3) for m in cls.MIXES]
        out += [TensorSpec(join(prefix, n), (H * d, W)) for n in ("r", "k", "v", "g")]
        out += [TensorSpec(join(prefix, "w1"), (rank, W)),
                TensorSpec(join(prefix, "w2"), (H * d, rank)),
                TensorSpec(join(prefix, "w0"), (H * d,)), TensorSpec(join(prefix, "u"), (H, d)),
                TensorSpec(join(prefix, "norm"), (H * d,), init="ones_normal"),
                TensorSpec(join(prefix, "o"), (W, H * d))]
        return out

    def __init__(self, params: Dict[str, Any], prefix: str, ctx: BuildContext):
        super().__init__(params, prefix, ctx)
        self.width = int(params["hidden_size"])
        self.heads, self.dim = int(params["num_heads"]), int(params["head_dim"])
        self.eps = float(params["eps"])
        take = lambda n: ctx.take(join(prefix, n))
        self.mu = torch.stack([_f32(take(f"mu.{m}")) for m in self.MIXES]).contiguous()
        self.w_r, self.w_k, self.w_v, self.w_g = take("r"), take("k"), take("v"), take("g")
        self.w_1, self.w_2 = take("w1"), take("w2")
        self.w0, self.bonus, self.norm = _f32(take("w0")), _f32(take("u")), _f32(take("norm"))
        self.w_o = take("o")
        self.act_dtype = ctx.act_dtype

    def state_bytes(self) -> int:
        return 4 * (self.width + self.heads * self.dim * self.dim)

    def forward(self, x: torch.Tensor, step: Any, binding: CacheBinding) -> Any:
        tail, S = _state_views(binding, self.width)
        cu, slots, n = step.cu_seqlens, step.state_slots, step.num_seqs
        mixes = ops.shift_mix(x, self.mu, tail, step.seq_of_token, cu, slots, n)
        ops.tail_update(tail, x, self.width, 1, cu, slots, n)
        f32 = torch.float32
        r = ops.linear_f32(mixes[0], self.w_r)
        k = ops.linear_f32(mixes[1], self.w_k)
        v = ops.linear_f32(mixes[2], self.w_v)
        gate = ops.linear_f32(mixes[3], self.w_g)
        low = ops.soft_cap_(ops.linear(mixes[4], self.w_1, self.act_dtype), 1.0)     # tanh
        z = ops.linear(low, self.w_2, f32)
        o = ops.decay_scan(r, k, v, z, self.w0, self.bonus, S, cu, slots, n, self.heads, self.dim)
        y = ops.head_norm_gate(o, self.norm, gate, self.heads, self.dim, self.eps, self.act_dtype)
        return ops.pending_linear(y, self.w_o, self.act_dtype)


# --------------------------------------------------------------------------- gated delta
@register("mixer", "gated_delta")
class GatedDelta(Mixer):
    """Parameters: ``hidden_size``, ``num_heads`` (value heads), ``num_kv_heads`` (query/key
    heads; value head h uses head ``h // (heads / kv_heads)``), ``head_dim``, ``value_dim``,
    ``conv`` (taps), ``eps`` (of the per-head norm of the read-out).

    Tensors under the prefix: ``q``, ``k`` (kv_heads * d, W), ``v`` (heads * dv, W), each with
    ``.conv`` (channels, taps); ``b``, ``a`` (heads, W); ``A_log``, ``dt_bias`` (heads);
    ``g`` (heads * dv, W); ``norm`` (dv); ``o`` (W, heads * dv).

    One product makes q, k, v, the gate and the raw step size and decay (rows concatenated, each
    part starting on a multiple of 8 columns), stored in float32."""

    graph_safe = True
    takes_normed_input = True        # the norm in front goes into the one input product where it can
    UNIT_EPS = 1e-6

    @classmethod
    def tensor_specs(cls, params: Dict[str, Any], prefix: str) -> List[TensorSpec]:
        W, H, G = params["hidden_size"], params["num_heads"], params["num_kv_heads"]
        d, dv, taps = params["head_dim"], params["value_dim"], params["conv"]
        out = []
        for n, rows in (("q", G * d), ("k", G * d), ("v", H * dv)):
            out += [TensorSpec(join(prefix, n), (rows, W)),
                    TensorSpec(join(prefix, f"{n}.conv"), (rows, taps), std=0.3)]
        out += [TensorSpec(join(prefix, "b"), (H, W)), TensorSpec(join(prefix, "A_log"), (H,)),
                TensorSpec(join(prefix, "norm"), (dv,), init="ones_normal"),
                TensorSpec(join(prefix, "a"), (H, W)), TensorSpec(join(prefix, "dt_bias"), (H,)),
                TensorSpec(join(prefix, "g"), (H * dv, W)), TensorSpec(join(prefix, "o"), (W, H * dv))]
        return out

    def __init__(self, params: Dict[str, Any], prefix: str, ctx: BuildContext):
        super().__init__(params, prefix, ctx)
        self.width = int(params["hidden_size"])
        self.heads, self.kv_heads = int(params["num_heads"]), int(params["num_kv_heads"])
        self.dim, self.vdim = int(params["head_dim"]), int(params["value_dim"])
        self.taps = int(params["conv"])
        self.eps = float(params["eps"])
        if self.heads % self.kv_heads:
            raise ValueError(f"gated_delta: {self.heads} heads are not a multiple of "
                             f"{self.kv_heads} query/key heads")
        if not 1 <= self.taps <= 16:
            raise ValueError(f"gated_delta: {self.taps} taps (1 to 16)")
        take = lambda n: ctx.take(join(prefix, n))
        G, H, d, dv = self.kv_heads, self.heads, self.dim, self.vdim
        self.conv_channels = C = 2 * G * d + H * dv
        parts = [take("q"), take("k"), take("v"), take("g"), take("b"), take("a")]
        if len({p.dtype for p in parts}) > 1:
            parts = [p.to(torch.float32) for p in parts]
        # column ranges of the one product: q | k | v | gate | b | a, each from a multiple of 8
        self.cols: Dict[str, int] = {}
        rows, at = [], 0
        for name, p in zip(("q", "k", "v", "g", "b", "a"), parts):
            if name in ("g", "b", "a"):
                pad = -at % 8
                if pad:
                    rows.append(p.new_zeros((pad, self.width)))
                    at += pad
            self.cols[name] = at
            rows.append(p)
            at += p.shape[0]
        if at % 8:
            rows.append(parts[0].new_zeros((-at % 8, self.width)))
        self.w_in = torch.cat(rows, dim=0).contiguous()
        self.conv_w = torch.cat([_f32(take(f"{n}.conv")) for n in "qkv"], dim=0).contiguous()
        self.a_log, self.dt_bias = _f32(take("A_log")), _f32(take("dt_bias"))
        self.norm = _f32(take("norm"))
        self.w_o = take("o")
        self.act_dtype = ctx.act_dtype

    def state_bytes(self) -> int:
        return 4 * ((self.taps - 1) * self.conv_channels + self.heads * self.vdim * self.dim)

    def forward(self, x: Any, step: Any, binding: CacheBinding) -> Any:
        G, H, d, dv, C = self.kv_heads, self.heads, self.dim, self.vdim, self.conv_channels
        tail, S = _state_views(binding, (self.taps - 1) * C)
        cu, slots, n = step.cu_seqlens, step.state_slots, step.num_seqs
        if isinstance(x, NormedInput) and not ops.can_fuse_norm_linear(
                x.stream.x, self.w_in, x.stream.x.shape[0]):
            x = x.tensor()
        p = (project(x, self.w_in, torch.float32) if isinstance(x, NormedInput)
             else ops.linear_f32(x, self.w_in))                           # (T, q|k|v|g|b|a)
        qkv = ops.causal_conv(p, self.conv_w, tail, step.seq_of_token, cu, slots, n,
                              unit_channels=2 * G * d, unit_group=d, scaled_channels=G * d,
                              scale=d ** -0.5, unit_eps=self.UNIT_EPS, rest_group=dv,
                              keep_tail=True)
        c = self.cols
        o = ops.delta_scan(qkv[:, :G * d], qkv[:, G * d:2 * G * d], qkv[:, 2 * G * d:],
                           p[:, c["b"]:c["b"] + H], p[:, c["a"]:c["a"] + H], self.a_log,
                           self.dt_bias, S, cu, slots, n, H, G, d, dv)
        y = ops.head_norm_gate(o, self.norm, p[:, c["g"]:c["g"] + H * dv], H, dv, self.eps,
                               self.act_dtype)
        return ops.pending_linear(y, self.w_o, self.act_dtype)


# ------------------------------------------------------------------------ selective scan
@register("mixer", "selective_scan")
class SelectiveScan(Mixer):
    """Parameters: ``hidden_size``, ``inner`` (channels), ``state`` (numbers per channel),
    ``dt_rank``, ``conv`` (taps).

    Tensors under the prefix: ``in`` (2 * inner, W): x in front of z; ``conv`` (inner, taps)
    and ``conv.b`` (inner); ``x`` (dt_rank + 2 * state, inner): the step's low-rank input, B
    and C; ``dt`` (inner, dt_rank) and ``dt.b`` (inner); ``A_log`` (inner, state); ``D``
    (inner); ``o`` (W, inner).

    Per token and channel: ``dt = softplus(W_dt low + dt.b)``, ``S <- exp(dt A) S + dt x B``
    with ``A = -exp(A_log)``, ``y = S . C + D x``, result ``y * silu(z)``.  The state slot holds
    the last ``conv - 1`` inputs of the convolution and S, float32; steps, decays and the state
    are float32 in either activation dtype."""

    graph_safe = True

    @classmethod
    def tensor_specs(cls, params: Dict[str, Any], prefix: str) -> List[TensorSpec]:
        W, C, N = params["hidden_size"], params["inner"], params["state"]
        rank, taps = params["dt_rank"], params["conv"]
        return [TensorSpec(join(prefix, "in"), (2 * C, W)),
                TensorSpec(join(prefix, "conv"), (C, taps), std=0.3),
                TensorSpec(join(prefix, "conv.b"), (C,)),
                TensorSpec(join(prefix, "x"), (rank + 2 * N, C)),
                TensorSpec(join(prefix, "dt"), (C, rank), std=0.3),
                TensorSpec(join(prefix, "dt.b"), (C,), std=0.5),
                TensorSpec(join(prefix, "A_log"), (C, N), std=0.5),
                TensorSpec(join(prefix, "D"), (C,), init="ones_normal"),
                TensorSpec(join(prefix, "o"), (W, C))]

    def __init__(self, params: Dict[str, Any], prefix: str, ctx: BuildContext):
        super().__init__(params, prefix, ctx)
        self.channels, self.states = int(params["inner"]), int(params["state"])
        self.rank, self.taps = int(params["dt_rank"]), int(params["conv"])
        if not 1 <= self.taps <= 16:
            raise ValueError(f"selective_scan: {self.taps} taps (1 to 16)")
        take = lambda n: ctx.take(join(prefix, n))
        self.w_in, self.w_x, self.w_dt, self.w_o = take("in"), take("x"), take("dt"), take("o")
        self.conv_w, self.conv_b = _f32(take("conv")), _f32(take("conv.b"))
        self.dt_bias, self.a_log, self.skip = _f32(take("dt.b")), _f32(take("A_log")), _f32(take("D"))
        self.act_dtype = ctx.act_dtype

    def state_bytes(self) -> int:
        return 4 * ((self.taps - 1) * self.channels + self.channels * self.states)

    def forward(self, x: torch.Tensor, step: Any, binding: CacheBinding) -> Any:
        C, N, rank = self.channels, self.states, self.rank
        tail, S = _state_views(binding, (self.taps - 1) * C)
        cu, slots, n = step.cu_seqlens, step.state_slots, step.num_seqs
        xz = ops.linear_f32(x, self.w_in)                                  # (T, x | z)
        xc = ops.causal_conv(xz, self.conv_w, tail, step.seq_of_token, cu, slots, n,
                             bias=self.conv_b, out_dtype=self.act_dtype, keep_tail=True)
        low = ops.linear_f32(xc, self.w_x)                                 # (T, dt | B | C)
        dt_raw = ops.linear(low[:, :rank], self.w_dt, torch.float32)
        y = ops.selective_scan(xc, dt_raw, self.dt_bias, low[:, rank:rank + N],
                               low[:, rank + N:rank + 2 * N], xz[:, C:], self.a_log, self.skip,
                               S, cu, slots, n)
        return ops.pending_linear(y, self.w_o, self.act_dtype)


# ----------------------------------------------------------------------- decay attention
@register("mixer", "decay_attention")
class DecayAttention(Mixer):
    """Parameters: ``hidden_size``, ``num_heads``, ``head_dim`` (queries and keys),
    ``value_dim``, ``decay`` (one number in (0, 1] per head), ``eps`` (of the norm over the
    concatenated heads).

    Tensors under the prefix: ``q``, ``k`` (heads * d, W), ``v``, ``g`` (heads * dv, W),
    ``norm`` (heads * dv), ``o`` (W, heads * dv).

    Per token: ``q, k, v = silu(W h)``; per head ``S <- decay_h S + k v^T``, ``o = S^T q`` (no
    other scale); the concatenated heads are divided by their root mean square, multiplied by
    ``norm`` and by ``sigmoid(W_g h)``, and projected by ``o``.  One product makes q, k, v and
    the gate (rows concatenated), stored in float32; SiLU, the state (float32, in the request's
    slot, [head][value channel][key channel]), the norm and the gate are float32 in either
    activation dtype."""

    graph_safe = True
    takes_normed_input = True        # the norm in front goes into the one input product where it can

    @classmethod
    def tensor_specs(cls, params: Dict[str, Any], prefix: str) -> List[TensorSpec]:
        W, H = params["hidden_size"], params["num_heads"]
        d, dv = params["head_dim"], params["value_dim"]
        return [TensorSpec(join(prefix, "q"), (H * d, W)), TensorSpec(join(prefix, "k"), (H * d, W)),
                TensorSpec(join(prefix, "v"), (H * dv, W)), TensorSpec(join(prefix, "g"), (H * dv, W)),
                TensorSpec(join(prefix, "o"), (W, H * dv)),
                TensorSpec(join(prefix, "norm"), (H * dv,), init="ones_normal")]

    def __init__(self, params: Dict[str, Any], prefix: str, ctx: BuildContext):
        super().__init__(params, prefix, ctx)
        self.width = int(params["hidden_size"])
        self.heads = int(params["num_heads"])
        self.dim, self.vdim = int(params["head_dim"]), int(params["value_dim"])
        self.eps = float(params["eps"])
        decay = [float(x) for x in params["decay"]]
        if len(decay) != self.heads or not all(0.0 < x <= 1.0 for x in decay):
            raise ValueError(f"decay_attention: {self.heads} heads need a decay in (0, 1] each, "
                             f"got {decay}")
        if self.dim > 256:
            raise ValueError(f"decay_attention: heads of {self.dim} key channels (at most 256)")
        self.decay = torch.tensor(decay, dtype=torch.float32, device=ctx.device)
        take = lambda n: ctx.weights.pop(join(prefix, n))
        parts = [take("q"), take("k"), take("v"), take("g")]
        if len({p.dtype for p in parts}) > 1:
            parts = [p.to(torch.float32) for p in parts]
        # column ranges of the one product: q | k | v | gate, each from a multiple of 8
        self.cols: Dict[str, int] = {}
        rows, at = [], 0
        for name, p in zip("qkvg", parts):
            pad = -at % 8
            if pad:
                rows.append(p.new_zeros((pad, self.width)))
                at += pad
            self.cols[name] = at
            rows.append(p)
            at += p.shape[0]
        if at % 8:
            rows.append(parts[0].new_zeros((-at % 8, self.width)))
        self.w_in = torch.cat(rows, dim=0).contiguous()
        del parts, rows
        self.norm = _f32(ctx.take(join(prefix, "norm")))
        self.w_o = ctx.take(join(prefix, "o"))
        self.act_dtype = ctx.act_dtype

    def state_bytes(self) -> int:
        return 4 * self.heads * self.vdim * self.dim

    def forward(self, x: Any, step: Any, binding: CacheBinding) -> Any:
        H, d, dv = self.heads, self.dim, self.vdim
        if binding.state is None:
            raise ValueError("decay_attention needs a state slot per request; the runner has none")
        S = binding.state.view(torch.float32)
        cu, slots, n = step.cu_seqlens, step.state_slots, step.num_seqs
        if isinstance(x, NormedInput) and not ops.can_fuse_norm_linear(
                x.stream.x, self.w_in, x.stream.x.shape[0]):
            x = x.tensor()
        p = (project(x, self.w_in, torch.float32) if isinstance(x, NormedInput)
             else ops.linear_f32(x, self.w_in))                           # (T, q | k | v | gate)
        c = self.cols
        o = ops.decay_attention(p[:, c["q"]:c["q"] + H * d], p[:, c["k"]:c["k"] + H * d],
                                p[:, c["v"]:c["v"] + H * dv], self.decay, S, cu, slots, n,
                                H, d, dv, longest=getattr(step, "max_new", None))
        y = ops.head_norm_gate(o, self.norm, p[:, c["g"]:c["g"] + H * dv], 1, H * dv, self.eps,
                               self.act_dtype, sigmoid_gate=True)
        return ops.pending_linear(y, self.w_o, self.act_dtype)


# -------------------------------------------------------------------------- channel delta
@register("mixer", "channel_delta")
class ChannelDelta(Mixer):
    """Parameters: ``hidden_size``, ``num_heads`` (value heads), ``num_kv_heads`` (query/key
    heads; value head h uses head ``h // (heads / kv_heads)``), ``head_dim``, ``value_dim``,
    ``conv`` (taps), ``decay_rank``, ``gate_rank``, ``eps`` (of the per-head norm of the read-out).

    Tensors under the prefix: ``q``, ``k`` (kv_heads * d, W), ``v`` (heads * dv, W), each with
    ``.conv`` (channels, taps); ``b`` (heads, W); ``A_log`` (heads); ``a1`` (decay_rank, W), ``a2``
    (heads * d, decay_rank), ``dt_bias`` (heads * d); ``g1`` (gate_rank, W), ``g2`` (heads * dv,
    gate_rank); ``norm`` (dv); ``o`` (W, heads * dv).

    Per token and head, with ``g = exp(-exp(A_log) softplus(a2 (a1 h) + dt_bias))`` per key
    channel: ``S <- diag(g) S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q``, ``beta =
    sigmoid(b h)``, q and k unit vectors behind convolution and SiLU, q times ``d^-1/2``.

    One product makes q, k, v and b (stored float32); the two low-rank pairs share two products:
    ``[a1; g1]`` and the block-diagonal ``[a2 0; 0 g2]``."""

    graph_safe = True
    UNIT_EPS = 1e-6

    @classmethod
    def tensor_specs(cls, params: Dict[str, Any], prefix: str) -> List[TensorSpec]:
        W, H, G = params["hidden_size"], params["num_heads"], params["num_kv_heads"]
        d, dv, taps = params["head_dim"], params["value_dim"], params["conv"]
        ra, rg = params["decay_rank"], params["gate_rank"]
        out = []
        for n, rows in (("q", G * d), ("k", G * d), ("v", H * dv)):
            out += [TensorSpec(join(prefix, n), (rows, W)),
                    TensorSpec(join(prefix, f"{n}.conv"), (rows, taps), std=0.3)]
        out += [TensorSpec(join(prefix, "b"), (H, W)), TensorSpec(join(prefix, "A_log"), (H,)),
                TensorSpec(join(prefix, "norm"), (dv,), init="ones_normal"),
                TensorSpec(join(prefix, "a1"), (ra, W)), TensorSpec(join(prefix, "a2"), (H * d, ra)),
                TensorSpec(join(prefix, "dt_bias"), (H * d,)),
                TensorSpec(join(prefix, "g1"), (rg, W)), TensorSpec(join(prefix, "g2"), (H * dv, rg)),
                TensorSpec(join(prefix, "o"), (W, H * dv))]
        return out

    def __init__(self, params: Dict[str, Any], prefix: str, ctx: BuildContext):
        super().__init__(params, prefix, ctx)
        self.width = int(params["hidden_size"])
        self.heads, self.kv_heads = int(params["num_heads"]), int(params["num_kv_heads"])
        self.dim, self.vdim = int(params["head_dim"]), int(params["value_dim"])
        self.taps = int(params["conv"])
        self.eps = float(params["eps"])
        if self.heads % self.kv_heads:
            raise ValueError(f"channel_delta: {self.heads} heads are not a multiple of "
                             f"{self.kv_heads} query/key heads")
        if not 1 <= self.taps <= 16:
            raise ValueError(f"channel_delta: {self.taps} taps (1 to 16)")
        if self.dim > 256:
            raise ValueError(f"channel_delta: heads of {self.dim} key channels (at most 256)")
        pop = lambda n: ctx.weights.pop(join(prefix, n))
        take = lambda n: ctx.take(join(prefix, n))
        G, H, d, dv = self.kv_heads, self.heads, self.dim, self.vdim
        self.conv_channels = C = 2 * G * d + H * dv
        parts = [pop("q"), pop("k"), pop("v"), pop("b")]
        if len({p.dtype for p in parts}) > 1:
            parts = [p.to(torch.float32) for p in parts]
        # columns of the product: q | k | v | b, b from a multiple of 8
        self.b_at = -(-C // 8) * 8
        rows = parts[:3]
        if self.b_at > C:
            rows.append(parts[0].new_zeros((self.b_at - C, self.width)))
        rows.append(parts[3])
        if H % 8:
            rows.append(parts[0].new_zeros((-H % 8, self.width)))
        self.w_in = torch.cat(rows, dim=0).contiguous()
        del parts, rows
        self.conv_w = torch.cat([_f32(take(f"{n}.conv")) for n in "qkv"], dim=0).contiguous()
        a1, g1, a2, g2 = pop("a1"), pop("g1"), pop("a2"), pop("g2")
        if len({p.dtype for p in (a1, g1, a2, g2)}) > 1:
            a1, g1, a2, g2 = (p.to(torch.float32) for p in (a1, g1, a2, g2))
        ra, rg = a1.shape[0], g1.shape[0]
        at = -(-ra // 8) * 8
        self.w_low = a1.new_zeros((at + -(-rg // 8) * 8, self.width))
        self.w_low[:ra], self.w_low[at:at + rg] = a1, g1
        # (the second product's gate columns start on a multiple of 8 too)
        self.gate_at = -(-H * d // 8) * 8
        self.w_up = a2.new_zeros((self.gate_at + H * dv, self.w_low.shape[0]))
        self.w_up[:H * d, :ra], self.w_up[self.gate_at:, at:at + rg] = a2, g2
        self.a_log, self.dt_bias = _f32(take("A_log")), _f32(take("dt_bias"))
        self.norm = _f32(take("norm"))
        self.w_o = take("o")
        self.act_dtype = ctx.act_dtype

    def state_bytes(self) -> int:
        return 4 * ((self.taps - 1) * self.conv_channels + self.heads * self.vdim * self.dim)

    def forward(self, x: torch.Tensor, step: Any, binding: CacheBinding) -> Any:
        G, H, d, dv, C = self.kv_heads, self.heads, self.dim, self.vdim, self.conv_channels
        tail, S = _state_views(binding, (self.taps - 1) * C)
        cu, slots, n = step.cu_seqlens, step.state_slots, step.num_seqs
        p = ops.linear_f32(x, self.w_in)                                   # (T, q|k|v|b)
        up = ops.linear_f32(ops.linear(x, self.w_low, self.act_dtype), self.w_up)
        qkv = ops.causal_conv(p, self.conv_w, tail, step.seq_of_token, cu, slots, n,
                              unit_channels=2 * G * d, unit_group=d, scaled_channels=G * d,
                              scale=d ** -0.5, unit_eps=self.UNIT_EPS, rest_group=min(dv, 1024),
                              keep_tail=True)
        o = ops.channel_delta_scan(qkv[:, :G * d], qkv[:, G * d:2 * G * d], qkv[:, 2 * G * d:],
                                   p[:, self.b_at:self.b_at + H], up[:, :H * d], self.a_log,
                                   self.dt_bias, S, cu, slots, n, H, G, d, dv,
                                   longest=getattr(step, "max_new", None))
        y = ops.head_norm_gate(o, self.norm, up[:, self.gate_at:], H, dv, self.eps, self.act_dtype,
                               sigmoid_gate=True)
        return ops.pending_linear(y, self.w_o, self.act_dtype)


# --------------------------------------------------------- real-gated linear recurrent unit
@register("mixer", "rglru")
class RGLRU(Mixer):
    """Parameters: ``hidden_size``, ``width`` (channels), ``blocks`` (equal parts of the channels
    that the gates' products stay inside), ``conv`` (taps), ``power`` (the factor in the log
    decay).

    Tensors under the prefix: ``y``, ``x`` (width, W) with ``.b`` (width); ``conv`` (width, taps)
    and ``conv.b``; ``ra``, ``ri`` (blocks, n, n), each [out, in], with ``.b`` (blocks, n);
    ``lam`` (width); ``o`` (W, width).

    Per token and channel: ``u = conv(x h + x.b)`` (zeros in front of the sequence), ``r, i =
    sigmoid(ra u + ra.b), sigmoid(ri u + ri.b)`` block by block, ``log a = -power r
    softplus(lam)``, ``S <- a S + sqrt(1 - a^2) i u``, result ``S gelu(y h + y.b)`` (tanh form).
    The state slot holds the last ``conv - 1`` inputs of the convolution and S, float32."""

    graph_safe = True

    @classmethod
    def tensor_specs(cls, params: Dict[str, Any], prefix: str) -> List[TensorSpec]:
        W, C, B, taps = (params[k] for k in ("hidden_size", "width", "blocks", "conv"))
        n = C // B
        out = []
        for name in ("y", "x"):
            out += [TensorSpec(join(prefix, name), (C, W)), TensorSpec(join(prefix, name + ".b"), (C,))]
        out += [TensorSpec(join(prefix, "conv"), (C, taps), std=0.3),
                TensorSpec(join(prefix, "conv.b"), (C,))]
        for name in ("ra", "ri"):
            out += [TensorSpec(join(prefix, name), (B, n, n)),
                    TensorSpec(join(prefix, name + ".b"), (B, n))]
        return out + [TensorSpec(join(prefix, "lam"), (C,), std=0.5),
                      TensorSpec(join(prefix, "o"), (W, C))]

    def __init__(self, params: Dict[str, Any], prefix: str, ctx: BuildContext):
        super().__init__(params, prefix, ctx)
        self.width = int(params["hidden_size"])
        self.channels, self.blocks = int(params["width"]), int(params["blocks"])
        self.taps, self.power = int(params["conv"]), float(params["power"])
        if self.channels % self.blocks:
            raise ValueError(f"rglru: {self.channels} channels in {self.blocks} blocks")
        if not 1 <= self.taps <= 16:
            raise ValueError(f"rglru: {self.taps} taps (1 to 16)")
        pop = lambda n: ctx.weights.pop(join(prefix, n))
        take = lambda n: ctx.take(join(prefix, n))
        C = self.channels
        wx, wy = pop("x"), pop("y")
        if wx.dtype != wy.dtype:
            wx, wy = wx.to(torch.float32), wy.to(torch.float32)
        # columns of the one product: x | y, y from a multiple of 8
        self.y_at = -(-C // 8) * 8
        rows = [wx] + ([wx.new_zeros((self.y_at - C, self.width))] if self.y_at > C else []) + [wy]
        self.w_in = torch.cat(rows, dim=0).contiguous()
        del wx, wy, rows
        self.x_bias, self.y_bias = _f32(take("x.b")), _f32(take("y.b"))
        self.conv_w, self.conv_b = _f32(take("conv")), _f32(take("conv.b"))
        # per block the rows of ra in front of those of ri
        self.w_gates = torch.cat([pop("ra").to(ctx.act_dtype), pop("ri").to(ctx.act_dtype)],
                                 dim=1).contiguous()
        self.r_bias = _f32(take("ra.b")).reshape(-1).contiguous()
        self.i_bias = _f32(take("ri.b")).reshape(-1).contiguous()
        # -power softplus(lam), float32, made once
        self.rate = (-self.power * torch.nn.functional.softplus(
            take("lam").to(torch.float64), threshold=40.0)).to(torch.float32).contiguous()
        self.w_o = take("o")
        self.act_dtype = ctx.act_dtype

    def state_bytes(self) -> int:
        return 4 * self.taps * self.channels

    def forward(self, x: torch.Tensor, step: Any, binding: CacheBinding) -> Any:
        C, n = self.channels, self.channels // self.blocks
        tail, S = _state_views(binding, (self.taps - 1) * C)
        cu, slots, num = step.cu_seqlens, step.state_slots, step.num_seqs
        p = ops.linear_f32(x, self.w_in)                                   # (T, x | y)
        u = ops.causal_conv(p, self.conv_w, tail, step.seq_of_token, cu, slots, num,
                            bias=self.conv_b, out_dtype=self.act_dtype, activation=False,
                            in_bias=self.x_bias, keep_tail=True)
        gates = ops.head_linear(u, self.w_gates, n, out_dtype=torch.float32)
        y = ops.rglru_scan(u, gates, self.r_bias, self.i_bias, self.rate,
                           p[:, self.y_at:self.y_at + C], self.y_bias, S, cu, slots, num,
                           self.blocks, longest=getattr(step, "max_new", None))
        return ops.pending_linear(y, self.w_o, self.act_dtype)


# ------------------------------------------------------------------------------ parallel
@register("mixer", "parallel")
class ParallelMixers(Mixer):
    """Two mixers on one input: ``scale_a * a(x) + scale_b * b(x)``, the sum in float32.

    Parameters: ``branches``: two dicts ``{"mixer": PartSpec, "name": suffix under the prefix,
    "scale": number}``.  At most one branch may keep pages (the cache request and the step
    planner are that branch's); state bytes are the branches' one after the other."""

    @classmethod
    def tensor_specs(cls, params: Dict[str, Any], prefix: str) -> List[TensorSpec]:
        out: List[TensorSpec] = []
        for b in params["branches"]:
            out += tensor_specs("mixer", b["mixer"], join(prefix, b["name"]))
        return out

    def __init__(self, params: Dict[str, Any], prefix: str, ctx: BuildContext):
        super().__init__(params, prefix, ctx)
        branches = params["branches"]
        if len(branches) != 2:
            raise ValueError(f"parallel mixer: two branches, got {len(branches)}")
        self.branches: List[Mixer] = [create("mixer", b["mixer"], join(prefix, b["name"]), ctx)
                                      for b in branches]
        self.scales = [float(b["scale"]) for b in branches]
        with_cache = [m for m in self.branches if m.cache_request() is not None]
        if len(with_cache) > 1:
            raise ValueError("parallel mixer: only one branch may keep pages")
        self._cached: Optional[Mixer] = with_cache[0] if with_cache else None
        planners = [m.step_planner() for m in self.branches if m.step_planner() is not None]
        if len(planners) > 1:
            raise ValueError("parallel mixer: only one branch may bring a step planner")
        self._planner = planners[0] if planners else None
        self._offsets, at = [], 0
        for m in self.branches:
            n = int(m.state_bytes())
            self._offsets.append((at, n))
            at += -(-n // 16) * 16
        self._state_bytes = at

    @property
    def graph_safe(self) -> bool:
        return all(m.graph_safe for m in self.branches)

    def cache_request(self) -> Optional[CacheRequest]:
        return self._cached.cache_request() if self._cached is not None else None

    def step_planner(self):
        return self._planner

    def state_bytes(self) -> int:
        return self._state_bytes

    def forward(self, x: torch.Tensor, step: Any, binding: CacheBinding) -> torch.Tensor:
        outs = []
        for m, (at, n) in zip(self.branches, self._offsets):
            own = CacheBinding(counters=binding.counters)
            if m is self._cached:
                own.group, own.pages, own.writes = binding.group, binding.pages, binding.writes
            if n:
                if binding.state is None:
                    raise ValueError("parallel mixer: a branch needs state, the runner has none")
                own.state = binding.state[:, at:at + n]
            outs.append(_ran(m.forward(x, step, own)))
        return ops.weighted_sum(outs[0], self.scales[0], outs[1], self.scales[1],
                                round_parts=x.dtype == torch.bfloat16)
