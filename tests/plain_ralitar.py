"""The Ralitar decoder in plain, slow torch (float64, one sequence at a time, no cache): what the
engine is held against.  One function per mechanism; nothing here is shared with the package.
``config`` is the dict that config.json holds, ``w`` maps tensor names to tensors.

Notation.  ``x`` is the residual stream ``(T, W)``; a linear weight is ``(out, in)``;
``unit(x) = x / sqrt(mean(x^2) + eps)``.

    input:   x = E[token] + B[row of (previous token, token)]
    layer i: x += unit(mixer(x)) * n1;  x += unit(ff(x)) * n2;
             x += unit(P (gelu(G x) * e_i[token])) * n3
    output:  head (unit(x) * n)

Mixers: a gated linear recurrence per channel (``rglru``), the gated delta rule with a decay per
key channel (``channel_delta``), softmax attention inside chunks whose values are its keys
(``attention``).
"""
from __future__ import annotations

import math
from typing import Any, Dict, List, Optional, Tuple

import torch

F64 = torch.float64
UNIT_EPS = 1e-6


def _w(w: Dict[str, torch.Tensor], name: str) -> torch.Tensor:
    return w[name].to(F64)


# ------------------------------------------------------------------------------- pieces
def unit(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def softplus(z: torch.Tensor) -> torch.Tensor:
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def bigram_rows(tokens: List[int], bigram: Dict[str, Any]) -> List[int]:
    """Which row of the pair table every token takes; a sequence's first takes the last row."""
    buckets = int(bigram["buckets"])
    rows = [buckets]
    for a, b in zip(tokens, tokens[1:]):
        rows.append((a * int(bigram["mul_prev"]) + b * int(bigram["mul_cur"])) % buckets)
    return rows[:len(tokens)]


def embed(config: Dict[str, Any], w: Dict[str, torch.Tensor], tokens: List[int]) -> torch.Tensor:
    x = _w(w, "embed")[torch.tensor(tokens)]
    bigram = (config.get("embedding") or {}).get("bigram")
    if bigram:
        x = x + _w(w, "bigram")[torch.tensor(bigram_rows(tokens, bigram))]
    return x


def short_conv(u: torch.Tensor, taps: torch.Tensor, bias: Optional[torch.Tensor] = None
               ) -> torch.Tensor:
    """y[t, c] = bias[c] + sum_j taps[c, j] u[t - (K - 1) + j, c], zeros before the sequence."""
    T, C = u.shape
    K = taps.shape[1]
    padded = torch.cat([torch.zeros((K - 1, C), dtype=u.dtype), u], dim=0)
    y = torch.zeros_like(u) if bias is None else bias.reshape(1, C).repeat(T, 1)
    for j in range(K):
        y = y + padded[j:j + T] * taps[:, j]
    return y


def frequencies(rot: Dict[str, Any]) -> torch.Tensor:
    """One frequency per pair of dims; slow ones are stretched by ``factor``, fast ones kept."""
    dims, base = int(rot["dims"]), float(rot["base"])
    out = []
    sc = rot.get("scaling")
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if sc:
            factor, low, high, original = (float(sc[k]) for k in ("factor", "low", "high", "original"))
            wave = 2.0 * math.pi / f
            if wave > original / low:
                f = f / factor
            elif wave >= original / high:
                s = (original / wave - low) / (high - low)
                f = (1.0 - s) * f / factor + s * f
        out.append(f)
    return torch.tensor(out, dtype=F64)


def rotate_pairs(x: torch.Tensor, positions: torch.Tensor, rot: Dict[str, Any]) -> torch.Tensor:
    """x ``(T, heads, d)``: dims 2i and 2i + 1 turn together, for the first ``rot.dims`` dims."""
    dims = int(rot["dims"])
    ang = positions.to(F64).reshape(-1, 1, 1) * frequencies(rot).reshape(1, 1, -1)
    c, s = torch.cos(ang), torch.sin(ang)
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    y = x.clone()
    y[..., 0:dims:2] = u * c - v * s
    y[..., 1:dims:2] = v * c + u * s
    return y


# ------------------------------------------------------------------------------- mixers
def rglru_scan(log_a: torch.Tensor, drive: torch.Tensor) -> torch.Tensor:
    """S_t = a_t S_(t-1) + sqrt(1 - a_t^2) drive_t from zero; rows of all S_t."""
    a = torch.exp(log_a)
    S = torch.zeros_like(drive[0])
    out = []
    for t in range(drive.shape[0]):
        S = a[t] * S + torch.sqrt(-torch.expm1(2.0 * log_a[t])) * drive[t]
        out.append(S)
    return torch.stack(out)


def rglru_mixer(w: Dict[str, torch.Tensor], p: str, m: Dict[str, Any], h: torch.Tensor
                ) -> torch.Tensor:
    T = h.shape[0]
    width, blocks = int(m["width"]), int(m["blocks"])
    y = gelu_tanh(h @ _w(w, p + ".y").T + _w(w, p + ".y.b"))
    u = short_conv(h @ _w(w, p + ".x").T + _w(w, p + ".x.b"), _w(w, p + ".conv"),
                   _w(w, p + ".conv.b"))
    parts = u.reshape(T, blocks, width // blocks)
    gates = {}
    for n in ("ra", "ri"):
        mats, bias = _w(w, f"{p}.{n}"), _w(w, f"{p}.{n}.b")
        gates[n] = torch.stack([torch.sigmoid(parts[:, b] @ mats[b].T + bias[b])
                                for b in range(blocks)], dim=1).reshape(T, width)
    log_a = -8.0 * gates["ra"] * softplus(_w(w, p + ".lam"))
    S = rglru_scan(log_a, gates["ri"] * u)
    return (S * y) @ _w(w, p + ".o").T


def channel_delta_scan(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, g: torch.Tensor,
                       beta: torch.Tensor) -> torch.Tensor:
    """One head: q, k, g ``(T, d)``, v ``(T, dv)``, beta ``(T)``.  Row i of S belongs to key
    channel i and decays by g[t, i]; then the token corrects what its key reads and reads."""
    S = torch.zeros((q.shape[1], v.shape[1]), dtype=q.dtype)
    out = torch.zeros_like(v)
    for t in range(q.shape[0]):
        S = g[t].reshape(-1, 1) * S
        u = beta[t] * (v[t] - S.T @ k[t])
        S = S + torch.outer(k[t], u)
        out[t] = S.T @ q[t]
    return out


def channel_delta_mixer(w: Dict[str, torch.Tensor], p: str, m: Dict[str, Any], h: torch.Tensor,
                        eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    q, k, v = (silu(short_conv(h @ _w(w, f"{p}.{n}").T, _w(w, f"{p}.{n}.conv"))) for n in "qkv")

    def unit_heads(z):
        z = z.reshape(T, G, d)
        return z / torch.sqrt((z * z).sum(-1, keepdim=True) + UNIT_EPS)

    q, k, v = unit_heads(q) * d ** -0.5, unit_heads(k), v.reshape(T, H, dv)
    beta = torch.sigmoid(h @ _w(w, p + ".b").T)
    z = (h @ _w(w, p + ".a1").T) @ _w(w, p + ".a2").T + _w(w, p + ".dt_bias")
    g = torch.exp(-torch.exp(_w(w, p + ".A_log")).reshape(1, H, 1) * softplus(z).reshape(T, H, d))
    gate = torch.sigmoid((h @ _w(w, p + ".g1").T) @ _w(w, p + ".g2").T).reshape(T, H, dv)
    o = torch.stack([channel_delta_scan(q[:, j // (H // G)], k[:, j // (H // G)], v[:, j], g[:, j],
                                        beta[:, j]) for j in range(H)], dim=1)
    o = unit(o, eps) * _w(w, p + ".norm") * gate
    return o.reshape(T, H * dv) @ _w(w, p + ".o").T


def chunk_mask(positions: torch.Tensor, size: Optional[int]) -> torch.Tensor:
    i, j = positions.reshape(-1, 1), positions.reshape(1, -1)
    seen = j <= i
    return seen if size is None else seen & (i // size == j // size)


def attention_scores(w: Dict[str, torch.Tensor], p: str, m: Dict[str, Any], h: torch.Tensor,
                     eps: float) -> Tuple[torch.Tensor, torch.Tensor]:
    """Softmax weights ``(H, T, T)`` and values ``(T, G, d)``."""
    T = h.shape[0]
    H, G, d = int(m["heads"]), int(m["kv_heads"]), int(m["dim"])
    pos = torch.arange(T)
    q = h @ _w(w, p + ".q").T + _w(w, p + ".q.b")
    k = h @ _w(w, p + ".k").T + _w(w, p + ".k.b")
    v = k.reshape(T, G, d)
    q = (unit(q, eps) * _w(w, p + ".q.norm")).reshape(T, H, d)
    k = (unit(k, eps) * _w(w, p + ".k.norm")).reshape(T, G, d)
    if m.get("rot"):
        q, k = rotate_pairs(q, pos, m["rot"]), rotate_pairs(k, pos, m["rot"])
    seen = chunk_mask(pos, int(m["mask"]["size"]) if m.get("mask") else None)
    probs = []
    for j in range(H):
        s = (q[:, j] @ k[:, j // (H // G)].T) * float(m["scale"])
        if m.get("softcap"):
            s = float(m["softcap"]) * torch.tanh(s / float(m["softcap"]))
        probs.append(torch.softmax(s.masked_fill(~seen, -math.inf), dim=-1))
    return torch.stack(probs), v


def attention_mixer(w: Dict[str, torch.Tensor], p: str, m: Dict[str, Any], h: torch.Tensor,
                    eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, G, d = int(m["heads"]), int(m["kv_heads"]), int(m["dim"])
    probs, v = attention_scores(w, p, m, h, eps)
    out = torch.stack([probs[j] @ v[:, j // (H // G)] for j in range(H)], dim=1).reshape(T, H * d)
    out = out * torch.sigmoid(h @ _w(w, p + ".g").T)
    return out @ _w(w, p + ".o").T


def mixer(w: Dict[str, torch.Tensor], p: str, layer: Dict[str, Any], h: torch.Tensor, eps: float
          ) -> torch.Tensor:
    kind, m = layer["type"], layer["mixer"]
    if kind == "rglru":
        return rglru_mixer(w, p, m, h)
    if kind == "channel_delta":
        return channel_delta_mixer(w, p, m, h, eps)
    if kind == "attention":
        return attention_mixer(w, p, m, h, eps)
    raise ValueError(kind)


# --------------------------------------------------------------- feed-forward, token input
def dense_ff(w: Dict[str, torch.Tensor], p: str, h: torch.Tensor) -> torch.Tensor:
    return (gelu_tanh(h @ _w(w, p + ".gate").T) * (h @ _w(w, p + ".up").T)) @ _w(w, p + ".down").T


def token_side(w: Dict[str, torch.Tensor], p: str, index: int, dim: int, x: torch.Tensor,
               tokens: List[int], eps: float) -> torch.Tensor:
    e = _w(w, "side.embed")[torch.tensor(tokens)][:, index * dim:(index + 1) * dim]
    y = (gelu_tanh(x @ _w(w, p + ".gate").T) * e) @ _w(w, p + ".proj").T
    return unit(y, eps) * _w(w, p + ".norm")


# ------------------------------------------------------------------------------ the model
def forward_layers(config: Dict[str, Any], w: Dict[str, torch.Tensor], tokens: List[int]
                   ) -> Tuple[torch.Tensor, torch.Tensor]:
    """Logits ``(T, vocab)`` and the stream behind every layer ``(layers, T, width)``."""
    eps = float(config["norm"]["eps"])
    side = config.get("token_side")
    x = embed(config, w, tokens)
    after = []
    for i, layer in enumerate(config["layers"]):
        p = f"l{i}"
        x = x + unit(mixer(w, p + ".mix", layer, x, eps), eps) * _w(w, p + ".norm1")
        if layer.get("mlp") is not None:
            x = x + unit(dense_ff(w, p + ".mlp", x), eps) * _w(w, p + ".norm2")
        if side:
            x = x + token_side(w, p + ".side", i, int(side["dim"]), x, tokens, eps)
        after.append(x)
    return (unit(x, eps) * _w(w, "final.norm")) @ _w(w, "head").T, torch.stack(after)


def forward(config: Dict[str, Any], w: Dict[str, torch.Tensor], tokens: List[int]) -> torch.Tensor:
    return forward_layers(config, w, tokens)[0]
