"""The Pozelix decoder written out plainly in torch (float64 by default), one function per
mechanism, for tests to hold the engine against.  It shares nothing with the package: it reads
a config.json dictionary and a dictionary of tensors by their checkpoint names, and runs whole
sequences without a cache.

Notation: ``x`` is a sequence of rows ``(n, width)``; positions count from 0.
"""
from __future__ import annotations

import math
from typing import Any, Dict, List, Optional

import torch


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """Every row divided by the root of (its mean square plus eps)."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def plain_frequencies(dims: int, base: float, dtype) -> torch.Tensor:
    i = torch.arange(dims // 2, dtype=dtype)
    return base ** (-2.0 * i / dims)


def yarn_pair_index(turns: float, dims: int, base: float, original: float) -> float:
    """The (fractional) pair whose wave makes ``turns`` turns over ``original`` positions."""
    return dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))


def yarn_frequencies(dims: int, base: float, s: Dict[str, Any], dtype) -> torch.Tensor:
    """Fast pairs keep their frequency, slow ones get it divided by the factor, a linear ramp
    over the pair index lies between."""
    f = plain_frequencies(dims, base, dtype)
    lo = max(math.floor(yarn_pair_index(s["fast"], dims, base, s["original"])), 0)
    hi = min(math.ceil(yarn_pair_index(s["slow"], dims, base, s["original"])), dims - 1)
    out = []
    for i in range(dims // 2):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(float(f[i]) / s["factor"] * ramp + float(f[i]) * (1.0 - ramp))
    return torch.tensor(out, dtype=dtype)


def angles(n: int, rot: Dict[str, Any], dtype):
    """cos and sin ``(n, dims / 2)``, stretched and scaled where ``rot`` says so."""
    s = rot.get("scaling")
    if s:
        f = yarn_frequencies(rot["dims"], rot["base"], s, dtype)
        m = 0.1 * math.log(s["factor"]) + 1.0
    else:
        f, m = plain_frequencies(rot["dims"], rot["base"], dtype), 1.0
    a = torch.arange(n, dtype=dtype).reshape(n, 1) * f.reshape(1, -1)
    return torch.cos(a) * m, torch.sin(a) * m


def rotate_neighbours(x: torch.Tensor, rot: Dict[str, Any]) -> torch.Tensor:
    """``x (n, heads, size)``: numbers 2i and 2i + 1 of the first ``dims`` form a pair."""
    c, s = (t.unsqueeze(1) for t in angles(x.shape[0], rot, x.dtype))
    out = x.clone()
    d = rot["dims"]
    u, v = x[..., 0:d:2], x[..., 1:d:2]
    out[..., 0:d:2] = u * c - v * s
    out[..., 1:d:2] = v * c + u * s
    return out


def rotate_halves(x: torch.Tensor, rot: Dict[str, Any]) -> torch.Tensor:
    """``x (n, heads, size)``: numbers i and i + dims / 2 form a pair."""
    c, s = (t.unsqueeze(1) for t in angles(x.shape[0], rot, x.dtype))
    d = rot["dims"]
    u, v = x[..., :d // 2], x[..., d // 2:d]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., d:]], dim=-1)


def visible(n: int, size: Optional[int]) -> torch.Tensor:
    """``(n, n)`` booleans: may query i (rows) see key j (columns)?  Causal, and with a window
    of ``size`` fewer than ``size`` positions back."""
    i, j = torch.arange(n).reshape(n, 1), torch.arange(n).reshape(1, n)
    ok = j <= i
    return ok if size is None else ok & (i - j < size)


def attend(scores: torch.Tensor, ok: torch.Tensor, v: torch.Tensor) -> torch.Tensor:
    """``scores (heads, n, n)``, ``v (n, heads, dv)`` -> ``(n, heads, dv)``."""
    p = torch.softmax(scores.masked_fill(~ok, float("-inf")), dim=-1)
    return torch.stack([p[h] @ v[:, h] for h in range(v.shape[1])], dim=1)


def latent_attention(h: torch.Tensor, m: Dict[str, Any], w: Dict[str, torch.Tensor], pre: str,
                     eps: float) -> torch.Tensor:
    """Queries through a latent of their own; keys and values from a latent per position, and a
    rotated key part that the heads share."""
    n, H, d, r, R = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["kv_rank"]
    cq = rms(h @ w[pre + "dq"].T, eps) * w[pre + "dq.norm"]
    q = (cq @ w[pre + "uq"].T).reshape(n, H, d + r)
    down = h @ w[pre + "dkv"].T
    c = rms(down[:, :R], eps) * w[pre + "dkv.norm"]
    q_rot = rotate_neighbours(q[..., d:], m["rot"])
    k_rot = rotate_neighbours(down[:, R:].reshape(n, 1, r), m["rot"])[:, 0]
    k = (c @ w[pre + "uk"].T).reshape(n, H, d)
    v = (c @ w[pre + "uv"].T).reshape(n, H, m["vdim"])
    scores = torch.stack([q[:, i, :d] @ k[:, i].T + q_rot[:, i] @ k_rot.T for i in range(H)])
    out = attend(scores * m["scale"], visible(n, None), v)
    return out.reshape(n, -1) @ w[pre + "o"].T


def attention(h: torch.Tensor, m: Dict[str, Any], w: Dict[str, torch.Tensor], pre: str,
              eps: float) -> torch.Tensor:
    """Grouped heads under a sliding window; queries and keys rotated, then divided by their root
    mean square; a gate per head on the result."""
    n, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q = (h @ w[pre + "q"].T).reshape(n, H, m["dim"])
    k = (h @ w[pre + "k"].T).reshape(n, G, m["dim"])
    if m.get("rot"):
        q, k = rotate_halves(q, m["rot"]), rotate_halves(k, m["rot"])
    q, k = rms(q, eps), rms(k, eps)
    v = (h @ w[pre + "v"].T).reshape(n, G, m["vdim"])
    of = [i // (H // G) for i in range(H)]
    scores = torch.stack([q[:, i] @ k[:, of[i]].T for i in range(H)]) * m["scale"]
    out = attend(scores, visible(n, (m.get("mask") or {}).get("size")), v[:, of])
    out = out * torch.sigmoid(h @ w[pre + "g"].T).unsqueeze(-1)
    return out.reshape(n, -1) @ w[pre + "o"].T


MIXERS = {"latent_attention": latent_attention, "attention": attention}


def gated_unit(h: torch.Tensor, w: Dict[str, torch.Tensor], pre: str) -> torch.Tensor:
    return (silu(h @ w[pre + "gate"].T) * (h @ w[pre + "up"].T)) @ w[pre + "down"].T


def choose(z: torch.Tensor, correction: torch.Tensor, top: int):
    """Logits ``(n, E)`` -> the chosen experts ``(n, top)`` and their weights: the softmax scores
    over all experts; the correction moves the choice alone."""
    s = torch.softmax(z, dim=-1)
    chosen = torch.topk(s + correction, top, dim=-1).indices
    return chosen, torch.gather(s, 1, chosen)


def mixture(h: torch.Tensor, mlp: Dict[str, Any], w: Dict[str, torch.Tensor], pre: str
            ) -> torch.Tensor:
    """The weighted sum of the chosen experts' outputs; experts from ``experts`` on hand back
    their input."""
    router = mlp["router"]
    chosen, weights = choose(h @ w[pre + "router"].T, w[pre + "correction"], router["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for r in range(router["top"]):
            e = int(chosen[t, r])
            y = h[t] if e >= router["experts"] else gated_unit(h[t], w, f"{pre}e{e}.")
            out[t] = out[t] + weights[t, r] * y
    return out


def feed_forward(h, mlp, w, pre):
    return gated_unit(h, w, pre) if mlp["kind"] == "dense" else mixture(h, mlp, w, pre)


def rejoin(x: torch.Tensor, x0: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """What a pass of the loop starts from: one map of the stream and the embedding output."""
    return torch.cat([x, x0], dim=-1) @ w.T


def run_order(config: Dict[str, Any]) -> List[tuple]:
    """(layer, does a pass of the loop begin in front of it?) of every layer run."""
    n = len(config["layers"])
    loop = config.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    return ([(i, False) for i in range(a)] + [(i, i == a) for i in range(a, b)] * loop["times"]
            + [(i, False) for i in range(b, n)])


def forward(config: Dict[str, Any], weights: Dict[str, torch.Tensor], tokens: List[int],
            dtype=torch.float64, layer_outputs: Optional[list] = None) -> torch.Tensor:
    """Logits ``(n, vocab)`` of a whole sequence.  ``layer_outputs``: a list that receives the
    stream behind every layer run."""
    w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in weights.items()}
    eps = config["norm"]["eps"]
    norm = lambda v, name: rms(v, eps) * w[name]
    x0 = w["embed"][torch.tensor(tokens)]
    x = x0
    for i, enters in run_order(config):
        layer, pre = config["layers"][i], f"l{i}."
        if enters:
            x = rejoin(x, x0, w["loop.in"])
        y = MIXERS[layer["type"]](norm(x, pre + "norm1"), layer["mixer"], w, pre + "mix.", eps)
        x = x + norm(y, pre + "norm1b")
        if layer.get("mlp"):
            y = feed_forward(norm(x, pre + "norm2"), layer["mlp"], w, pre + "mlp.")
            x = x + norm(y, pre + "norm2b")
        if layer_outputs is not None:
            layer_outputs.append(x)
    return norm(x, "final.norm") @ w["head"].T
