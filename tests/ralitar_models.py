"""Small Ralitar configurations and weights for the tests: sizes that differ from layer to layer
and between the configurations (one to six heads, grouped and ungrouped key/value heads, key and
value sizes on either side of each other and off the multiples of 8, whole, partial and no
rotation with and without stretched frequencies, chunks of a page, shorter, longer and none, with
and without a cap, one to five taps, one to four blocks of gates, ranks of the two low-rank pairs
that differ, layers without a feed-forward, a token input and a pair table or none, multipliers
beyond 32 bits of product, every kind of layer first and last), and weights at scales at which
every mechanism matters: norm weights spread around one, biases, slow and fast decays."""
from __future__ import annotations

from typing import Dict, List

import torch

from gipotar_models import (as_stored, prompts, row_error, write_folder,  # noqa: F401
                            TOLERANCE)


def judge(errors: List[float], dtype: str) -> None:
    """float32: no row beyond two and a half times the tolerance and at most one in fifty beyond
    it.  bfloat16: the median within half of the tolerance, at most one row in twelve beyond it and
    none beyond 0.7.  (Norms stand behind the sublayers here, and behind the delta rule's heads:
    where a read-out or a sublayer's result happens to be small, its rounding is scaled up with
    it.  The engine's own rounding on the CPU double, whose every sum is exact to float32, puts one
    row in fifty at two to three times the tolerance; a token lost from the cache or a state
    moves most of the rows behind it.)"""
    tol = TOLERANCE[dtype]
    over = sum(e > tol for e in errors)
    if dtype == "float32":
        assert over <= max(1, len(errors) // 50), f"{over} of {len(errors)} rows beyond {tol}"
        assert max(errors) < 2.5 * tol, f"worst row error {max(errors):.3g}"
    else:
        assert over <= max(2, len(errors) // 12), f"{over} of {len(errors)} rows beyond {tol}"
        assert max(errors) < 0.7, f"worst row error {max(errors):.3g}"
        median = sorted(errors)[len(errors) // 2]
        assert median < tol / 2 or len(errors) < 20, f"median of the row errors {median:.3g}"


def _dense(ff):
    return None if ff is None else {"kind": "dense", "ff": ff}


def _delta(heads, kv_heads, dim, vdim, conv, ranks, ff):
    return {"type": "channel_delta", "mlp": _dense(ff), "mixer": {
        "heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv,
        "decay_rank": ranks[0], "gate_rank": ranks[1]}}


def _rglru(width, blocks, conv, ff):
    return {"type": "rglru", "mlp": _dense(ff),
            "mixer": {"width": width, "blocks": blocks, "conv": conv}}


def _attention(heads, kv_heads, dim, scale, chunk, rot, softcap, ff):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale}
    if chunk is not None:
        mixer["mask"] = {"size": chunk}
    if rot is not None:
        mixer["rot"] = {"dims": rot[0], "base": rot[1]}
        if len(rot) > 2:
            mixer["rot"]["scaling"] = dict(zip(("factor", "low", "high", "original"), rot[2:]))
    if softcap:
        mixer["softcap"] = softcap
    return {"type": "attention", "mlp": _dense(ff), "mixer": mixer}


def _model(vocab, width, eps, layers, bigram=None, side=None):
    cfg = {"architecture": "Ralitar", "vocab": vocab, "width": width, "norm": {"eps": eps},
           "layers": layers}
    if bigram is not None:
        cfg["embedding"] = {"bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))}
    if side is not None:
        cfg["token_side"] = {"dim": side}
    return cfg


# All kinds; chunks of 20, of a page and of 33; partial rotation with frequencies in all three
# ranges of the stretching, whole rotation, none; grouped heads in both kinds that have them.
CONFIG_A = _model(97, 48, 1e-5, [
    _delta(4, 2, 16, 24, 4, (6, 10), 72),
    _attention(4, 2, 16, 0.3, 20, (12, 500.0, 4.0, 1.0, 4.0, 64.0), 6.0, 56),
    _rglru(60, 3, 3, None),
    _attention(6, 3, 12, 0.35, 16, (12, 10000.0), 9.0, 40),
    _delta(3, 3, 20, 12, 2, (9, 5), None),
    _rglru(40, 1, 5, 64),
    _attention(2, 1, 24, 0.25, 33, None, 5.0, 48),
], bigram=(53, 37, 11), side=8)
# No pair table, no token input; attention over all earlier keys without a cap; one tap; more
# than 64 key channels; one head.
CONFIG_B = _model(64, 40, 1e-6, [
    _attention(5, 5, 6, 0.4, None, (4, 300.0), 0.0, 60),
    _rglru(33, 3, 1, 24),
    _delta(1, 1, 70, 33, 1, (3, 12), None),
    _attention(1, 1, 30, 0.2, 7, (20, 2000.0, 8.0, 1.0, 2.0, 32.0), 0.0, None),
    _delta(6, 2, 8, 10, 3, (8, 8), 36),
])
# Widths, feed-forward widths and a vocabulary that are no multiples of 8 or 4; products of the
# multipliers beyond 32 bits; more buckets than tokens; a chunk of one position.
CONFIG_C = _model(333, 50, 1e-5, [
    _rglru(52, 4, 4, 75),
    _delta(2, 1, 12, 20, 3, (7, 4), 58),
    _attention(3, 1, 20, 0.28, 25, (10, 900.0, 4.0, 1.0, 4.0, 128.0), 7.0, 30),
    _attention(2, 2, 14, 0.3, 1, (14, 100.0), 4.0, None),
], bigram=(1009, 2147483629, 1999999973), side=5)
# Head sizes that the matrix-core kernels take (64 and 128), for prompts of hundreds of tokens;
# chunks of 100 and of 500; whole and partial rotation.
CONFIG_D = _model(200, 128, 1e-6, [
    _rglru(256, 2, 4, 192),
    _attention(4, 1, 64, 0.125, 100, (64, 10000.0, 8.0, 1.0, 4.0, 256.0), 20.0, 160),
    _delta(4, 2, 64, 64, 4, (16, 32), 192),
    _attention(2, 2, 128, 0.09, 500, (32, 500000.0), 30.0, 128),
    _delta(2, 2, 128, 96, 3, (24, 8), None),
], bigram=(300, 17, 5), side=32)
# Recurrent layers only: nothing is paged.  Layouts in steps of four channels.
CONFIG_E = _model(80, 32, 1e-5, [
    _rglru(48, 2, 2, 40),
    _delta(4, 4, 8, 16, 4, (5, 6), None),
    _rglru(64, 4, 4, None),
    _delta(2, 1, 32, 36, 5, (4, 9), 30),
], bigram=(41, 13, 29))
CONFIGS = {"a": CONFIG_A, "b": CONFIG_B, "c": CONFIG_C, "d": CONFIG_D, "e": CONFIG_E}


def spec_of(config: dict):
    from rust_llm_inference_server_amd.registry import architecture_of
    arch = architecture_of(config)
    return arch.build_spec(arch.parse_config(config))


def make_weights(config: dict, seed: int) -> Dict[str, torch.Tensor]:
    """float32 tensors by checkpoint name, values chosen by what the tensor is."""
    g = torch.Generator().manual_seed(seed)
    normal = lambda shape, std=1.0: torch.randn(shape, generator=g) * std
    uniform = lambda shape, lo, hi: lo + (hi - lo) * torch.rand(shape, generator=g)
    out = {}
    for t in spec_of(config).tensor_specs():
        name, shape = t.name, tuple(t.shape)
        last = name.split(".")[-1]
        if name in ("embed", "bigram"):
            w = normal(shape, 0.7)
        elif name == "side.embed":
            w = normal(shape, 1.0)
        elif last in ("norm1", "norm2", "norm") or name == "final.norm":
            w = 1.0 + normal(shape, 0.3)
        elif name.endswith((".ra.b", ".ri.b")):
            w = normal(shape, 1.0)
        elif last == "b" and len(shape) == 1:
            w = normal(shape, 0.4)
        elif last == "conv":
            w = normal(shape, 0.6)
        elif last == "A_log":
            w = uniform(shape, -3.0, 0.5)
        elif last == "dt_bias":
            w = uniform(shape, -3.0, 1.0)
        elif last == "lam":
            w = uniform(shape, -6.0, 0.5)
        elif len(shape) >= 2:
            w = normal(shape, shape[-1] ** -0.5)
        else:
            raise AssertionError(f"no rule for {name}")
        out[name] = w.contiguous()
    return out


def plain_logits(plain, cfg: dict, stored: Dict[str, torch.Tensor], tokens: List[int]) -> torch.Tensor:
    return plain.forward(cfg, stored, tokens)
