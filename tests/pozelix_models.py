"""Small Pozelix configurations and weights for the tests: sizes that differ from layer to layer and
between the configurations (one to six heads, grouped and ungrouped key/value heads, key and value
sizes on either side of each other and off the multiples of 8, latents of two sizes a layer, rotated
parts of two numbers and more, whole, partial and no rotation in the windowed layers, frequencies in
all three ranges of the stretching, windows of one position, of a page, shorter and longer), a loop
in the middle, over the whole model, over one layer, run once and none, layers without a
feed-forward, mixtures with more and with fewer identity experts than others, with none, and with
every expert chosen, either kind of layer first and last), and weights at scales at which every
mechanism matters: norm weights spread around one, corrections that change the choice."""
from __future__ import annotations

from typing import Dict, List

import torch

from gipotar_models import (as_stored, prompts, row_error, write_folder,  # noqa: F401
                            TOLERANCE)


def judge(errors: List[float], dtype: str) -> None:
    """float32: no row beyond two and a half times the tolerance and at most one in fifty beyond
    it.  bfloat16: the median within half of the tolerance and at most one row in twelve beyond it.
    (Norms stand behind the sublayers: where a sublayer's result happens to be small, its rounding
    is scaled up with it.  Where two experts' choice scores lie closer than bfloat16 resolves the
    router's input, the engine may take the other one, and that row is then far from the plain
    logits, whatever the distance; a looped mixture has that chance once a pass.  A token lost from
    a cache, or a pass that reads another's, moves most of the rows behind it.)"""
    tol = TOLERANCE[dtype]
    over = sum(e > tol for e in errors)
    if dtype == "float32":
        assert over <= max(1, len(errors) // 50), f"{over} of {len(errors)} rows beyond {tol}"
        assert max(errors) < 2.5 * tol, f"worst row error {max(errors):.3g}"
    else:
        assert over <= max(2, len(errors) // 12), f"{over} of {len(errors)} rows beyond {tol}"
        median = sorted(errors)[len(errors) // 2]
        assert median < tol / 2 or len(errors) < 20, f"median of the row errors {median:.3g}"


def _dense(ff):
    return {"kind": "dense", "ff": ff}


def _moe(ff, experts, identity, top):
    return {"kind": "moe", "expert": {"ff": ff},
            "router": {"experts": experts, "identity": identity, "top": top}}


def _latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, base, scaling, mlp):
    rot = {"dims": rot_dim, "base": base}
    if scaling is not None:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return {"type": "latent_attention", "mlp": mlp, "mixer": {
        "heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank,
        "kv_rank": kv_rank, "scale": scale, "rot": rot}}


def _attention(heads, kv_heads, dim, vdim, scale, window, rot, mlp):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if window is not None:
        mixer["mask"] = {"size": window}
    if rot is not None:
        mixer["rot"] = {"dims": rot[0], "base": rot[1]}
    return {"type": "attention", "mlp": mlp, "mixer": mixer}


def _model(vocab, width, eps, layers, loop=None):
    cfg = {"architecture": "Pozelix", "vocab": vocab, "width": width, "norm": {"eps": eps},
           "layers": layers}
    if loop is not None:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


# Both kinds of mixer inside and outside of the loop; windows of 20, of a page and of 33; one layer
# of the loop without a feed-forward.
CONFIG_A = _model(97, 48, 1e-5, [
    _attention(4, 2, 16, 24, 0.3, 20, (12, 500.0), _dense(72)),
    _latent(3, 16, 12, 20, 40, 24, 0.2, 300.0, (4.0, 64.0, 8.0, 1.0), _moe(24, 5, 3, 3)),
    _attention(6, 3, 12, 12, 0.35, 16, (12, 10000.0), None),
    _attention(2, 1, 24, 8, 0.25, 33, (8, 100.0), _moe(40, 3, 2, 2)),
    _latent(2, 8, 8, 16, 16, 40, 0.25, 1000.0, (8.0, 128.0, 4.0, 0.5), _dense(56)),
], loop=(1, 4, 3))
# No loop; no stretching; a rotated part of two numbers; one head; no identity experts, every expert
# chosen; no rotation and no window in a windowed layer's place.
CONFIG_B = _model(64, 40, 1e-6, [
    _latent(5, 6, 2, 10, 12, 33, 0.4, 500.0, None, _dense(60)),
    _attention(1, 1, 30, 14, 0.2, 7, (20, 2000.0), _moe(20, 3, 0, 3)),
    _latent(1, 20, 10, 6, 50, 18, 0.25, 50.0, (2.0, 32.0, 4.0, 1.0), None),
    _attention(5, 5, 6, 6, 0.4, None, None, _moe(16, 2, 6, 4)),
])
# Widths, feed-forward widths and a vocabulary that are no multiples of 8 or 4; the loop is the
# whole model; a window of one position.
CONFIG_C = _model(333, 50, 1e-5, [
    _attention(3, 1, 20, 22, 0.28, 25, (10, 900.0), _dense(75)),
    _latent(4, 14, 6, 14, 21, 30, 0.3, 10000.0, (4.0, 128.0, 16.0, 2.0), _moe(30, 4, 1, 1)),
    _attention(2, 2, 14, 14, 0.3, 1, (14, 100.0), None),
], loop=(0, 3, 2))
# Sizes that the matrix-core kernels take, for prompts of hundreds of tokens; the loop is the last
# layer, which runs four times.
CONFIG_D = _model(200, 128, 1e-6, [
    _latent(4, 64, 32, 48, 96, 128, 0.1, 20000.0, (4.0, 256.0, 32.0, 1.0), _moe(64, 6, 3, 3)),
    _attention(4, 1, 64, 64, 0.12, 100, (64, 10000.0), _dense(160)),
    _attention(2, 2, 128, 128, 0.09, 300, (32, 500000.0), _moe(48, 8, 8, 4)),
    _latent(16, 32, 64, 32, 72, 64, 0.12, 500.0, (16.0, 64.0, 4.0, 1.0), _dense(96)),
], loop=(3, 4, 4))
# A loop that runs once (its junction still stands in front of it); the layer it holds is the first.
CONFIG_E = _model(80, 32, 1e-5, [
    _latent(2, 16, 8, 16, 24, 32, 0.25, 100.0, (4.0, 64.0, 4.0, 1.0), _dense(40)),
    _attention(4, 4, 8, 8, 0.4, 9, (4, 1000.0), _moe(8, 2, 2, 1)),
], loop=(0, 1, 1))
CONFIGS = {"a": CONFIG_A, "b": CONFIG_B, "c": CONFIG_C, "d": CONFIG_D, "e": CONFIG_E}


def spec_of(config: dict):
    from rust_llm_inference_server_amd.registry import architecture_of
    arch = architecture_of(config)
    return arch.build_spec(arch.parse_config(config))


STEADY = 4          # the last coordinates of the stream: the routers' choices hang on them


def _steady_routers(config: dict, w: Dict[str, torch.Tensor], g: torch.Generator) -> None:
    """Choices of experts that bfloat16 does not decide: the last coordinates of the stream carry a
    token's pattern of signs unchanged through all layers and passes (the norms behind the
    sublayers let nothing through to them, the loop's map takes half from the stream and half from
    the embedding output), and the routers read them above all; of 200 drawn the router stays whose
    closest choice over all patterns, at several sizes of the other coordinates, is the clearest."""
    n, W = STEADY, config["width"]
    w["embed"][:, -n:] = torch.sign(torch.randn((config["vocab"], n), generator=g))
    for name in w:
        if name.endswith((".norm1b", ".norm2b")):
            w[name][-n:] = 0.0
        elif name.endswith(".norm2"):
            w[name][-n:] = 1.0
    if "loop.in" in w:
        w["loop.in"][-n:] = 0.0
        for c in range(n):
            w["loop.in"][W - 1 - c, W - 1 - c] = w["loop.in"][W - 1 - c, 2 * W - 1 - c] = 0.5
    signs = torch.tensor([[1.0 if i >> b & 1 else -1.0 for b in range(n)] for i in range(2 ** n)])
    for name in [k for k in w if k.endswith(".router")]:
        mlp = config["layers"][int(name.split(".")[0][1:])]["mlp"]
        top, corr = mlp["router"]["top"], w[name[:-len("router")] + "correction"]
        w[name] *= 0.05
        best = -1.0
        for _ in range(200):
            draw = torch.randn((w[name].shape[0], n), generator=g) * 3.0
            margin = 1.0
            if top < draw.shape[0]:
                for size in (0.35, 0.5, 0.7, 1.0):
                    s = torch.softmax(size * signs @ draw.T, -1) + corr
                    ranked = s.sort(-1, descending=True).values
                    margin = min(margin, float((ranked[:, top - 1] - ranked[:, top]).min()))
            if margin > best:
                best, w[name][:, -n:] = margin, draw


def make_weights(config: dict, seed: int) -> Dict[str, torch.Tensor]:
    """float32 tensors by checkpoint name, values chosen by what the tensor is."""
    g = torch.Generator().manual_seed(seed)
    normal = lambda shape, std=1.0: torch.randn(shape, generator=g) * std
    out = {}
    for t in spec_of(config).tensor_specs():
        name, shape = t.name, tuple(t.shape)
        last = name.split(".")[-1]
        if name == "embed":
            w = normal(shape, 0.7)
        elif len(shape) == 1 and last.startswith("norm"):
            w = 1.0 + normal(shape, 0.3)
        elif last == "correction":
            w = normal(shape, 0.15)
        elif last == "router":
            w = normal(shape, 2.0 * shape[-1] ** -0.5)
        elif len(shape) == 2:
            w = normal(shape, shape[-1] ** -0.5)
        else:
            raise AssertionError(f"no rule for {name}")
        out[name] = w.contiguous()
    _steady_routers(config, out, g)
    return out


def plain_logits(plain, cfg: dict, stored: Dict[str, torch.Tensor], tokens: List[int]) -> torch.Tensor:
    return plain.forward(cfg, stored, tokens)
