"""Each kernel that the Pozelix design added or extended, alone, against the plain formulas of
``plain_pozelix.py`` (float64), at sizes the models of the other tests do not have: queries and keys
normed behind their rotation on their way to the cache, and the decode attention that writes it; a
sublayer's norm and the next one's in one pass over the residual; the queries' latent normed beside
the other, the rotation of neighbouring pairs in a latent's rotated part; softmax routing over
experts and identity experts; routed units some of which hand back their input."""
import math

import pytest
import torch

import plain_pozelix as plain

pytestmark = pytest.mark.gpu
DEV = "cuda"
TOL = {torch.float32: 2e-5, torch.bfloat16: 2e-2}


def rel(got, want):
    want = want.double().cpu()
    return float((got.double().cpu() - want).norm() / want.norm().clamp_min(1e-12))


def rnd(*shape, seed=0, std=1.0, dtype=torch.float32):
    g = torch.Generator().manual_seed(seed + 1000 * len(shape) + sum(shape))
    return (torch.randn(shape, generator=g) * std).to(dtype)


def _tables(n, rot):
    cos, sin = plain.angles(n, rot, torch.float64)
    return cos, sin, cos.float().to(DEV).contiguous(), sin.float().to(DEV).contiguous()


def _turn(x, pos, cos, sin, dims, interleaved):
    """``x (T, heads, size)`` at positions ``pos``."""
    c, s = cos[pos].unsqueeze(1), sin[pos].unsqueeze(1)
    out = x.clone()
    if interleaved:
        u, v = x[..., 0:dims:2], x[..., 1:dims:2]
        out[..., 0:dims:2], out[..., 1:dims:2] = u * c - v * s, v * c + u * s
    else:
        u, v = x[..., :dims // 2], x[..., dims // 2:dims]
        out[..., :dims // 2], out[..., dims // 2:dims] = u * c - v * s, v * c + u * s
    return out


# --------------------------------------------------------- norms behind the rotation
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("nh, nkv, D, real, rot", [
    (4, 2, 16, 16, 16), (3, 1, 48, 36, 12), (5, 5, 16, 6, 0), (6, 2, 64, 64, 64),
    (7, 1, 128, 128, 32), (2, 2, 256, 256, 256), (1, 1, 80, 80, 48), (3, 3, 32, 30, 2)])
@pytest.mark.parametrize("interleaved", [False, True])
@pytest.mark.parametrize("T", [1, 21, 900])
def test_heads_normed_behind_their_rotation(dtype, nh, nkv, D, real, rot, interleaved, T):
    """Rows with eight more columns behind the values; heads padded with zeros; steps whose lanes
    take one head and four.  Written to pages (tokens in slots of any order, one of them without a
    slot), with the keys left in their rows, and with the queries alone."""
    from rust_llm_inference_server_amd import ops
    eps, ps, cols = 1e-3, 16, (nh + 2 * nkv) * D
    rows = rnd(T, cols + 8, seed=1, dtype=dtype)
    heads = rows[:, :cols].reshape(T, nh + 2 * nkv, D)
    heads[..., real:] = 0
    heads[0, 0] *= 1e-3                       # a head whose size eps decides
    pos = torch.randint(0, 700, (T,), generator=torch.Generator().manual_seed(2))
    x = heads.double()[:, :nh + nkv]
    args = (None, None)
    if rot:
        cos, sin, dcos, dsin = _tables(700, {"dims": rot, "base": 300.0})
        x, args = _turn(x, pos, cos, sin, rot, interleaved), (dcos, dsin)
    want = x / torch.sqrt((x[..., :real] ** 2).mean(-1, keepdim=True) + eps)
    dpos = pos.to(torch.int32).to(DEV)
    pages = -(-T // ps) + 2
    slots = torch.randperm(pages * ps, generator=torch.Generator().manual_seed(3))[:T].to(torch.int32)
    if T > 1:
        slots[T // 2] = -1
    untouched = heads[:, nh + nkv:].double()
    for mode in ("pages", "rows", "queries"):
        qkv = rows.to(DEV)
        kp = torch.full((pages, nkv, ps, D), 9.0, dtype=dtype, device=DEV)
        vp = torch.full((pages, nkv, D, ps), 9.0, dtype=dtype, device=DEV)
        ops.norm_rope_kv_write(qkv[:, :cols], nh, nkv, D, real, eps, *args, dpos, slots.to(DEV), kp, vp,
                               ps, write_kv=mode == "pages", interleaved=interleaved,
                               keys_in_place=mode == "rows")
        got = qkv[:, :cols].reshape(T, nh + 2 * nkv, D)
        assert rel(got[:, :nh], want[:, :nh]) < TOL[dtype]
        assert torch.equal(got[:, nh + nkv:].double().cpu(), untouched)
        assert torch.equal(qkv[:, cols:].cpu(), rows[:, cols:])
        if mode == "rows":
            assert rel(got[:, nh:nh + nkv], want[:, nh:]) < TOL[dtype]
        else:
            assert torch.equal(got[:, nh:nh + nkv].cpu(), heads[:, nh:nh + nkv])
        if mode != "pages":
            assert bool((kp == 9.0).all()) and bool((vp == 9.0).all())
            continue
        written = 0
        for t in range(T):
            if slots[t] < 0:
                continue
            pg, off = int(slots[t]) // ps, int(slots[t]) % ps
            written += 1
            if t % 37 == 0 or t < 3:
                assert rel(kp[pg, :, off], want[t, nh:]) < TOL[dtype] * 2
                assert torch.equal(vp[pg, :, :, off].double().cpu(), untouched[t])
        assert int((kp != 9.0).any(-1).any(1).sum()) == written


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("nh, nkv, d", [(6, 2, 64), (4, 4, 128), (3, 1, 48)])
def test_attention_behind_normed_heads(dtype, nh, nkv, d, monkeypatch):
    """Decode batches (whose matrix-core kernel writes keys and values itself, or does not) and
    portions beside single tokens, in a window: against the plain sums, and the pages hold the
    same keys and values either way."""
    import rust_llm_inference_server_amd.ops as ops
    from test_kernels_gpu import paged_case
    eps, window, scale = 1e-5, 40, 3.0 / d
    cos, sin, dcos, dsin = _tables(400, {"dims": d // 2 // 16 * 16, "base": 500.0})
    dims = 2 * cos.shape[1]
    for cached, new in (([4, 99, 0, 210], [1, 1, 1, 1]), ([30, 7, 0], [1, 20, 90])):
        pages = {}
        for fuse in (True, False):
            monkeypatch.setattr(ops, "FUSE_ROPE_DECODE", fuse)
            qkv, kp, vp, bt, step, ks, vs, cu = paged_case(cached, new, nh, nkv, d, 16, dtype, seed=nh)
            raw = qkv.double().cpu().reshape(-1, nh + 2 * nkv, d)
            pos = torch.cat([torch.arange(c, c + n) for c, n in zip(cached, new)])
            slots = torch.tensor([int(bt[s, p // 16]) * 16 + p % 16
                                  for s, (c, n) in enumerate(zip(cached, new))
                                  for p in range(c, c + n)], dtype=torch.int32, device=DEV)
            turned = plain.rms(_turn(raw[:, :nh + nkv], pos, cos, sin, dims, False), eps)
            wants, at = [], 0
            for s, (c, n) in enumerate(zip(cached, new)):
                k = torch.cat([ks[s].double()[:c], turned[at:at + n, nh:].to(dtype).double()])
                v = torch.cat([vs[s].double()[:c], raw[at:at + n, nh + nkv:]])
                scores = torch.stack([turned[at:at + n, h, :] @ k[:, h // (nh // nkv)].T
                                      for h in range(nh)]) * scale
                ok = plain.visible(c + n, window)[c:]
                p = torch.softmax(scores.masked_fill(~ok, float("-inf")), -1)
                wants.append(torch.stack([p[h] @ v[:, h // (nh // nkv)] for h in range(nh)], 1)
                             .reshape(n, nh * d))
                at += n
            got = ops.norm_rope_attention(
                qkv, nh, nkv, d, d, eps, dcos, dsin, pos.to(torch.int32).to(DEV), slots, kp, vp, 16, bt,
                step, scale, window)
            assert rel(got, torch.cat(wants)) < TOL[dtype]
            pages[fuse] = [torch.stack([kp[int(s) // 16, :, int(s) % 16] for s in slots]).cpu(),
                           torch.stack([vp[int(s) // 16, :, :, int(s) % 16] for s in slots]).cpu()]
        assert all(torch.equal(a, b) for a, b in zip(pages[True], pages[False]))


def test_bad_operands_of_the_normed_heads_are_refused():
    from rust_llm_inference_server_amd import ops
    from rust_llm_inference_server_amd.ops.lib import KernelError
    qkv = torch.zeros((2, 4 * 16), device=DEV)
    pos = torch.zeros(2, dtype=torch.int32, device=DEV)
    with pytest.raises(KernelError, match="columns"):
        ops.norm_rope_kv_write(qkv, 4, 2, 16, 16, 1e-5, None, None, pos, None, None, None, 16, False)
    with pytest.raises(KernelError, match="needs pages"):
        ops.norm_rope_kv_write(qkv, 2, 1, 16, 16, 1e-5, None, None, pos, None, None, None, 16)
    wide = torch.zeros((700, 9), device=DEV)
    with pytest.raises(KernelError, match="rotated"):
        ops.norm_rope_kv_write(qkv, 2, 1, 16, 16, 1e-5, wide, wide, pos, None, None, None, 16, False)


# ------------------------------------------------------------- norms on both sides
@pytest.mark.parametrize("T, W", [(1, 40), (3, 50), (9, 200), (70, 512), (5, 2048), (130, 2048),
                                  (2, 9000), (3, 17000)])
@pytest.mark.parametrize("parts", [0, 1, 5])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_a_norm_behind_and_the_next_norm_in_one_pass(T, W, parts, dtype):
    """A sublayer's result in the activation dtype, as one float32 tensor, or as a stack of partial
    sums that is rounded once: it is normed, joins the float32 residual, and the row comes back
    under the next norm, each with its own weight and epsilon."""
    from rust_llm_inference_server_amd import ops
    eps, next_eps = 1e-3, 1e-2
    x = rnd(T, W, seed=1)
    y = rnd(max(parts, 1), T, W, seed=2, std=0.2)
    y[:, 0] *= 1e-2
    w = (1 + rnd(W, seed=3, std=0.3)).to(dtype)
    nw = (1 + rnd(W, seed=4, std=0.3)).to(dtype)
    act = torch.bfloat16 if dtype == torch.bfloat16 else torch.float32
    delta = y if parts > 1 else y[0] if parts else y[0].to(act)
    total = delta.double().sum(0) if parts > 1 else delta.double()
    if parts > 1 and act == torch.bfloat16:
        total = total.float().to(act).double()
    want_x = x.double() + plain.rms(total, eps) * w.double()
    want = plain.rms(want_x, next_eps) * nw.double()
    r = x.to(DEV).clone()
    got = ops.norm_join(r, delta.to(DEV), w.to(DEV), eps, act, round_parts=act == torch.bfloat16,
                        next_weight=nw.to(DEV), next_eps=next_eps)
    assert rel(r, want_x) < (1e-6 if parts <= 1 or act == torch.float32 else 1e-3)
    assert got.dtype == act and rel(got, want) < (1e-5 if act == torch.float32 else 4e-3)


# -------------------------------------------------------------------- the two latents
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H, d, r, R, Rq", [(3, 12, 6, 28, 20), (4, 16, 32, 64, 96), (1, 8, 2, 33, 7),
                                            (16, 64, 64, 512, 1536), (2, 24, 16, 40, 300)])
@pytest.mark.parametrize("interleaved", [False, True])
@pytest.mark.parametrize("T", [1, 37])
def test_both_latents_and_the_turned_queries(dtype, H, d, r, R, Rq, interleaved, T):
    """One kernel norms the latent and the queries' latent and writes the cache (and the copy with
    the positions innermost); another call turns the queries' last part beside what stands in
    their rows already; both together as a mixer without a queries' latent does them."""
    from rust_llm_inference_server_amd import ops
    eps, ps, D = 1e-3, 16, R + r
    rot = {"dims": r, "base": 200.0, "scaling": {"factor": 4.0, "original": 64, "fast": 8.0,
                                                 "slow": 1.0}}
    cos, sin, dcos, dsin = _tables(300, rot)
    pos = torch.randint(0, 300, (T,), generator=torch.Generator().manual_seed(5))
    pos[0] = 299
    dpos = pos.to(torch.int32).to(DEV)
    down = rnd(T, Rq + 8 + D + 3, seed=6)
    down[0] *= 1e-2
    w, qw = 1 + rnd(R, seed=7, std=0.3), 1 + rnd(Rq, seed=8, std=0.3)
    kv, cq = down[:, Rq + 8:Rq + 8 + D], down[:, :Rq]
    q = rnd(T, H * (d + r), seed=9, dtype=dtype)
    slots = torch.randperm(6 * ps, generator=torch.Generator().manual_seed(10))[:T].to(torch.int32)
    pages = torch.full((6, ps, D), 9.0, dtype=dtype, device=DEV)
    pages_t = torch.full((6, R, ps), 9.0, dtype=dtype, device=DEV)
    q_out = torch.full((T, H * D), 3.0, dtype=dtype, device=DEV)
    cq_out = torch.empty((T, Rq), dtype=dtype, device=DEV)
    on = down.to(DEV)
    ops.latent_write(on[:, Rq + 8:Rq + 8 + D], w.to(DEV), eps, R, r, r, dcos, dsin, dpos, slots.to(DEV),
                     pages, None, d + r, None, H, pages_t, interleaved,
                     (on[:, :Rq], qw.to(DEV), cq_out))
    row = torch.cat([plain.rms(kv[:, :R].double(), eps) * w.double(),
                     _turn(kv[:, R:].double().unsqueeze(1), pos, cos, sin, r, interleaved)[:, 0]], -1)
    got = pages.reshape(-1, D)[slots.long().to(DEV)]
    assert rel(got, row) < TOL[dtype] and int((pages != 9.0).any(-1).sum()) == T
    assert torch.equal(pages_t.transpose(1, 2).reshape(-1, R)[slots.long().to(DEV)], got[:, :R])
    assert rel(cq_out, plain.rms(cq.double(), eps) * qw.double()) < TOL[dtype]
    assert bool((q_out == 3.0).all())
    before = pages.clone()
    ops.latent_write(None, None, eps, R, r, r, dcos, dsin, dpos, None, pages, q.to(DEV), d + r, q_out, H,
                     None, interleaved)
    heads = q.double().reshape(T, H, d + r)[..., d:]
    out = q_out.reshape(T, H, D)
    assert rel(out[..., R:], _turn(heads, pos, cos, sin, r, interleaved)) < TOL[dtype]
    assert bool((out[..., :R] == 3.0).all()) and torch.equal(pages, before)
    both = torch.full((T, H * D), 3.0, dtype=dtype, device=DEV)
    pages2 = torch.full((6, ps, D), 9.0, dtype=dtype, device=DEV)
    ops.latent_write(on[:, Rq + 8:Rq + 8 + D], w.to(DEV), eps, R, r, r, dcos, dsin, dpos, slots.to(DEV),
                     pages2, q.to(DEV), d + r, both, H, None, interleaved)
    assert torch.equal(pages2, pages)
    # (another kernel turns queries alone: the same products and sum)
    assert rel(both, q_out) < 1e-6 if dtype == torch.float32 else rel(both, q_out) < 3e-3


# ------------------------------------------------------------------ experts and identities
@pytest.mark.parametrize("E, identity, top", [(8, 4, 2), (3, 9, 5), (1, 1, 2), (64, 70, 12), (5, 0, 5)])
@pytest.mark.parametrize("T", [1, 65])
def test_softmax_choice_over_all_experts(E, identity, top, T):
    """Scores are the softmax over experts and identities; corrections (negative ones that push a
    choice score below zero among them) move the choice alone; weights are the scores."""
    from rust_llm_inference_server_amd import ops
    n = E + identity
    z, corr = rnd(T, n, seed=1, std=2.0), rnd(n, seed=2, std=0.6)
    chosen, weights = plain.choose(z.double(), corr.double(), top)
    got, gw = ops.route(z.to(DEV), corr.to(DEV), 1, 1, top, 1.0, scores="softmax", group_score="max")
    assert torch.equal(got.long().cpu(), chosen)
    assert rel(gw, weights) < 1e-5


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("T, E, identity, top, W, F", [
    (1, 4, 2, 3, 48, 24), (37, 5, 3, 3, 50, 30), (64, 2, 6, 4, 40, 16), (200, 8, 4, 2, 128, 64),
    (700, 4, 4, 4, 64, 72), (3, 1, 1, 2, 9, 5)])
def test_units_that_hand_back_their_input(dtype, T, E, identity, top, W, F):
    """Tiles of 16, 64 and 128 rows; rows that choose identities alone, experts alone and both; x
    with a row stride of its own."""
    from rust_llm_inference_server_amd import ops
    wide = rnd(T, W + 8, seed=1, dtype=dtype)
    x = wide[:, :W]
    gate, up = rnd(E, F, W, seed=2, std=W ** -0.5), rnd(E, F, W, seed=3, std=W ** -0.5)
    down = rnd(E, W, F, seed=4, std=F ** -0.5)
    gu, dn = torch.cat([gate, up], 1).to(dtype), down.to(dtype)
    z = rnd(T, E + identity, seed=5, std=2.0)
    z[0, :E] -= 50.0 if identity >= top else 0.0
    chosen, weights = plain.choose(z, torch.zeros(E + identity), top)
    weights = weights.float()
    if identity == top and T > 1:
        assert bool((chosen[0] >= E).all())
    want = torch.zeros(T, W, dtype=torch.float64)
    w = {}
    for e in range(E):
        w.update({f"e{e}.gate": gu[e, :F].double(), f"e{e}.up": gu[e, F:].double(),
                  f"e{e}.down": dn[e].double()})
    for t in range(T):
        for e, wt in zip(chosen[t].tolist(), weights[t].tolist()):
            h = x[t].double()
            want[t] += wt * (h if e >= E else plain.gated_unit(h, w, f"e{e}."))
    got = ops.routed_units(wide.to(DEV)[:, :W], gu.to(DEV), dn.to(DEV), chosen.to(torch.int32).to(DEV),
                           weights.to(DEV).contiguous(), identity=True)
    assert got.dtype == torch.float32 and rel(got, want) < (2e-5 if dtype == torch.float32 else 8e-3)


def test_every_choice_an_identity():
    from rust_llm_inference_server_amd import ops
    x = rnd(20, 32, seed=1).to(DEV)
    gu, dn = torch.full((2, 16, 32), math.nan, device=DEV), torch.full((2, 32, 8), math.nan, device=DEV)
    chosen = torch.tensor([[2, 3]] * 20, dtype=torch.int32, device=DEV)
    weights = torch.tensor([[0.25, 0.5]] * 20, device=DEV)
    got = ops.routed_units(x, gu, dn, chosen, weights, identity=True)
    assert rel(got, x * 0.75) < 1e-6
