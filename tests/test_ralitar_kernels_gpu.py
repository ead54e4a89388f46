"""Each kernel that the Ralitar design added or extended, alone, against the plain formulas of
``plain_ralitar.py`` (float64), at sizes the models of the other tests do not have: chunked
attention through the vector-unit, matrix-core and generic kernels (portions beside single tokens,
decode partitions, key runs, tiles of 128 queries); the norm on its way into the residual from
whole rows and stacks of partial sums; the pair table; the token input's gate; rows of queries and
keys behind whole-row norms in both rotation layouts; the channel-wise delta rule and the gated
linear recurrence in every form, state carried over steps in slots that are not in order; the
convolution with a bias on its inputs."""
import math

import pytest
import torch

import plain_ralitar as plain
from test_gipotar_kernels_gpu import SLOTS, STEPS, _cut, _meta, _ops, _state

pytestmark = pytest.mark.gpu
DEV = "cuda"


def rel(got, want):
    return float((got.double().cpu() - want.double().cpu()).norm() / want.double().cpu().norm())


# ------------------------------------------------------------------------------ attention
def _reference(qkv, ks, vs, cu, cached, new, nh, nkv, d, scale, chunk, cap):
    outs = []
    q_all = qkv.double().cpu()[:, :nh * d]
    for s, (c, n) in enumerate(zip(cached, new)):
        q = q_all[cu[s]:cu[s + 1]].reshape(n, nh, d)
        ok = plain.chunk_mask(torch.arange(c + n), chunk)[c:]
        kk = ks[s].double().repeat_interleave(nh // nkv, dim=1)
        vv = vs[s].double().repeat_interleave(nh // nkv, dim=1)
        sc = torch.einsum("ihd,jhd->hij", q, kk) * scale
        if cap:
            sc = cap * torch.tanh(sc / cap)
        w = torch.softmax(sc.masked_fill(~ok, -math.inf), dim=-1)
        outs.append(torch.einsum("hij,jhd->ihd", w, vv).reshape(n, nh * d))
    return torch.cat(outs)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("nh,nkv,d,ps", [(6, 2, 32, 8), (5, 5, 48, 16), (32, 8, 64, 16),
                                         (8, 2, 128, 16), (4, 1, 80, 16)])
def test_attention_inside_chunks(dtype, nh, nkv, d, ps, monkeypatch):
    """Chunks of 1, 7, a page, 50, 64, 300, 1,000 and more than any context, with and without a
    cap; queries at a chunk's first and last position, portions over several chunks, contexts of
    several chunks.  A chunk that is one position longer is far off."""
    from test_kernels_gpu import attention_constants, key_runs, paged_case
    import rust_llm_inference_server_amd.ops as ops
    scale = 1.0 / math.sqrt(d)
    tol = 2e-5 if dtype == torch.float32 else 2e-2
    for cached, new in (([0, 5, 40, 130, 17], [33, 1, 70, 2, 64]), ([4, 99, 0, 639, 640], [1] * 5),
                        ([1, 1100], [1, 1]), ([1200, 2], [1, 130]), ([20], [300]), ([700], [90])):
        for chunk, cap in ((1, 0.0), (7, 2.0), (ps, 0.0), (50, 3.0), (64, 0.0), (300, 2.0),
                           (1000, 0.0), (5000, 4.0)):
            qkv, kp, vp, bt, step, ks, vs, cu = paged_case(cached, new, nh, nkv, d, ps, dtype,
                                                           seed=nh + 5, q_scale=2.0)
            want = _reference(qkv, ks, vs, cu, cached, new, nh, nkv, d, scale, chunk, cap)
            for matrix in (True, False):
                monkeypatch.setattr(ops, "SHAPED_SCORES_MATRIX", matrix)
                with attention_constants(DECODE_PART_KEYS=256, PREFILL_WIDE_MIN_GROUPS=0,
                                         **key_runs(3)):
                    for force in (None, "generic"):
                        got = ops.paged_attention(qkv, nh, nkv, d, kp, vp, ps, bt, step, scale,
                                                  force=force, chunk=chunk, softcap=cap)
                        assert rel(got, want) < tol, (cached, new, chunk, cap, matrix, force)
                got = ops.paged_attention(qkv, nh, nkv, d, kp, vp, ps, bt, step, scale, chunk=chunk,
                                          softcap=cap)
                assert rel(got, want) < tol, (cached, new, chunk, cap, matrix)
            asked = [p for c, n in zip(cached, new) for p in range(c, c + n)]
            if dtype == torch.float32 and any(p % chunk != p % (chunk + 1) for p in asked):
                off = ops.paged_attention(qkv, nh, nkv, d, kp, vp, ps, bt, step, scale,
                                          chunk=chunk + 1, softcap=cap)
                assert rel(off, want) > 5e-5


def test_attention_refuses_a_window_beside_chunks():
    from test_kernels_gpu import paged_case
    ops = _ops()
    qkv, kp, vp, bt, step, *_ = paged_case([3], [4], 2, 1, 32, 16, torch.float32, seed=1)
    with pytest.raises(ops.KernelError, match="not both"):
        ops.paged_attention(qkv, 2, 1, 32, kp, vp, 16, bt, step, 0.2, 8, chunk=8)


# ------------------------------------------------------------------------- the residual
@pytest.mark.parametrize("T, W", [(1, 40), (3, 50), (9, 200), (70, 512), (5, 2048), (130, 2048),
                                  (2, 3072), (4, 5000), (3, 9000), (2, 20000), (11, 125)])
@pytest.mark.parametrize("parts", [0, 1, 5, 14])
@pytest.mark.parametrize("w_dtype", [torch.float32, torch.bfloat16])
def test_norm_on_the_way_into_the_residual(T, W, parts, w_dtype):
    """Whole rows in either dtype (parts 0: bfloat16) and stacks of partial sums, with and without
    the rounding of the sum; the residual comes back in bfloat16, as itself or not at all."""
    ops = _ops()
    g = torch.Generator().manual_seed(T * 7 + W + parts)
    x = torch.randn(T, W, generator=g)
    w = (1.0 + 0.3 * torch.randn(W, generator=g)).to(w_dtype)
    if parts == 0:
        y = (torch.randn(T, W, generator=g) * 0.2).to(torch.bfloat16)
    elif parts == 1:
        y = torch.randn(T, W, generator=g) * 0.2
    else:
        y = torch.randn(parts, T, W, generator=g) * 0.1
    for rounds in (False, True):
        total = (y.double().sum(0) if y.dim() == 3 else y.double())
        if rounds and y.dim() == 3:
            total = y.sum(0).to(torch.bfloat16).double()
        want = x.double() + plain.unit(total, 1e-3) * w.double()
        for out_dtype in (torch.bfloat16, torch.float32, None):
            r = x.to(DEV).clone()
            out = ops.norm_join(r, y.to(DEV), w.to(DEV), 1e-3, out_dtype, round_parts=rounds)
            assert float((r.double().cpu() - want).abs().max()) < (2e-2 if rounds else 2e-5)
            if out_dtype is None:
                assert out is None
            elif out_dtype == torch.float32:
                assert out.data_ptr() == r.data_ptr()
            else:
                assert torch.equal(out, r.to(torch.bfloat16))
    r = x.to(DEV)
    assert torch.equal(ops.norm_join(r, None, None, 0.0, torch.bfloat16), r.to(torch.bfloat16))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_geglu_and_the_token_input(dtype):
    ops = _ops()
    g = torch.Generator().manual_seed(3)
    tol = 2e-6 if dtype == torch.float32 else 6e-3
    for T, I in ((1, 7), (5, 64), (33, 100), (300, 2048)):
        gu = (torch.randn(T, 2 * I, generator=g) * 2.0).to(dtype)
        want = plain.gelu_tanh(gu[:, :I].double()) * gu[:, I:].double()
        assert rel(ops.geglu(gu.to(DEV)), want) < tol
    for T, W, I in ((1, 96, 40), (7, 256, 64), (16, 2048, 512), (21, 1024, 256), (50, 512, 128),
                    (3, 50, 30), (25, 512, 48), (32, 2048, 80)):
        x = torch.randn(T, W, generator=g).to(dtype)
        w = (torch.randn(2 * I, W, generator=g) * W ** -0.5).to(dtype)
        gu = x.double() @ w.double().T
        want = plain.gelu_tanh(gu[:, :I]) * gu[:, I:]
        assert rel(ops.linear_geglu(x.to(DEV), w.to(DEV)), want) < 2 * tol
    for T, n, parts, V in ((1, 5, 3, 11), (40, 64, 4, 50), (9, 256, 2, 300)):
        z = torch.randn(T, n, generator=g).to(dtype)
        table = torch.randn(V, parts * n, generator=g).to(dtype)
        ids = torch.randint(0, V, (T,), generator=g, dtype=torch.int32)
        for part in range(parts):
            want = plain.gelu_tanh(z.double()) * table[ids.long()][:, part * n:(part + 1) * n].double()
            got = ops.side_gate_(z.to(DEV).clone(), table.to(DEV), part * n, ids.to(DEV))
            assert rel(got, want) < tol


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("buckets, mul_prev, mul_cur", [(1, 1, 1), (97, 29, 12),
                                                        (5003, 2147483629, 2147483647)])
def test_pair_table_over_steps(dtype, buckets, mul_prev, mul_cur):
    """Three sequences over several steps (single tokens and portions), each step's first token
    behind the last one of the step before; slots that are not in order, other slots untouched."""
    ops = _ops()
    W = 24
    g = torch.Generator().manual_seed(buckets)
    table, pairs = torch.randn(500, W, generator=g).to(dtype), torch.randn(buckets + 1, W, generator=g).to(dtype)
    seqs = [torch.randint(0, 500, (sum(s[i] for s in STEPS),), generator=g).tolist() for i in range(3)]
    buf = torch.full((4, 20), 9, dtype=torch.int32, device=DEV)
    last = buf[:, 4:5]
    last[SLOTS] = 0
    got = [[], [], []]
    for step, lengths in enumerate(STEPS):
        cu, slots, seq = _meta(lengths, SLOTS)
        ids = torch.tensor([t for i in range(3) for t in seqs[i][_cut(None, STEPS, step, i)]],
                           dtype=torch.int32, device=DEV)
        out = ops.embed_pairs(ids, table.to(DEV), 1.5, pairs.to(DEV), mul_prev, mul_cur, last, seq,
                              cu, slots).cpu()
        for i, rows in enumerate(out.split(lengths)):
            got[i].append(rows)
    for i in range(3):
        rows = plain.bigram_rows(seqs[i], {"buckets": buckets, "mul_prev": mul_prev,
                                           "mul_cur": mul_cur})
        want = table[torch.tensor(seqs[i])].double() * 1.5 + pairs[torch.tensor(rows)].double()
        assert float((torch.cat(got[i]).double() - want).abs().max()) < 1e-5
        assert int(last[SLOTS[i]].cpu()) == seqs[i][-1] + 1
    assert int(buf[1, 4]) == 9 and int(buf[:, 5:].min()) == 9


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("nh, nkv, D, real, rot", [(4, 2, 16, 16, 12), (3, 1, 48, 36, 36),
                                                   (8, 2, 64, 64, 64), (2, 2, 128, 128, 32),
                                                   (5, 5, 6, 6, 4), (1, 1, 32, 20, 0),
                                                   (40, 8, 128, 128, 128), (60, 20, 160, 152, 8),
                                                   (96, 32, 256, 256, 256)])
@pytest.mark.parametrize("interleaved", [True, False])
def test_rows_behind_whole_row_norms(dtype, nh, nkv, D, real, rot, interleaved):
    """Biases, norms over whole rows, both rotation layouts, values as the keys in front of the
    norm; rows that carry gates behind the heads, heads padded with zeros."""
    ops = _ops()
    g = torch.Generator().manual_seed(nh * 100 + D + rot)
    T, extra, eps = 13, 16, 1e-3
    cols = (nh + nkv) * D
    pad = torch.zeros(nh + nkv, D)
    pad[:, :real] = 1.0
    pad = pad.reshape(-1)
    p = torch.cat([torch.randn(T, cols, generator=g) * pad, torch.randn(T, extra, generator=g)],
                  dim=1).to(dtype)
    bias = torch.randn(cols, generator=g) * pad
    wq, wk = torch.randn(nh * D, generator=g) * pad[:nh * D], torch.randn(nkv * D, generator=g) * pad[nh * D:]
    pos = torch.randint(0, 600, (T,), generator=g, dtype=torch.int32)
    cos = sin = None
    if rot:
        f = plain.frequencies({"dims": rot, "base": 500.0})
        ang = torch.arange(600, dtype=torch.float64).reshape(-1, 1) * f
        cos, sin = torch.cos(ang).float(), torch.sin(ang).float()
    x = p[:, :cols].double() + bias.double()
    parts = []
    for rows, heads, w in ((x[:, :nh * D], nh, wq), (x[:, nh * D:], nkv, wk)):
        keep = pad.bool()[:heads * D]
        y = torch.zeros_like(rows)
        y[:, keep] = plain.unit(rows[:, keep], eps)
        y = (y * w.double()).reshape(T, heads, D)
        if rot and interleaved:
            y = plain.rotate_pairs(y, pos, {"dims": rot, "base": 500.0})
        elif rot:
            c, s = cos[pos.long()].double()[:, None], sin[pos.long()].double()[:, None]
            a, b = y[..., :rot // 2].clone(), y[..., rot // 2:rot].clone()
            y[..., :rot // 2], y[..., rot // 2:rot] = a * c - b * s, b * c + a * s
        parts.append(y.reshape(T, -1))
    want = torch.cat(parts + [x[:, nh * D:]], dim=1)
    dev = lambda t: None if t is None else t.to(DEV)
    got = ops.row_prepare(dev(p), nh, nkv, D, real, dev(bias), dev(wq), dev(wk), eps, dev(cos),
                          dev(sin), dev(pos), interleaved)
    assert rel(got, want) < (2e-6 if dtype == torch.float32 else 5e-3)


# ------------------------------------------------------------------------ the recurrences
@pytest.mark.parametrize("tiled", [False, "wide", "narrow", None, "chunked"])
@pytest.mark.parametrize("heads, kv_heads, dk, dv", [(4, 2, 16, 24), (2, 1, 96, 50), (3, 3, 160, 33),
                                                     (2, 2, 64, 64), (1, 1, 128, 128)])
def test_channel_delta_scan(heads, kv_heads, dk, dv, tiled):
    """One decay per head and key channel, from near one to near zero; the state carried over
    steps with runs that end at, before and behind a tile's edge."""
    ops = _ops()
    if tiled == "chunked" and dk > 128:
        pytest.skip("the chunked form takes up to 128 key channels")
    g = torch.Generator().manual_seed(heads * 1000 + dk)
    totals = [sum(s[i] for s in STEPS) for i in range(3)]
    rand = lambda T, n: torch.randn(T, n, generator=g)
    data = []
    for T in totals:
        q, k = (t / t.norm(dim=-1, keepdim=True) for t in
                (rand(T, kv_heads * dk).reshape(T, kv_heads, dk) for _ in range(2)))
        data.append({"q": q.reshape(T, -1), "k": k.reshape(T, -1), "v": rand(T, heads * dv),
                     "b": rand(T, heads), "z": rand(T, heads * dk) * 2.0})
    a_log, dt = torch.rand(heads, generator=g) * 3.0 - 2.5, rand(1, heads * dk).reshape(-1) - 1.0
    buf, state = _state(4, heads * dv * dk)
    state[SLOTS] = 0.0
    want = []
    for x in data:
        T = x["q"].shape[0]
        dec = torch.exp(-torch.exp(a_log.double()).reshape(1, heads, 1)
                        * plain.softplus(x["z"].double() + dt.double()).reshape(T, heads, dk))
        q, k = (x[n].double().reshape(T, kv_heads, dk) for n in "qk")
        v = x["v"].double().reshape(T, heads, dv)
        want.append(torch.cat([plain.channel_delta_scan(
            q[:, h // (heads // kv_heads)], k[:, h // (heads // kv_heads)], v[:, h], dec[:, h],
            torch.sigmoid(x["b"].double()[:, h])) for h in range(heads)], dim=1))
    got = [[], [], []]
    for step, lengths in enumerate(STEPS):
        cu, slots, _ = _meta(lengths, SLOTS)
        rows = {n: torch.cat([data[i][n][_cut(None, STEPS, step, i)] for i in range(3)]).to(DEV)
                for n in data[0]}
        qkv = torch.cat([rows["q"], rows["k"], rows["v"]], dim=1).contiguous()
        bz = torch.cat([rows["z"], rows["b"]], dim=1).contiguous()
        n = kv_heads * dk
        o = ops.channel_delta_scan(qkv[:, :n], qkv[:, n:2 * n], qkv[:, 2 * n:], bz[:, heads * dk:],
                                   bz[:, :heads * dk], a_log.to(DEV), dt.to(DEV), state, cu, slots, 3,
                                   heads, kv_heads, dk, dv, tiled=tiled).cpu()
        for i, part in enumerate(o.split(lengths)):
            got[i].append(part)
    for i in range(3):
        assert rel(torch.cat(got[i]), want[i]) < 1e-5
    assert float((buf[1] - 7.5).abs().max()) == 0.0
    assert float((buf[:, :8] - 7.5).abs().max()) == 0.0


@pytest.mark.parametrize("strength", [0.0, 3.0, 9.0])
@pytest.mark.parametrize("heads, kv_heads, dk, dv", [(2, 1, 128, 128), (3, 3, 40, 70)])
def test_long_runs_of_the_channel_delta_rule(heads, kv_heads, dk, dv, strength):
    """Hundreds of tokens in one step beside short ones, in chunks on the matrix cores: decays that
    hardly forget, and decays so strong that their products over a few tokens leave the float32
    range (a single token may wipe a channel out between tokens that keep it)."""
    ops = _ops()
    g = torch.Generator().manual_seed(dk + int(strength))
    lengths, slots_of = [1, 500, 65, 64, 7], [4, 0, 2, 5, 1]
    T = sum(lengths)
    rand = lambda *shape: torch.randn(*shape, generator=g)
    q, k = (t / t.norm(dim=-1, keepdim=True) for t in (rand(T, kv_heads, dk), rand(T, kv_heads, dk)))
    v, b = rand(T, heads * dv), rand(T, heads)
    z = rand(T, heads * dk) * 2.0
    z[torch.rand(T, heads * dk, generator=g) < 0.02] = 60.0
    a_log, dt = torch.full((heads,), strength - 4.0), rand(heads * dk) - 2.0
    start = rand(6, heads, dv, dk)
    buf, state = _state(6, heads * dv * dk)
    state.copy_(start.reshape(6, -1))
    cu, slots, _ = _meta(lengths, slots_of)
    qkv = torch.cat([q.reshape(T, -1), k.reshape(T, -1), v], dim=1).to(DEV)
    n = kv_heads * dk
    got = ops.channel_delta_scan(qkv[:, :n], qkv[:, n:2 * n], qkv[:, 2 * n:], b.to(DEV), z.to(DEV),
                                 a_log.to(DEV), dt.to(DEV), state, cu, slots, 5, heads, kv_heads,
                                 dk, dv, longest=max(lengths)).double().cpu()
    dec = torch.exp(-torch.exp(a_log.double()).reshape(1, heads, 1)
                    * plain.softplus(z.double() + dt.double()).reshape(T, heads, dk))
    beta, at = torch.sigmoid(b.double()), 0
    for length, slot in zip(lengths, slots_of):
        S = start[slot].double().transpose(1, 2).clone()                     # [head][key][value]
        for t in range(at, at + length):
            for h in range(heads):
                kt, qt = k[t, h // (heads // kv_heads)].double(), q[t, h // (heads // kv_heads)].double()
                S[h] = dec[t, h].reshape(-1, 1) * S[h]
                u = beta[t, h] * (v[t, h * dv:(h + 1) * dv].double() - S[h].T @ kt)
                S[h] = S[h] + torch.outer(kt, u)
                want = S[h].T @ qt
                assert float((got[t, h * dv:(h + 1) * dv] - want).abs().max()) < 1e-4, (length, t - at)
        left = state[slot].cpu().double().reshape(heads, dv, dk)
        assert float((left - S.transpose(1, 2)).abs().max()) < 1e-4
        at += length
    assert float((state[3].cpu() - start[3].reshape(-1)).abs().max()) == 0.0


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("C, blocks", [(40, 1), (60, 3), (33, 3), (512, 2), (4200, 4)])
@pytest.mark.parametrize("chunked", [False, True])
def test_gated_linear_recurrence(dtype, C, blocks, chunked, monkeypatch):
    """Decays from one to near zero, states carried over steps, both forms: token by token, and in
    chunks of four tokens that are joined in order."""
    import rust_llm_inference_server_amd.ops.recurrent as rec
    ops = _ops()
    if chunked:
        monkeypatch.setattr(rec, "RGLRU_CHUNK_LEN", 4)
    g = torch.Generator().manual_seed(C + blocks)
    n = C // blocks
    totals = [sum(s[i] for s in STEPS) for i in range(3)]
    data = [{"u": torch.randn(T, C, generator=g).to(dtype), "y": torch.randn(T, C, generator=g),
             "g": torch.randn(T, 2 * C, generator=g) * 2.0} for T in totals]
    rb, ib, yb = (torch.randn(C, generator=g) for _ in range(3))
    rate = -8.0 * torch.nn.functional.softplus(torch.rand(C, generator=g) * 8.0 - 7.0)
    buf, state = _state(4, C)
    state[SLOTS] = 0.0
    want = []
    for x in data:
        gates = x["g"].double().reshape(-1, blocks, 2, n)
        r = torch.sigmoid(gates[:, :, 0].reshape(-1, C) + rb.double())
        i = torch.sigmoid(gates[:, :, 1].reshape(-1, C) + ib.double())
        S = plain.rglru_scan(rate.double() * r, i * x["u"].double())
        want.append(S * plain.gelu_tanh(x["y"].double() + yb.double()))
    got = [[], [], []]
    for step, lengths in enumerate(STEPS):
        cu, slots, _ = _meta(lengths, SLOTS)
        rows = {k: torch.cat([data[i][k][_cut(None, STEPS, step, i)] for i in range(3)]).to(DEV)
                for k in data[0]}
        wide = torch.cat([torch.zeros_like(rows["y"]), rows["y"]], dim=1).contiguous()
        out = ops.rglru_scan(rows["u"], rows["g"], rb.to(DEV), ib.to(DEV), rate.to(DEV),
                             wide[:, C:], yb.to(DEV), state, cu, slots, 3, blocks,
                             longest=1000 if chunked else 1).float().cpu()
        for i, part in enumerate(out.split(lengths)):
            got[i].append(part)
    for i in range(3):
        assert rel(torch.cat(got[i]), want[i]) < (5e-6 if dtype == torch.float32 else 5e-3)
    assert float((buf[1] - 7.5).abs().max()) == 0.0


def test_a_slow_decay_keeps_what_it_took():
    """Over 3,000 tokens in one step, decays of 1 - 1e-6: the first token's input is still there,
    in chunks and token by token (1 - a^2 must not lose its digits; what is lost is a's own
    rounding, 3e-8 a token)."""
    ops = _ops()
    C, T = 64, 3000
    gates = torch.full((T, 2 * C), -12.0)
    u = torch.zeros(T, C)
    u[0] = 1e4
    y = torch.full((T, C), 3.0)
    zero, rate = torch.zeros(C), torch.full((C,), -0.2)
    r = torch.sigmoid(gates[:, :C].double())
    want = plain.rglru_scan(rate.double() * r, torch.sigmoid(gates[:, C:].double()) * u.double())
    want = want * plain.gelu_tanh(y.double())
    for longest in (1, T):
        state = torch.zeros(1, C, device=DEV)
        cu, slots, _ = _meta([T], [0])
        out = ops.rglru_scan(u.to(DEV), gates.to(DEV), zero.to(DEV), zero.to(DEV), rate.to(DEV),
                             y.to(DEV), zero.to(DEV), state, cu, slots, 1, 1, longest=longest)
        assert rel(out, want) < 2e-4


@pytest.mark.parametrize("K", [1, 2, 5])
def test_convolution_with_a_bias_on_its_inputs(K):
    """The zeros in front of a sequence are zeros, not the bias; the rows a step leaves behind are
    the biased ones."""
    ops = _ops()
    C = 50
    g = torch.Generator().manual_seed(K)
    totals = [sum(s[i] for s in STEPS) for i in range(3)]
    data = [torch.randn(T, C + 6, generator=g) for T in totals]
    taps, bias, in_bias = torch.randn(C, K, generator=g), torch.randn(C, generator=g), torch.randn(C, generator=g)
    buf, state = _state(4, max(1, C * (K - 1)))
    state[SLOTS] = 0.0
    got = [[], [], []]
    for step, lengths in enumerate(STEPS):
        cu, slots, seq = _meta(lengths, SLOTS)
        x = torch.cat([data[i][_cut(None, STEPS, step, i)] for i in range(3)]).to(DEV)
        out = ops.causal_conv(x, taps.to(DEV), state, seq, cu, slots, 3, bias=bias.to(DEV),
                              activation=False, in_bias=in_bias.to(DEV)).cpu()
        ops.tail_update(state, x, C, K - 1, cu, slots, 3, bias=in_bias.to(DEV))
        for i, part in enumerate(out.split(lengths)):
            got[i].append(part)
    for i in range(3):
        want = plain.short_conv(data[i][:, :C].double() + in_bias.double(), taps.double(), bias.double())
        assert rel(torch.cat(got[i]), want) < 1e-6


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("K", [1, 2, 3, 4, 5])
def test_convolution_that_keeps_its_tail(K, dtype):
    """Layouts in steps of four channels, and one that is not: portions long and short, steps in
    which every sequence brings one token, unit vectors over 4 to 256 channels; the rows left for
    the next step are those of the separate update, bit for bit."""
    ops = _ops()
    steps = [[1, 1, 1], [2, 700, 5], [1, 1, 1], [1, 1, 1], [K, 1, 3], [1, 1, 1]]
    for unit_group, heads, rest, extra in ((4, 6, 20, 4), (64, 3, 1100, 0), (256, 2, 36, 8),
                                           (0, 0, 36, 4), (48, 2, 8, 4), (16, 2, 9, 3)):
        U, C = unit_group * heads, unit_group * heads + rest
        g = torch.Generator().manual_seed(K * 1000 + C)
        totals = [sum(s[i] for s in steps) for i in range(3)]
        xs = [torch.randn(T, C + extra, generator=g) for T in totals]
        taps, bias, in_bias = (torch.randn(C, K, generator=g), torch.randn(C, generator=g),
                               torch.randn(C, generator=g))
        scaled = heads // 2 * unit_group
        want = []
        for x in xs:
            y = plain.short_conv(x[:, :C].double() + in_bias.double(), taps.double(), bias.double())
            y = y * torch.sigmoid(y)
            if U:
                u = y[:, :U].reshape(-1, heads, unit_group)
                u = (u / torch.sqrt((u * u).sum(-1, keepdim=True) + 1e-6)).reshape(-1, U)
                u[:, :scaled] *= 0.3
                y = torch.cat([u, y[:, U:]], 1)
            want.append(y)
        width = max(4, C * (K - 1))
        states = []
        for _ in range(2):
            buf = torch.full((4, width + 4), 7.5, device=DEV)
            state = buf[:, :width]
            state[SLOTS] = 0.0
            states.append((buf, state))
        for step, lengths in enumerate(steps):
            cu, slots, seq = _meta(lengths, SLOTS)
            x = torch.cat([xs[i][_cut(None, steps, step, i)] for i in range(3)]).to(DEV)
            outs = []
            for (_, state), keep in zip(states, (True, False)):
                outs.append(ops.causal_conv(
                    x, taps.to(DEV), state, seq, cu, slots, 3, unit_channels=U,
                    unit_group=unit_group, scaled_channels=scaled, scale=0.3, unit_eps=1e-6,
                    rest_group=64, bias=bias.to(DEV), in_bias=in_bias.to(DEV), out_dtype=dtype,
                    keep_tail=keep))
            if K > 1:
                ops.tail_update(states[1][1], x, C, K - 1, cu, slots, 3, bias=in_bias.to(DEV))
            assert torch.equal(outs[0], outs[1]) and torch.equal(states[0][0], states[1][0])
            for i, part in enumerate(outs[0].cpu().split(lengths)):
                ref = want[i][_cut(None, steps, step, i)]
                tol = 1e-5 if dtype == torch.float32 else 1e-2
                assert torch.allclose(part.double(), ref, rtol=tol, atol=tol)
        assert float(states[0][0][1].min()) == 7.5


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("N, K", [(100, 72), (40, 128), (64, 30)])
def test_products_per_head_by_number_of_rows(dtype, N, K):
    """Rows on both sides of every form's edge agree with the same rows alone."""
    ops = _ops()
    H, T = 3, 600
    g = torch.Generator().manual_seed(N)
    x = torch.randn(T, H * K, generator=g).to(dtype)
    w = (torch.randn(H, N, K, generator=g) * K ** -0.5).to(dtype)
    want = torch.matmul(x.double().reshape(T, H, K).transpose(0, 1).contiguous(),
                        w.double().transpose(1, 2).contiguous()).transpose(0, 1).reshape(T, H * N)
    whole = ops.head_linear(x.to(DEV), w.to(DEV), K, out_dtype=torch.float32)
    assert rel(whole, want) < (2e-6 if dtype == torch.float32 else 5e-3)
    for rows in (1, 16, 17, 64, 65, 256, 511, 512, 513):
        part = ops.head_linear(x[:rows].to(DEV), w.to(DEV), K, out_dtype=torch.float32)
        assert rel(part, want[:rows]) < (2e-6 if dtype == torch.float32 else 5e-3)
        if dtype == torch.bfloat16:
            assert torch.equal(part, whole[:rows])
