"""The Pozelix decoder in the engine against the plain implementation (``plain_pozelix.py``): whole
prompts, token-by-token decoding, portions down to two tokens, batches of unequal requests with
pages used again, long decoding, keys made to stand out far away, at page borders, just inside and
just outside every window (also of layers that run several times, each pass with a cache of its
own), the first tokens of a sequence, and greedy generation through the engine's scheduler.  Every
case runs on the GPU (``-m gpu``, float32 and bfloat16) and, with the kernels replaced by the slow
torch double, on the CPU, where it tests the host logic: the run order and its caches, the
junctions, the residual stream's pending norms, the step layout."""
import copy
import json

import pytest
import torch

import plain_pozelix as plain
import pozelix_models as pm
import traces
from rust_llm_inference_server_amd.config import ConfigError, EngineConfig
from rust_llm_inference_server_amd.sampling import SamplingParams

BACKENDS = ["double", pytest.param("gpu", marks=pytest.mark.gpu)]


@pytest.fixture(params=BACKENDS)
def backend(request):
    if request.param == "double":
        import cpu_ops
        cpu_ops.install(request.getfixturevalue("monkeypatch"))
        return torch.device("cpu")
    return torch.device("cuda", 0)


@pytest.fixture(params=["float32", pytest.param("bfloat16", marks=pytest.mark.gpu)])
def dtype(request, backend):
    if request.param == "bfloat16" and backend.type != "cuda":
        pytest.skip("bfloat16 runs on the GPU only")
    return request.param


_CACHE = {}


def model_case(name, dtype, tmp_path_factory, weights=None, tag="", config=None):
    """(folder, config, the stored numbers in float64) of a configuration; made once."""
    key = (name, dtype, tag)
    if key not in _CACHE:
        cfg = config if config is not None else pm.CONFIGS[name]
        w = weights if weights is not None else pm.make_weights(cfg, seed=len(name) + 23)
        store = torch.float32 if dtype == "float32" else torch.bfloat16
        folder = pm.write_folder(tmp_path_factory.mktemp(f"pozelix_{name}_{dtype}{tag}"), cfg, w,
                                 store)
        _CACHE[key] = (folder, cfg, pm.as_stored(w, store))
    return _CACHE[key]


def runner_for(folder, device, dtype, num_pages=64, page_size=16, max_num_seqs=4,
               max_positions=512, use_graphs=True):
    from rust_llm_inference_server_amd.engine import ModelRunner, load_model
    model = load_model(folder, dtype, max_positions, device)
    return ModelRunner(model, num_pages=num_pages, page_size=page_size,
                       max_num_seqs=max_num_seqs, use_graphs=use_graphs)


def check_trace(runner, steps, reqs, cfg, stored, dtype):
    """Replay ``steps`` and hold every wanted row against the plain logits of its request."""
    outputs = traces.replay_in_process(runner, steps)
    got = traces.collect(steps, outputs, cfg["vocab"])
    errors = []
    for rid, tokens in reqs.items():
        want = pm.plain_logits(plain, cfg, stored, tokens)
        assert sorted(got[rid]) == list(range(len(tokens)))
        errors += [pm.row_error(row, want[pos]) for pos, row in got[rid].items()]
    pm.judge(errors, dtype)


# ----------------------------------------------------------------------- configuration
def test_config_round_trip_and_the_specification():
    from rust_llm_inference_server_amd.registry import architecture_of
    for cfg in pm.CONFIGS.values():
        arch = architecture_of(cfg)
        assert arch.name == "Pozelix"
        assert arch.config_to_dict(arch.parse_config(cfg)) == cfg
    spec = pm.spec_of(pm.CONFIG_A)
    names = {t.name: tuple(t.shape) for t in spec.tensor_specs()}
    assert names["embed"] == (97, 48) and names["head"] == (97, 48) and names["loop.in"] == (48, 96)
    assert names["l0.mix.v"] == (48, 48) and names["l0.mix.g"] == (4, 48)
    assert names["l1.mix.dq"] == (40, 48) and names["l1.mix.dq.norm"] == (40,)
    assert names["l1.mix.uq"] == (3 * 28, 40) and names["l1.mix.dkv"] == (36, 48)
    assert names["l1.mix.dkv.norm"] == (24,) and names["l1.mix.uv"] == (60, 24)
    assert names["l1.mlp.router"] == (8, 48) and names["l1.mlp.correction"] == (8,)
    assert "l1.mlp.e4.down" in names and "l1.mlp.e5.gate" not in names
    assert names["l0.norm1b"] == names["l0.norm2b"] == (48,)
    # no feed-forward, neither of its norms
    assert not any(n.startswith(("l2.mlp", "l2.norm2")) for n in names) and "l2.norm1b" in names
    assert [r.layer for r in spec.runs()] == [0, 1, 2, 3, 1, 2, 3, 1, 2, 3, 4]
    assert [i for i, r in enumerate(spec.runs()) if r.junction is not None] == [1, 4, 7]
    assert "loop.in" not in {t.name for t in pm.spec_of(pm.CONFIG_B).tensor_specs()}


_DROP = object()


def _edit(path, value):
    def apply(cfg):
        node = cfg
        for key in path[:-1]:
            node = node[key]
        if value is _DROP:
            del node[path[-1]]
        else:
            node[path[-1]] = value
    return apply


@pytest.mark.parametrize("edit, message", [
    (_edit(("layers", 0, "type"), "delta"), "type 'delta'"),
    (_edit(("layers", 0, "mixer", "kv_heads"), 3), "'kv_heads'"),
    (_edit(("layers", 0, "mixer", "rot", "dims"), 7), "'dims' 7"),
    (_edit(("layers", 0, "mixer", "rot", "dims"), 18), "'dims' 18"),
    (_edit(("layers", 0, "mixer", "rot", "scaling"), {"factor": 2.0}), "'scaling'"),
    (_edit(("layers", 0, "mixer", "mask", "size"), 0), "'size'"),
    (_edit(("layers", 0, "mixer", "scale"), _DROP), "'scale'"),
    (_edit(("layers", 1, "mixer", "q_rank"), _DROP), "'q_rank'"),
    (_edit(("layers", 1, "mixer", "kv_rank"), 0), "'kv_rank'"),
    (_edit(("layers", 1, "mixer", "rot", "scaling", "factor"), 0.0), "'factor'"),
    (_edit(("layers", 1, "mlp", "router", "top"), 9), "'top' 9"),
    (_edit(("layers", 1, "mlp", "router", "identity"), -1), "'identity' -1"),
    (_edit(("layers", 0, "mlp", "kind"), "sparse"), "kind 'sparse'"),
    (_edit(("loop", "stop"), 6), "'stop' 6"),
    (_edit(("loop", "start"), 4), "'start' 4"),
    (_edit(("loop", "times"), 0), "'times'"),
    (_edit(("norm", "eps"), 0.0), "'eps'"),
    (_edit(("width",), _DROP), "'width'"),
])
def test_config_errors_name_the_key(edit, message):
    from rust_llm_inference_server_amd.registry import architecture_of
    cfg = copy.deepcopy(pm.CONFIG_A)
    edit(cfg)
    with pytest.raises(ConfigError) as e:
        architecture_of(cfg).parse_config(cfg)
    assert message in str(e.value)


def test_stretched_frequencies_cover_all_three_ranges():
    """The rotation part's tables against the plain angles, for a stretching under which some
    frequencies are kept, some divided and some blended."""
    from rust_llm_inference_server_amd.parts.base import BuildContext, PartSpec, create
    seen = set()
    for cfg in (pm.CONFIG_A, pm.CONFIG_B, pm.CONFIG_D):
        for layer in cfg["layers"]:
            rot = layer["mixer"].get("rot") or {}
            s = rot.get("scaling")
            if not s:
                continue
            share = (plain.yarn_frequencies(rot["dims"], rot["base"], s, torch.float64)
                     / plain.plain_frequencies(rot["dims"], rot["base"], torch.float64))
            seen |= {"kept" if f > 1 - 1e-12 else "divided" if f < 1 / s["factor"] + 1e-12
                     else "blended" for f in share.tolist()}
            ctx = BuildContext(device=torch.device("cpu"), act_dtype=torch.float32, weights={},
                               max_positions=500)
            part = create("position", PartSpec("rope", {
                "rot_dim": rot["dims"], "theta": rot["base"], "precise": True, "interleaved": True,
                "scaling": {"rope_type": "yarn", **s}}), "", ctx)
            cos, sin = plain.angles(500, rot, torch.float64)
            assert float((part.cos.double() - cos).abs().max()) < 2e-7
            assert float((part.sin.double() - sin).abs().max()) < 2e-7
    assert seen == {"kept", "divided", "blended"}


def test_the_plain_implementation_does_not_look_ahead():
    """A position's plain logits depend on the tokens up to it and on nothing behind it; and they
    do depend on a token far back."""
    cfg = pm.CONFIG_A
    stored = pm.as_stored(pm.make_weights(cfg, 5), torch.float32)
    tokens = pm.prompts(cfg["vocab"], [60], seed=1)[0]
    whole = pm.plain_logits(plain, cfg, stored, tokens)
    part = pm.plain_logits(plain, cfg, stored, tokens[:41])
    assert float((whole[:41] - part).abs().max()) < 1e-9
    other = list(tokens)
    other[3] = (other[3] + 1) % cfg["vocab"]
    assert float((pm.plain_logits(plain, cfg, stored, other)[-1] - whole[-1]).abs().max()) > 1e-6


# Other readings of a mechanism, each planted in the plain implementation.
def _no_identity(h, mlp, w, pre):
    gone = dict(mlp, router=dict(mlp["router"]))
    chosen, weights = plain.choose(h @ w[pre + "router"].T, w[pre + "correction"], gone["router"]["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, wt in zip(chosen[t].tolist(), weights[t].tolist()):
            if e < gone["router"]["experts"]:
                out[t] = out[t] + wt * plain.gated_unit(h[t], w, f"{pre}e{e}.")
    return out


def _chosen_on_scores(z, correction, top):
    s = torch.softmax(z, -1)
    chosen = torch.topk(s, top, dim=-1).indices
    return chosen, torch.gather(s, 1, chosen)


def _weights_with_correction(z, correction, top):
    s = torch.softmax(z, -1) + correction
    chosen = torch.topk(s, top, dim=-1).indices
    return chosen, torch.gather(s, 1, chosen)


def _first_pass_without_rejoin(config):
    order = _ORDER(config)
    first = next(i for i, (_, enters) in enumerate(order) if enters)
    return [(layer, enters and i != first) for i, (layer, enters) in enumerate(order)]


def _rejoin_at_every_layer(config):
    a, b = config["loop"]["start"], config["loop"]["stop"]
    return [(layer, a <= layer < b) for layer, _ in _ORDER(config)]


def _one_pass_fewer(config):
    fewer = dict(config, loop=dict(config["loop"], times=config["loop"]["times"] - 1))
    return _ORDER(fewer)


_ORDER = plain.run_order


def _halves_of_pairs(x, rot):
    c, s = (t.unsqueeze(1) for t in plain.angles(x.shape[0], rot, x.dtype))
    half = rot["dims"] // 2
    u, v = x[..., :half], x[..., half:rot["dims"]]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., rot["dims"]:]], -1)


def _bare_angles(n, rot, dtype):
    f = plain.plain_frequencies(rot["dims"], rot["base"], dtype)
    a = torch.arange(n, dtype=dtype).reshape(n, 1) * f
    return torch.cos(a), torch.sin(a)


_ANGLES = plain.angles


def _unscaled_angles(n, rot, dtype):
    cos, sin = _ANGLES(n, rot, dtype)
    m = (cos * cos + sin * sin).sqrt()
    return cos / m, sin / m


@pytest.mark.parametrize("name, other", [
    ("mixture", _no_identity), ("choose", _chosen_on_scores), ("choose", _weights_with_correction),
    ("run_order", _first_pass_without_rejoin), ("run_order", _rejoin_at_every_layer),
    ("run_order", _one_pass_fewer),
    ("rejoin", lambda x, x0, w: torch.cat([x0, x], -1) @ w.T),
    ("rejoin", lambda x, x0, w: torch.cat([x, x], -1) @ w.T),
    ("rotate_neighbours", _halves_of_pairs), ("angles", _bare_angles),
    ("angles", _unscaled_angles)])
def test_other_readings_move_the_plain_rows(name, other, monkeypatch):
    """What the engine is held against depends on each of these.  (Chosen weights divided by their
    sum are not among them: the norm behind the sublayer takes a common factor out again.)"""
    cfg = pm.CONFIG_A
    stored = pm.as_stored(pm.make_weights(cfg, 7), torch.float32)
    tokens = pm.prompts(cfg["vocab"], [40], seed=8)[0]
    a = pm.plain_logits(plain, cfg, stored, tokens)
    monkeypatch.setattr(plain, name, other)
    b = pm.plain_logits(plain, cfg, stored, tokens)
    assert max(pm.row_error(x, y) for x, y in zip(a, b)) > 1e-2


def test_the_junction_alone(backend, dtype):
    """The stream becomes one map of itself and of the embedding output, in float32, whatever is
    pending on it; the embedding output is the step's, not the stream's."""
    from rust_llm_inference_server_amd.parts.base import (BuildContext, PartSpec, ResidualStream,
                                                          create)
    act = torch.float32 if dtype == "float32" else torch.bfloat16
    W = 72
    g = torch.Generator().manual_seed(3)
    w = (torch.randn((W, 2 * W), generator=g) * W ** -0.5).to(act)
    x0 = torch.randn((9, W), generator=g).to(act).float()
    delta = torch.randn((9, W), generator=g).to(act)
    ctx = BuildContext(device=backend, act_dtype=act, weights={"loop.in": w.to(backend)},
                       max_positions=16)
    part = create("junction", PartSpec("embedding_rejoin", {"hidden_size": W}), "loop.in", ctx)
    stream = ResidualStream(x0.to(backend).clone(), act)
    kept = part.begin(stream)
    want, x = x0.double(), x0.double()
    for _ in range(3):
        stream.add(delta.to(backend))
        part.forward(stream, kept)
        want = plain.rejoin(want + delta.double(), x0.double(), w.double())
    got = stream.flush().double().cpu()
    tol = 1e-5 if dtype == "float32" else 2e-2
    assert float((got - want).norm() / want.norm()) < tol


# --------------------------------------------------------------------- the step function
@pytest.mark.parametrize("name", ["a", "b", "c", "e"])
def test_whole_prompts_and_first_tokens(backend, dtype, name, tmp_path_factory):
    folder, cfg, stored = model_case(name, dtype, tmp_path_factory)
    lengths = [1, 2, 3, 45] if backend.type == "cpu" else [1, 2, 3, 19, 70]
    reqs = traces.random_requests(cfg["vocab"], lengths, seed=11)
    steps, _ = traces.trace_whole(reqs)
    check_trace(runner_for(folder, backend, dtype), steps, reqs, cfg, stored, dtype)


@pytest.mark.parametrize("name", ["a", "b", "c", "e"])
def test_decoding_token_by_token_equals_the_prompt_pass(backend, dtype, name, tmp_path_factory):
    """One request decoded from its first token on, one after a prompt, so that windows pass over
    decoded tokens; single tokens go through captured steps on the GPU."""
    folder, cfg, stored = model_case(name, dtype, tmp_path_factory)
    lengths, tail = ([20, 45], 19) if backend.type == "cpu" else ([45, 80], 44)
    reqs = traces.random_requests(cfg["vocab"], lengths, seed=12)
    ids = list(reqs)
    steps, _ = traces.trace_tail({ids[0]: reqs[ids[0]]}, tail=tail)
    more, _ = traces.trace_tail({ids[1]: reqs[ids[1]]}, tail=tail + 1)
    for s in more:
        s["step"] += len(steps)
    check_trace(runner_for(folder, backend, dtype), steps + more, reqs, cfg, stored, dtype)


@pytest.mark.parametrize("name", ["a", "b", "c", "e"])
def test_portions_of_any_size(backend, dtype, name, tmp_path_factory):
    """Portions of 7, 2, 16, 3, 24, 2, 33, ... tokens: portions that end inside a page and inside a
    window."""
    folder, cfg, stored = model_case(name, dtype, tmp_path_factory)
    lengths = [60] if backend.type == "cpu" else [90, 37]
    reqs = traces.random_requests(cfg["vocab"], lengths, seed=13)
    steps, _ = traces.trace_portions(reqs)
    check_trace(runner_for(folder, backend, dtype), steps, reqs, cfg, stored, dtype)


@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_mixed_batches_reuse_pages_and_slots(backend, dtype, name, tmp_path_factory):
    """Seven unequal requests through three slots and a pool that holds three of them: portions
    beside single tokens, requests left out of steps, pages of finished requests taken by later
    ones with their old contents still there, in every pass's cache."""
    if backend.type == "cpu" and name == "b":
        pytest.skip("two of them on the double")
    folder, cfg, stored = model_case(name, dtype, tmp_path_factory)
    lengths = [20, 9, 35, 2, 17] if backend.type == "cpu" else [50, 9, 75, 33, 2, 64, 21]
    reqs = traces.random_requests(cfg["vocab"], lengths, seed=14)
    steps, peak = traces.trace_mixed(reqs, live=3, seed=5)
    runner = runner_for(folder, backend, dtype, num_pages=-(-peak // 16), max_num_seqs=3)
    check_trace(runner, steps, reqs, cfg, stored, dtype)
    assert runner.cache.num_free_pages() == -(-peak // 16)


def test_a_request_alone_equals_itself_in_a_batch(backend, dtype, tmp_path_factory):
    """The rows of a request do not depend on what else the step holds (beyond rounding)."""
    folder, cfg, stored = model_case("a", dtype, tmp_path_factory)
    lengths = [14, 9, 21] if backend.type == "cpu" else [40, 23, 31]
    reqs = traces.random_requests(cfg["vocab"], lengths, seed=15)
    alone = {}
    for rid, tokens in reqs.items():
        steps, _ = traces.trace_portions({rid: tokens})
        out = traces.replay_in_process(runner_for(folder, backend, dtype), steps)
        alone[rid] = traces.collect(steps, out, cfg["vocab"])[rid]
    steps, _ = traces.trace_mixed(reqs, live=3, seed=2)
    out = traces.replay_in_process(runner_for(folder, backend, dtype), steps)
    together = traces.collect(steps, out, cfg["vocab"])
    pm.judge([pm.row_error(row, alone[rid][pos]) for rid in reqs
              for pos, row in together[rid].items()], dtype)


@pytest.mark.gpu
@pytest.mark.parametrize("live", [8, 40])
def test_decode_steps_of_many_requests(backend, dtype, live, tmp_path_factory):
    """Decode batches beyond the small ones' kernels: every row against its plain logits."""
    if backend.type == "cpu":
        pytest.skip("the kernels' business")
    folder, cfg, stored = model_case("d", dtype, tmp_path_factory)
    g = torch.Generator().manual_seed(live)
    lengths = torch.randint(3, 60, (live,), generator=g).tolist()
    reqs = traces.random_requests(cfg["vocab"], lengths, seed=33)
    steps = [{"step": 0, "end": [], "entries": [
        {"id": r, "tokens": t[:-2], "want": list(range(len(t) - 2))} for r, t in reqs.items()]}]
    for i in (2, 1):
        steps.append({"step": 3 - i, "end": [], "entries": [
            {"id": r, "tokens": [t[-i]], "want": [0]} for r, t in reqs.items()]})
    steps[-1]["end"] = list(reqs)
    check_trace(runner_for(folder, backend, dtype, num_pages=5 * live, max_num_seqs=live), steps,
                reqs, cfg, stored, dtype)


def test_long_prompts_and_long_decoding(backend, dtype, tmp_path_factory):
    """A prompt of hundreds of tokens in one step, then hundreds of single-token steps: windows
    pass and give their pages back."""
    folder, cfg, stored = model_case("a", dtype, tmp_path_factory)
    n, tail = (70, 25) if backend.type == "cpu" else (390, 150)
    reqs = traces.random_requests(cfg["vocab"], [n], seed=16)
    steps, _ = traces.trace_tail(reqs, tail=tail)
    check_trace(runner_for(folder, backend, dtype), steps, reqs, cfg, stored, dtype)


def test_prompts_of_hundreds_of_tokens_at_head_sizes_of_real_models(backend, dtype,
                                                                    tmp_path_factory):
    """Heads of 64 and 128: whole prompts of up to 700 tokens in one step, the same prompts with
    their ends decoded, and in portions beside each other; a long portion beside single tokens of
    others."""
    folder, cfg, stored = model_case("d", dtype, tmp_path_factory)
    lengths = [60] if backend.type == "cpu" else [700, 300, 130, 257]
    reqs = traces.random_requests(cfg["vocab"], lengths, seed=71)
    make = lambda: runner_for(folder, backend, dtype, num_pages=130, max_positions=2048)
    steps, _ = traces.trace_whole(reqs)
    check_trace(make(), steps, reqs, cfg, stored, dtype)
    if backend.type == "cpu":
        return              # the rest is the kernels' business
    steps, _ = traces.trace_tail(reqs, tail=20)
    check_trace(make(), steps, reqs, cfg, stored, dtype)
    steps, peak = traces.trace_mixed(reqs, live=3, seed=6)
    check_trace(runner_for(folder, backend, dtype, num_pages=-(-peak // 16), max_num_seqs=3,
                           max_positions=2048), steps, reqs, cfg, stored, dtype)
    reqs = traces.random_requests(cfg["vocab"], [60, 70, 330], seed=72)
    cuts = [{"r0": (0, 40), "r1": (0, 50)}, {"r0": (40, 41), "r1": (50, 51), "r2": (0, 300)},
            {"r0": (41, 60), "r1": (51, 70), "r2": (300, 330)}]
    steps = [{"step": i, "end": [], "entries": [
        {"id": rid, "tokens": reqs[rid][lo:hi], "want": list(range(hi - lo))}
        for rid, (lo, hi) in cut.items()]} for i, cut in enumerate(cuts)]
    steps[-1]["end"] = ["r0", "r1", "r2"]
    check_trace(make(), steps, reqs, cfg, stored, dtype)


# ------------------------------------------------------------- tokens made to stand out
KEY_TOKEN, QUERY_TOKEN, FILL_TOKEN = 5, 9, 1


def _marked(cfg, seed):
    """Weights in which, all through the layers and passes, coordinate 0 of the stream is nonzero at
    ``KEY_TOKEN`` only and coordinate 1 at ``QUERY_TOKEN`` only: the embedding sets them, the norms
    behind the sublayers let nothing through to them, the loop's map takes half of each from the
    stream and half from the embedding output, and the final norm's weight hides them."""
    w = pm.make_weights(cfg, seed=seed)
    w["embed"][:, :2] = 0.0
    w["embed"][KEY_TOKEN, 0] = 3.0
    w["embed"][QUERY_TOKEN, 1] = 3.0
    W = cfg["width"]
    for name in w:
        if name.endswith((".norm1b", ".norm2b")) or name == "final.norm":
            w[name][:2] = 0.0
        elif name.endswith(".norm1"):
            w[name][:2] = 1.0
    if "loop.in" in w:
        w["loop.in"][:2] = 0.0
        for c in range(2):
            w["loop.in"][c, c] = w["loop.in"][c, W + c] = 0.5
    return w


def _stands_out(cfg, w, layer):
    """In every head of ``layer``'s mixer the key of ``KEY_TOKEN`` gets a score far above the others'
    from a query of ``QUERY_TOKEN``.  Windowed layers: one channel of every key head reads stream
    coordinate 0, the same channel of every query head coordinate 1 (a channel that is not
    rotated, or else one of the slowest pair, whose other one is emptied).  Latent layers: channel
    0 of the queries' latent reads coordinate 1, channel 0 of the other coordinate 0, and channel
    0 of every head's unrotated query and key reads channel 0 of its latent."""
    m, p = cfg["layers"][layer]["mixer"], f"l{layer}.mix"
    if cfg["layers"][layer]["type"] == "attention":
        d, dims = m["dim"], (m.get("rot") or {}).get("dims", 0)
        chans = [dims] if dims < d else [dims // 2 - 1, dims - 1]
        for name, heads, coordinate in (("q", m["heads"], 1), ("k", m["kv_heads"], 0)):
            for head in range(heads):
                for n, c in enumerate(chans):
                    w[f"{p}.{name}"][head * d + c] = 0.0
                w[f"{p}.{name}"][head * d + chans[0], coordinate] = 12.0
        m["scale"] = 10.0 / d
        return w
    d, q_head = m["dim"], m["dim"] + m["rot_dim"]
    for name, coordinate in (("dq", 1), ("dkv", 0)):
        w[f"{p}.{name}"][0] = 0.0
        w[f"{p}.{name}"][0, coordinate] = 12.0
        w[f"{p}.{name}.norm"][0] = 1.0
    gain = (12.0 / (m["scale"] * (m["q_rank"] * m["kv_rank"]) ** 0.5)) ** 0.5
    for name, size in (("uq", q_head), ("uk", d)):
        for head in range(m["heads"]):
            w[f"{p}.{name}"][head * size] = 0.0
            w[f"{p}.{name}"][head * size, 0] = gain
    return w


def _tokens(vocab, n, seed):
    return [t if t not in (KEY_TOKEN, QUERY_TOKEN) else FILL_TOKEN
            for t in pm.prompts(vocab, [n], seed=seed)[0]]


@pytest.mark.parametrize("layer, back", [(0, 0), (0, 1), (2, 0), (2, 1), (3, 0), (3, 1)])
def test_keys_just_inside_and_outside_a_window(backend, dtype, layer, back, tmp_path_factory,
                                               monkeypatch):
    """Windows of 20 and, in layers that run three times, of 16 (a page) and 33 positions.  A key
    that stands out is the last one a query sees, or one further back.  A window that is one
    token off, in a prompt's portion or decoded alone, moves the row far."""
    if backend.type == "cpu" and (layer, back) not in ((0, 0), (2, 1)):
        pytest.skip("the double takes its time: one of either side here, all on the GPU")
    cfg = copy.deepcopy(pm.CONFIG_A)
    size = cfg["layers"][layer]["mixer"]["mask"]["size"]
    w = _stands_out(cfg, _marked(cfg, seed=31 + layer), layer)
    folder, _, stored = model_case("a", dtype, tmp_path_factory, weights=w, tag=f"edge{layer}",
                                   config=cfg)
    n = 3 * size
    tokens = _tokens(cfg["vocab"], n, seed=32)
    queries = (size + size // 3, n - 3)
    for query in queries:
        tokens[query] = QUERY_TOKEN
        tokens[query - size + 1 - back] = KEY_TOKEN
    a = pm.plain_logits(plain, cfg, stored, tokens)
    visible = plain.visible
    monkeypatch.setattr(plain, "visible", lambda n, s: visible(
        n, s if s != size else s - 1 if back == 0 else s + 1))
    b = pm.plain_logits(plain, cfg, stored, tokens)
    monkeypatch.setattr(plain, "visible", visible)
    for query in queries:
        assert pm.row_error(a[query], b[query]) > 0.1
    reqs = {"r": tokens}
    steps, _ = traces.trace_tail(reqs, tail=size // 2)
    check_trace(runner_for(folder, backend, dtype), steps, reqs, cfg, stored, dtype)
    steps, _ = traces.trace_portions(reqs)
    check_trace(runner_for(folder, backend, dtype), steps, reqs, cfg, stored, dtype)


@pytest.mark.parametrize("layer, far", [(1, 0), (1, 15), (1, 16), (1, 48), (4, 0), (4, 31)])
def test_a_far_key_that_stands_out(backend, dtype, layer, far, tmp_path_factory, monkeypatch):
    """Latent layers, one of which runs three times, over pages of 16: the token at ``far`` (a
    page's first or last position among them) takes most of the weight of queries 100 and more
    positions on, in a prompt's portion and decoded alone."""
    if backend.type == "cpu" and (layer, far) not in ((1, 15), (4, 0)):
        pytest.skip("the double takes its time: one of either layer here, all on the GPU")
    cfg = copy.deepcopy(pm.CONFIG_A)
    w = _stands_out(cfg, _marked(cfg, seed=41 + layer), layer)
    folder, _, stored = model_case("a", dtype, tmp_path_factory, weights=w, tag=f"far{layer}",
                                   config=cfg)
    n, on = (70, 40) if backend.type == "cpu" else (180, 100)
    tokens = _tokens(cfg["vocab"], n, seed=42)
    tokens[far] = KEY_TOKEN
    tokens[far + on] = tokens[n - 4] = QUERY_TOKEN
    a = pm.plain_logits(plain, cfg, stored, tokens)
    attend = plain.attend
    monkeypatch.setattr(plain, "attend", lambda scores, ok, v: attend(
        scores, ok & ((torch.arange(n) != far) | torch.eye(n, dtype=torch.bool)), v))
    b = pm.plain_logits(plain, cfg, stored, tokens)
    monkeypatch.setattr(plain, "attend", attend)
    for query in (far + on, n - 4):
        assert pm.row_error(a[query], b[query]) > 0.1
    reqs = {"r": tokens}
    steps, _ = traces.trace_tail(reqs, tail=8)
    check_trace(runner_for(folder, backend, dtype), steps, reqs, cfg, stored, dtype)
    steps, _ = traces.trace_portions(reqs)
    check_trace(runner_for(folder, backend, dtype), steps, reqs, cfg, stored, dtype)


# -------------------------------------------------------------------- engine and scheduler
@pytest.mark.parametrize("seats, budget", [(3, 16), (4, 64)])
def test_greedy_generation_through_the_engine(backend, dtype, seats, budget, tmp_path_factory):
    """Five requests through three or four seats with a token budget that cuts the prompts: every
    generated token is the plain implementation's pick, up to a near-tie of its logits (bfloat16:
    or, seldom, up to a router's near-tie, after which the plain implementation goes on with the
    engine's token)."""
    from rust_llm_inference_server_amd.engine import Engine, load_model
    if backend.type == "cpu" and seats == 4:
        pytest.skip("one of them on the double")
    folder, cfg, stored = model_case("a", dtype, tmp_path_factory)
    model = load_model(folder, dtype, 256, backend)
    engine = Engine(model, EngineConfig(max_num_seqs=seats, max_batched_tokens=budget,
                                        num_pages=48, block_size=8, max_seq_len=256,
                                        watermark_pages=1))
    lengths, new = ([5, 13, 1], 4) if backend.type == "cpu" else ([5, 21, 1, 34, 12], 7)
    prompts = pm.prompts(cfg["vocab"], lengths, seed=18)
    outs = engine.generate(prompts, SamplingParams.greedy(new))
    margin = 1e-3 if dtype == "float32" else 0.5
    off = 0
    for p, o in zip(prompts, outs):
        assert o.finish_reason == "length" and len(o.token_ids) == new
        tokens = list(p)
        for got in o.token_ids:
            last = pm.plain_logits(plain, cfg, stored, tokens)[-1]
            off += int(float(last.max() - last[got]) >= margin)
            tokens.append(got)
    assert off <= (0 if dtype == "float32" else 2)
    engine.runner.cache.check_invariants()


def test_a_fork_goes_on_from_every_pass(backend, dtype, tmp_path_factory):
    """A request forked inside a page goes on with its parent's cache of every pass, and neither
    disturbs the other."""
    from rust_llm_inference_server_amd.engine import StepEntry
    folder, cfg, stored = model_case("a", dtype, tmp_path_factory)
    runner = runner_for(folder, backend, dtype)
    tokens = pm.prompts(cfg["vocab"], [40], seed=27)[0]
    runner.reserve(1, 25)
    runner.step([StepEntry(1, tokens[:25], [])])
    runner.fork(1, 2)
    other = [(t + 3) % cfg["vocab"] for t in tokens[25:33]]
    errors = []
    for seq, rest in ((1, tokens[25:33]), (2, other)):
        runner.reserve(seq, 33)
        got = runner.step([StepEntry(seq, rest, list(range(8)))]).float().cpu()
        want = pm.plain_logits(plain, cfg, stored, tokens[:25] + rest)[25:]
        errors += [pm.row_error(x, y) for x, y in zip(got, want)]
    pm.judge(errors, dtype)


@pytest.mark.gpu
@pytest.mark.parametrize("name, dtype_name", [("a", "float32"), ("a", "bfloat16"),
                                              ("c", "bfloat16")])
def test_the_replay_program_runs_the_model(name, dtype_name, tmp_path_factory, tmp_path):
    folder, cfg, stored = model_case(name, dtype_name, tmp_path_factory)
    reqs = traces.random_requests(cfg["vocab"], [40, 7, 25, 33, 18], seed=19)
    steps, peak = traces.trace_mixed(reqs, live=4, seed=3)
    out = traces.replay_program(folder, dtype_name, steps, peak, str(tmp_path / "out"),
                                cfg["vocab"])
    got = traces.collect(steps, out, cfg["vocab"])
    errors = []
    for rid, tokens in reqs.items():
        want = pm.plain_logits(plain, cfg, stored, tokens)
        errors += [pm.row_error(row, want[pos]) for pos, row in got[rid].items()]
    pm.judge(errors, dtype_name)


@pytest.mark.gpu
def test_the_command_line_generates_and_scores(tmp_path_factory, tmp_path, capsys):
    """``rlis generate`` picks the design by config.json and prints the plain implementation's
    greedy tokens; ``rlis perplexity`` scores a token file through the same step function."""
    from rust_llm_inference_server_amd import cli
    folder, cfg, stored = model_case("c", "float32", tmp_path_factory)
    prompt = pm.prompts(cfg["vocab"], [11], seed=20)[0]
    rc = cli.main(["generate", "--model", folder, "--dtype", "f32", "--max-seq-len", "128",
                   "--num-pages", "32", "--block-size", "8", "--max-num-seqs", "2",
                   "--max-tokens", "5", "--prompt-ids", ",".join(map(str, prompt))])
    out = capsys.readouterr()
    assert rc == 0
    got = [int(t) for t in out.out.split()]
    tokens = list(prompt)
    for g in got:
        last = pm.plain_logits(plain, cfg, stored, tokens)[-1]
        assert float(last.max() - last[g]) < 1e-3
        tokens.append(g)
    assert len(got) == 5 and "output 5 tok (length)" in out.err
    ids = tmp_path / "ids.txt"
    ids.write_text(" ".join(map(str, pm.prompts(cfg["vocab"], [96], seed=21)[0])))
    rc = cli.main(["perplexity", "--model", folder, "--dtype", "f32", "--max-seq-len", "128",
                   "--ids-file", str(ids), "--ctx", "32"])
    out = capsys.readouterr()
    assert rc == 0 and json.loads(out.out.strip().splitlines()[-1])["ppl"] > 1.0
