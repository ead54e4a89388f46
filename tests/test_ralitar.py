"""The Ralitar decoder in the engine against the plain implementation (``plain_ralitar.py``):
whole prompts, token-by-token decoding, portions down to two tokens, batches of unequal
requests with pages and state slots used again, long decoding, keys made to stand out far away,
at page borders, just inside and just outside a chunk, a far token in either recurrent state,
the first tokens of a sequence, and greedy generation through the engine's scheduler.  Every case
runs on the GPU (``-m gpu``, float32 and bfloat16) and, with the kernels replaced by the slow
torch double, on the CPU, where it tests the host logic: the state slots, the previous token that
a portion starts behind, the residual stream's pending norms, the step layout."""
import copy
import json

import pytest
import torch

import plain_ralitar as plain
import ralitar_models as rm
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
    """(folder, config, the stored numbers in float64) of a configuration; made once.  The folder's
    config.json leaves the low-rank projections' ranks to the tensors' shapes."""
    key = (name, dtype, tag)
    if key not in _CACHE:
        cfg = config if config is not None else rm.CONFIGS[name]
        w = weights if weights is not None else rm.make_weights(cfg, seed=len(name) + 23)
        store = torch.float32 if dtype == "float32" else torch.bfloat16
        written = copy.deepcopy(cfg)
        for layer in written["layers"]:
            for rank in ("decay_rank", "gate_rank"):
                layer["mixer"].pop(rank, None)
        folder = rm.write_folder(tmp_path_factory.mktemp(f"ralitar_{name}_{dtype}{tag}"), written,
                                 w, store)
        _CACHE[key] = (folder, cfg, rm.as_stored(w, store))
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
        want = rm.plain_logits(plain, cfg, stored, tokens)
        assert sorted(got[rid]) == list(range(len(tokens)))
        errors += [rm.row_error(row, want[pos]) for pos, row in got[rid].items()]
    rm.judge(errors, dtype)


# ----------------------------------------------------------------------- configuration
def test_config_round_trip_and_the_specification():
    from rust_llm_inference_server_amd.registry import architecture_of
    for cfg in rm.CONFIGS.values():
        arch = architecture_of(cfg)
        assert arch.name == "Ralitar"
        assert arch.config_to_dict(arch.parse_config(cfg)) == cfg
    spec = rm.spec_of(rm.CONFIG_A)
    names = {t.name: tuple(t.shape) for t in spec.tensor_specs()}
    assert names["embed"] == (97, 48) and names["bigram"] == (54, 48)
    assert names["side.embed"] == (97, 7 * 8) and names["head"] == (97, 48)
    assert names["l0.mix.k"] == (32, 48) and names["l0.mix.v.conv"] == (96, 4)
    assert names["l0.mix.a2"] == (64, 6) and names["l0.mix.g2"] == (96, 10)
    assert names["l1.mix.q.norm"] == (64,) and names["l1.mix.k.b"] == (32,)
    assert names["l1.mix.g"] == (64, 48) and "l1.mix.v" not in names
    assert names["l2.mix.ra"] == (3, 20, 20) and names["l2.mix.ri.b"] == (3, 20)
    # no feed-forward, no second norm; the token input and its norm are there all the same
    assert not any(n.startswith(("l2.mlp", "l2.norm2")) for n in names)
    assert names["l2.side.gate"] == (8, 48) and names["l2.side.norm"] == (48,)
    other = {t.name for t in rm.spec_of(rm.CONFIG_B).tensor_specs()}
    assert "bigram" not in other and not any("side" in n for n in other)


def test_ranks_come_from_the_tensors():
    from rust_llm_inference_server_amd.registry import architecture_of
    cfg = copy.deepcopy(rm.CONFIG_A)
    for layer in cfg["layers"]:
        layer["mixer"].pop("decay_rank", None)
        layer["mixer"].pop("gate_rank", None)
    arch = architecture_of(cfg)
    parsed = arch.parse_config(cfg)
    with pytest.raises(ConfigError, match="ranks"):
        arch.build_spec(parsed)
    shapes = {"l0.mix.a1": (6, 48), "l0.mix.g1": (10, 48), "l4.mix.a1": (9, 48),
              "l4.mix.g1": (5, 48)}
    assert arch.config_to_dict(arch.complete_config(parsed, shapes)) == rm.CONFIG_A


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
    (_edit(("layers", 0, "mixer", "conv"), 0), "'conv'"),
    (_edit(("layers", 1, "mixer", "kv_heads"), 3), "'kv_heads'"),
    (_edit(("layers", 1, "mixer", "vdim"), 8), "'vdim' 8"),
    (_edit(("layers", 1, "mixer", "rot", "dims"), 7), "'dims' 7"),
    (_edit(("layers", 1, "mixer", "rot", "dims"), 18), "'dims' 18"),
    (_edit(("layers", 1, "mixer", "rot", "scaling", "factor"), 0.0), "'factor'"),
    (_edit(("layers", 1, "mixer", "scale"), _DROP), "'scale'"),
    (_edit(("layers", 1, "mixer", "mask", "size"), 0), "'size'"),
    (_edit(("layers", 1, "mixer", "softcap"), -1.0), "'softcap'"),
    (_edit(("layers", 2, "mixer", "blocks"), 7), "'blocks'"),
    (_edit(("layers", 0, "mlp", "kind"), "moe"), "kind 'moe'"),
    (_edit(("embedding", "bigram", "buckets"), 0), "'buckets'"),
    (_edit(("embedding", "bigram", "mul_prev"), 1 << 31), "'mul_prev'"),
    (_edit(("token_side", "dim"), 0), "'dim'"),
    (_edit(("norm", "eps"), 0.0), "'eps'"),
    (_edit(("width",), _DROP), "'width'"),
])
def test_config_errors_name_the_key(edit, message):
    from rust_llm_inference_server_amd.registry import architecture_of
    cfg = copy.deepcopy(rm.CONFIG_A)
    edit(cfg)
    with pytest.raises(ConfigError) as e:
        architecture_of(cfg).parse_config(cfg)
    assert message in str(e.value)


def test_stretched_frequencies_cover_all_three_ranges():
    """The rotation part's tables against the plain frequencies, for a scaling under which some
    frequencies are kept, some divided and some blended."""
    from rust_llm_inference_server_amd.parts.base import BuildContext, PartSpec, create
    rot = rm.CONFIG_A["layers"][1]["mixer"]["rot"]
    f = plain.frequencies(rot)
    bare = plain.frequencies({"dims": rot["dims"], "base": rot["base"]})
    share = f / bare
    assert float(share[0]) == 1.0 and abs(float(share[-1]) - 0.25) < 1e-12
    assert any(0.26 < float(s) < 0.99 for s in share)
    s = rot["scaling"]
    ctx = BuildContext(device=torch.device("cpu"), act_dtype=torch.float32, weights={},
                       max_positions=700)
    part = create("position", PartSpec("rope", {
        "rot_dim": rot["dims"], "theta": rot["base"], "precise": True, "interleaved": True,
        "scaling": {"rope_type": "llama3", "factor": s["factor"], "low_freq_factor": s["low"],
                    "high_freq_factor": s["high"],
                    "original_max_position_embeddings": s["original"]}}), "", ctx)
    ang = torch.arange(700, dtype=torch.float64).reshape(-1, 1) * f.reshape(1, -1)
    assert float((part.cos.double() - torch.cos(ang)).abs().max()) < 1e-7
    assert float((part.sin.double() - torch.sin(ang)).abs().max()) < 1e-7
    assert part.interleaved


def test_the_plain_implementation_does_not_look_ahead():
    """A position's plain logits depend on the tokens up to it and on nothing behind it; and
    they do depend on a token far back (through the recurrent states)."""
    cfg = rm.CONFIG_A
    stored = rm.as_stored(rm.make_weights(cfg, 5), torch.float32)
    tokens = rm.prompts(cfg["vocab"], [60], seed=1)[0]
    whole = rm.plain_logits(plain, cfg, stored, tokens)
    part = rm.plain_logits(plain, cfg, stored, tokens[:41])
    assert float((whole[:41] - part).abs().max()) < 1e-9
    other = list(tokens)
    other[3] = (other[3] + 1) % cfg["vocab"]
    assert float((rm.plain_logits(plain, cfg, stored, other)[-1] - whole[-1]).abs().max()) > 1e-6


# --------------------------------------------------------------------- the step function
@pytest.mark.parametrize("name", ["a", "b", "c", "e"])
def test_whole_prompts_and_first_tokens(backend, dtype, name, tmp_path_factory):
    folder, cfg, stored = model_case(name, dtype, tmp_path_factory)
    reqs = traces.random_requests(cfg["vocab"], [1, 2, 3, 19, 70], seed=11)
    steps, _ = traces.trace_whole(reqs)
    check_trace(runner_for(folder, backend, dtype), steps, reqs, cfg, stored, dtype)


@pytest.mark.parametrize("name", ["a", "b", "c", "e"])
def test_decoding_token_by_token_equals_the_prompt_pass(backend, dtype, name, tmp_path_factory):
    """One request decoded from its first token on, one after a prompt, so that chunks begin
    inside decoded tokens; single tokens go through captured steps on the GPU."""
    folder, cfg, stored = model_case(name, dtype, tmp_path_factory)
    reqs = traces.random_requests(cfg["vocab"], [45, 80], seed=12)
    ids = list(reqs)
    steps, _ = traces.trace_tail({ids[0]: reqs[ids[0]]}, tail=44)
    more, _ = traces.trace_tail({ids[1]: reqs[ids[1]]}, tail=45)
    for s in more:
        s["step"] += len(steps)
    check_trace(runner_for(folder, backend, dtype), steps + more, reqs, cfg, stored, dtype)


@pytest.mark.parametrize("name", ["a", "b", "c", "e"])
def test_portions_of_any_size(backend, dtype, name, tmp_path_factory):
    """Portions of 7, 2, 16, 3, 24, 2, 33, ... tokens: portions that end inside a page, inside a
    chunk and inside the convolutions' reach, each starting behind a token of the one before."""
    folder, cfg, stored = model_case(name, dtype, tmp_path_factory)
    reqs = traces.random_requests(cfg["vocab"], [90, 37], seed=13)
    steps, _ = traces.trace_portions(reqs)
    check_trace(runner_for(folder, backend, dtype), steps, reqs, cfg, stored, dtype)


@pytest.mark.parametrize("name", ["a", "c", "e"])
def test_mixed_batches_reuse_pages_and_slots(backend, dtype, name, tmp_path_factory):
    """Seven unequal requests through three slots and a pool that holds three of them: portions
    beside single tokens, requests left out of steps, pages and slots of finished requests taken
    by later ones with their old contents still there."""
    folder, cfg, stored = model_case(name, dtype, tmp_path_factory)
    reqs = traces.random_requests(cfg["vocab"], [50, 9, 75, 33, 2, 64, 21], seed=14)
    steps, peak = traces.trace_mixed(reqs, live=3, seed=5)
    runner = runner_for(folder, backend, dtype, num_pages=-(-peak // 16), max_num_seqs=3)
    check_trace(runner, steps, reqs, cfg, stored, dtype)
    assert runner.cache.num_free_pages() == -(-peak // 16)


def test_one_slot_used_by_requests_in_a_row(backend, dtype, tmp_path_factory):
    """One state slot, three requests one after the other, decoded from their first token on and
    as portions: the convolutions' rows, both states and the previous token start anew."""
    folder, cfg, stored = model_case("a", dtype, tmp_path_factory)
    reqs = traces.random_requests(cfg["vocab"], [12, 17, 9], seed=17)
    steps, _ = traces.trace_tail(reqs, tail=100)
    runner = runner_for(folder, backend, dtype, num_pages=4, max_num_seqs=1)
    check_trace(runner, steps, reqs, cfg, stored, dtype)
    steps, _ = traces.trace_portions(reqs)
    check_trace(runner, steps, reqs, cfg, stored, dtype)


def test_a_request_alone_equals_itself_in_a_batch(backend, dtype, tmp_path_factory):
    """The rows of a request do not depend on what else the step holds (beyond rounding)."""
    folder, cfg, stored = model_case("a", dtype, tmp_path_factory)
    reqs = traces.random_requests(cfg["vocab"], [40, 23, 31], seed=15)
    alone = {}
    for rid, tokens in reqs.items():
        steps, _ = traces.trace_portions({rid: tokens})
        out = traces.replay_in_process(runner_for(folder, backend, dtype), steps)
        alone[rid] = traces.collect(steps, out, cfg["vocab"])[rid]
    steps, _ = traces.trace_mixed(reqs, live=3, seed=2)
    out = traces.replay_in_process(runner_for(folder, backend, dtype), steps)
    together = traces.collect(steps, out, cfg["vocab"])
    rm.judge([rm.row_error(row, alone[rid][pos]) for rid in reqs
              for pos, row in together[rid].items()], dtype)


def test_long_prompts_and_long_decoding(backend, dtype, tmp_path_factory):
    """A prompt of hundreds of tokens in one step, then hundreds of single-token steps: chunks
    begin and pass, their pages are given back, the states go on."""
    folder, cfg, stored = model_case("a", dtype, tmp_path_factory)
    n, tail = (90, 40) if backend.type == "cpu" else (390, 150)
    reqs = traces.random_requests(cfg["vocab"], [n], seed=16)
    steps, _ = traces.trace_tail(reqs, tail=tail)
    check_trace(runner_for(folder, backend, dtype), steps, reqs, cfg, stored, dtype)


def test_chunks_give_their_pages_back(backend, tmp_path_factory):
    """A model whose attention layers all have chunks holds no more pages than the longest chunk
    and a step take, however long the sequence: 300 tokens through 5 pages a group."""
    folder, cfg, stored = model_case("a", "float32", tmp_path_factory)
    n = 80 if backend.type == "cpu" else 300
    reqs = traces.random_requests(cfg["vocab"], [n], seed=26)
    steps, _ = traces.trace_tail(reqs, tail=n - 10)
    check_trace(runner_for(folder, backend, "float32", num_pages=5, max_num_seqs=1), steps, reqs,
                cfg, stored, "float32")


def test_prompts_of_hundreds_of_tokens_at_head_sizes_of_real_models(backend, dtype,
                                                                    tmp_path_factory):
    """Heads of 64 and 128: whole prompts of up to 700 tokens in one step (the attention
    kernels' tiles of 64 and 128 queries, long runs in the recurrences), the same prompts with
    their ends decoded, and in portions beside each other; a long portion beside single tokens
    of others; at the end a context of more than 1,024 keys."""
    folder, cfg, stored = model_case("d", dtype, tmp_path_factory)
    lengths = [120] if backend.type == "cpu" else [700, 300, 130, 257]
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
    """Weights in which, all through the layers, coordinate 0 of the stream is nonzero at
    ``KEY_TOKEN`` only, coordinate 1 at ``QUERY_TOKEN`` only and coordinate 2 the same at every
    token: the embedding sets them, the pair table and every sublayer's norm leave them alone, and
    the final norm's weight lets none through to the head."""
    w = rm.make_weights(cfg, seed=seed)
    w["embed"][:, :3] = 0.0
    w["embed"][:, 2] = 2.0
    w["embed"][KEY_TOKEN, 0] = 3.0
    w["embed"][QUERY_TOKEN, 1] = 3.0
    for name in w:
        if name == "bigram":
            w[name][:, :3] = 0.0
        elif name.endswith((".norm1", ".norm2", ".side.norm", "final.norm")):
            w[name][:3] = 0.0
    return w


def _attention_stands_out(cfg, w, layer, boost=12.0):
    """In every head of ``layer``'s attention the key of ``KEY_TOKEN`` gets a score far above the
    others' from a query of ``QUERY_TOKEN``: one channel of every key head reads stream
    coordinate 0, the same channel of every query head coordinate 1 (a channel that is not
    rotated, or else the first of the slowest pair, whose other one is emptied); the norms'
    weights let it through, the biases leave it alone."""
    m = cfg["layers"][layer]["mixer"]
    p, d = f"l{layer}.mix", m["dim"]
    dims = (m.get("rot") or {}).get("dims", 0)
    chans = [dims] if dims < d else [dims - 2, dims - 1]
    for name, heads in (("q", m["heads"]), ("k", m["kv_heads"])):
        for head in range(heads):
            for n, c in enumerate(chans):
                row = head * d + c
                w[f"{p}.{name}"][row] = 0.0
                if n == 0:
                    w[f"{p}.{name}"][row, 1 if name == "q" else 0] = boost
                w[f"{p}.{name}.b"][row] = 0.0
                w[f"{p}.{name}.norm"][row] = 2.5
    if "softcap" in m:
        m["softcap"] = 25.0
    return w


def _tokens(vocab, n, seed):
    return [t if t not in (KEY_TOKEN, QUERY_TOKEN) else FILL_TOKEN
            for t in rm.prompts(vocab, [n], seed=seed)[0]]


@pytest.mark.parametrize("layer, offset", [(1, 0), (1, -1), (3, 0), (3, -1), (6, 0), (6, -1)])
def test_keys_just_inside_and_outside_a_chunk(backend, dtype, layer, offset, tmp_path_factory,
                                              monkeypatch):
    """Chunks of 20, 16 (a page) and 33 positions.  A key that stands out is the first of a
    query's chunk or the last of the chunk before it; the query stands in the chunk's middle, at
    its end, and (decoded) in a later chunk.  A chunk that begins a token late or early,
    in a prompt's portion or decoded alone, moves the row far."""
    if backend.type == "cpu" and (layer, offset) not in ((1, 0), (3, -1), (6, 0)):
        pytest.skip("the double takes its time: one side of every edge here, all on the GPU")
    cfg = copy.deepcopy(rm.CONFIG_A)
    size = cfg["layers"][layer]["mixer"]["mask"]["size"]
    w = _attention_stands_out(cfg, _marked(cfg, seed=31 + layer), layer)
    folder, _, stored = model_case("a", dtype, tmp_path_factory, weights=w, tag=f"edge{layer}",
                                   config=cfg)
    n = 4 * size
    tokens = _tokens(cfg["vocab"], n, seed=32)
    queries = (size + size // 2, 3 * size - 2, n - 3)
    for query in queries:
        tokens[query] = QUERY_TOKEN
        tokens[query // size * size + offset] = KEY_TOKEN
    a = rm.plain_logits(plain, cfg, stored, tokens)
    mask = plain.chunk_mask

    def off_by_one(positions, c):
        seen = mask(positions, c)
        i, j = positions.reshape(-1, 1), positions.reshape(1, -1)
        if c != size:
            return seen
        start = i - i % c
        return seen & (j != start) | (j == i) if offset == 0 else seen | (j == start - 1)

    monkeypatch.setattr(plain, "chunk_mask", off_by_one)
    b = rm.plain_logits(plain, cfg, stored, tokens)
    monkeypatch.setattr(plain, "chunk_mask", mask)
    for query in queries:
        assert rm.row_error(a[query], b[query]) > 0.03
    reqs = {"r": tokens}
    steps, _ = traces.trace_tail(reqs, tail=size // 2)
    check_trace(runner_for(folder, backend, dtype), steps, reqs, cfg, stored, dtype)
    steps, _ = traces.trace_portions(reqs)
    check_trace(runner_for(folder, backend, dtype), steps, reqs, cfg, stored, dtype)


@pytest.mark.parametrize("far", [0, 15, 16, 17, 48])
def test_a_far_key_that_stands_out(backend, dtype, far, tmp_path_factory):
    """A layer that sees every earlier key, over pages of 16: the token at ``far`` (a page's first
    or last position among them) takes most of the weight of queries 100 and more positions on,
    in a prompt's portion and decoded alone."""
    if backend.type == "cpu" and far not in (0, 15):
        pytest.skip("the double takes its time: a page's two sides here, all on the GPU")
    cfg = copy.deepcopy(rm.CONFIG_B)
    w = _attention_stands_out(cfg, _marked(cfg, seed=41), 0)
    folder, _, stored = model_case("b", dtype, tmp_path_factory, weights=w, tag="far", config=cfg)
    tokens = _tokens(cfg["vocab"], 160, seed=42)
    tokens[far] = KEY_TOKEN
    tokens[far + 100] = tokens[157] = QUERY_TOKEN
    probs, _ = plain.attention_scores(stored, "l0.mix", cfg["layers"][0]["mixer"],
                                      plain.embed(cfg, stored, tokens), cfg["norm"]["eps"])
    assert float(probs[:, far + 100, far].min()) > 0.7 and float(probs[:, 157, far].min()) > 0.7
    reqs = {"r": tokens}
    steps, _ = traces.trace_tail(reqs, tail=6)
    check_trace(runner_for(folder, backend, dtype), steps, reqs, cfg, stored, dtype)
    steps, _ = traces.trace_portions(reqs)
    check_trace(runner_for(folder, backend, dtype), steps, reqs, cfg, stored, dtype)


def _delta_keeps(cfg, w, layer):
    """``layer``'s delta mixer hardly decays, writes at ``KEY_TOKEN`` only, and reads what that
    token wrote at ``QUERY_TOKEN``: one channel of every key head reads coordinate 0, the same
    channel of every query head coordinate 1, the step size coordinates 0 and 2."""
    m, p = cfg["layers"][layer]["mixer"], f"l{layer}.mix"
    w[p + ".A_log"][:] = -5.0
    w[p + ".a2"][:] = 0.0
    w[p + ".dt_bias"][:] = -2.0
    w[p + ".b"][:] = 0.0
    w[p + ".b"][:, 2] = -4.0
    w[p + ".b"][:, 0] = 4.0
    for n, coordinate in (("q", 1), ("k", 0)):
        for head in range(m["kv_heads"]):
            row = head * m["dim"] + 2
            w[f"{p}.{n}"][row] = 0.0
            w[f"{p}.{n}"][row, coordinate] = 20.0
            w[f"{p}.{n}.conv"][row] = 0.0
            w[f"{p}.{n}.conv"][row, -1] = 1.0


def _rglru_keeps(cfg, w, layer):
    """``layer``'s recurrence hardly decays, takes a large input at ``KEY_TOKEN`` and lets its
    state through at ``QUERY_TOKEN``."""
    p = f"l{layer}.mix"
    w[p + ".ra"][:] = 0.0
    w[p + ".ra.b"][:] = -6.0
    w[p + ".lam"][:] = 0.0
    w[p + ".x"][::2] = 0.0
    w[p + ".x"][::2, 0] = 30.0
    w[p + ".y"][::2, 1] = 10.0


@pytest.mark.parametrize("layer, far", [(0, 0), (0, 31), (4, 64), (2, 0), (2, 32), (5, 63)])
def test_a_far_token_in_the_states(backend, dtype, layer, far, tmp_path_factory):
    """A token 100 and more positions back (at the borders of the recurrences' tiles and chunks
    among them) decides what either recurrent state holds for the queries, in a prompt's portion,
    decoded alone, and with the prompt cut right behind it."""
    if backend.type == "cpu" and (layer, far) not in ((4, 64), (2, 32)):
        pytest.skip("the double takes its time: one of each kind here, all on the GPU")
    cfg = copy.deepcopy(rm.CONFIG_A)
    w = _marked(cfg, seed=51 + layer)
    (_delta_keeps if cfg["layers"][layer]["type"] == "channel_delta" else _rglru_keeps)(cfg, w, layer)
    folder, _, stored = model_case("a", dtype, tmp_path_factory, weights=w, tag=f"state{layer}",
                                   config=cfg)
    tokens = _tokens(cfg["vocab"], 180, seed=52)
    tokens[far] = KEY_TOKEN
    tokens[far + 100] = tokens[176] = QUERY_TOKEN
    moved = list(tokens)
    moved[far] = FILL_TOKEN
    a, b = rm.plain_logits(plain, cfg, stored, tokens), rm.plain_logits(plain, cfg, stored, moved)
    for query in (far + 100, 176):
        assert rm.row_error(a[query], b[query]) > 0.03
    reqs = {"r": tokens}
    steps, _ = traces.trace_tail(reqs, tail=8)
    check_trace(runner_for(folder, backend, dtype), steps, reqs, cfg, stored, dtype)
    cuts = [0, far + 1, far + 3, 176, 177, 180]
    steps = [{"step": i, "end": [], "entries": [
        {"id": "r", "tokens": tokens[lo:hi], "want": list(range(hi - lo))}]}
        for i, (lo, hi) in enumerate(zip(cuts, cuts[1:]))]
    steps[-1]["end"] = ["r"]
    check_trace(runner_for(folder, backend, dtype), steps, reqs, cfg, stored, dtype)


def test_scores_reach_the_cap(backend, dtype, tmp_path_factory):
    """Norm weights of queries and keys four times as large: most scores of the capped layers sit
    at the cap, where it, not the product, decides the weights."""
    cfg = rm.CONFIG_C
    w = rm.make_weights(cfg, seed=81)
    for i, layer in enumerate(cfg["layers"]):
        if layer["mixer"].get("softcap"):
            w[f"l{i}.mix.q.norm"] *= 4.0
            w[f"l{i}.mix.k.norm"] *= 4.0
    folder, _, stored = model_case("c", dtype, tmp_path_factory, weights=w, tag="cap")
    reqs = traces.random_requests(cfg["vocab"], [40, 24], seed=82)
    steps, _ = traces.trace_tail(reqs, tail=10)
    check_trace(runner_for(folder, backend, dtype), steps, reqs, cfg, stored, dtype)


@pytest.mark.parametrize("change", ["bigram", "side", "gate", "bias", "values"])
def test_every_input_mechanism_moves_the_plain_rows(change):
    """What the engine is held against depends on each of these: the pair table, the token input,
    the attention's gate, its biases, and that the values are the keys in front of the norm."""
    cfg = rm.CONFIG_A
    stored = rm.as_stored(rm.make_weights(cfg, 7), torch.float32)
    tokens = rm.prompts(cfg["vocab"], [24], seed=8)[0]
    other = dict(stored)
    if change == "bigram":
        other["bigram"] = stored["bigram"].roll(1, 0)
    elif change == "side":
        other["side.embed"] = stored["side.embed"].roll(1, 1)
    elif change == "gate":
        other["l1.mix.g"] = -stored["l1.mix.g"]
    elif change == "bias":
        other["l1.mix.k.b"] = torch.zeros_like(stored["l1.mix.k.b"])
    else:
        # signs turned in every second key channel and back in the norm's weight: the scores
        # stay as they are, the values do not
        sign = torch.ones_like(stored["l1.mix.k.b"])
        sign[::2] = -1.0
        other["l1.mix.k"] = stored["l1.mix.k"] * sign.reshape(-1, 1)
        other["l1.mix.k.b"] = stored["l1.mix.k.b"] * sign
        other["l1.mix.k.norm"] = stored["l1.mix.k.norm"] * sign
    a, b = rm.plain_logits(plain, cfg, stored, tokens), rm.plain_logits(plain, cfg, other, tokens)
    assert max(rm.row_error(x, y) for x, y in zip(a, b)) > 1e-2


# -------------------------------------------------------------------- engine and scheduler
@pytest.mark.parametrize("seats, budget", [(3, 16), (4, 64)])
def test_greedy_generation_through_the_engine(backend, dtype, seats, budget, tmp_path_factory):
    """Five requests through three or four seats with a token budget that cuts the prompts: every
    generated token is the plain implementation's pick, up to a near-tie of its logits.  (Decode
    steps are launched ahead on tokens that are on the device only, which the pair table reads
    there.)"""
    from rust_llm_inference_server_amd.engine import Engine, load_model
    if backend.type == "cpu" and seats == 4:
        pytest.skip("one of them on the double")
    folder, cfg, stored = model_case("a", dtype, tmp_path_factory)
    model = load_model(folder, dtype, 256, backend)
    engine = Engine(model, EngineConfig(max_num_seqs=seats, max_batched_tokens=budget,
                                        num_pages=48, block_size=8, max_seq_len=256,
                                        watermark_pages=1))
    prompts = rm.prompts(cfg["vocab"], [5, 21, 1, 34, 12], seed=18)
    outs = engine.generate(prompts, SamplingParams.greedy(7))
    margin = 1e-3 if dtype == "float32" else 0.5
    for p, o in zip(prompts, outs):
        assert o.finish_reason == "length" and len(o.token_ids) == 7
        tokens = list(p)
        for got in o.token_ids:
            last = rm.plain_logits(plain, cfg, stored, tokens)[-1]
            best = int(torch.argmax(last))
            if got != best:
                assert float(last[best] - last[got]) < margin
            tokens.append(got)
    engine.runner.cache.check_invariants()


def test_a_fork_takes_the_state_along(backend, dtype, tmp_path_factory):
    """A request forked inside a chunk goes on with its parent's states, convolution rows and
    previous token, and neither disturbs the other."""
    from rust_llm_inference_server_amd.engine import StepEntry
    folder, cfg, stored = model_case("a", dtype, tmp_path_factory)
    runner = runner_for(folder, backend, dtype)
    tokens = rm.prompts(cfg["vocab"], [40], seed=27)[0]
    runner.reserve(1, 25)
    runner.step([StepEntry(1, tokens[:25], [])])
    runner.fork(1, 2)
    other = [(t + 3) % cfg["vocab"] for t in tokens[25:33]]
    errors = []
    for seq, rest in ((1, tokens[25:33]), (2, other)):
        runner.reserve(seq, 33)
        got = runner.step([StepEntry(seq, rest, list(range(8)))]).float().cpu()
        want = rm.plain_logits(plain, cfg, stored, tokens[:25] + rest)[25:]
        errors += [rm.row_error(x, y) for x, y in zip(got, want)]
    rm.judge(errors, dtype)


@pytest.mark.gpu
@pytest.mark.parametrize("name, dtype_name", [("a", "float32"), ("a", "bfloat16"),
                                              ("e", "bfloat16")])
def test_the_replay_program_runs_the_model(name, dtype_name, tmp_path_factory, tmp_path):
    folder, cfg, stored = model_case(name, dtype_name, tmp_path_factory)
    reqs = traces.random_requests(cfg["vocab"], [40, 7, 25, 33, 18], seed=19)
    steps, peak = traces.trace_mixed(reqs, live=4, seed=3)
    out = traces.replay_program(folder, dtype_name, steps, peak, str(tmp_path / "out"),
                                cfg["vocab"])
    got = traces.collect(steps, out, cfg["vocab"])
    errors = []
    for rid, tokens in reqs.items():
        want = rm.plain_logits(plain, cfg, stored, tokens)
        errors += [rm.row_error(row, want[pos]) for pos, row in got[rid].items()]
    rm.judge(errors, dtype_name)


@pytest.mark.gpu
def test_the_command_line_generates_and_scores(tmp_path_factory, tmp_path, capsys):
    """``rlis generate`` picks the design by config.json and prints the plain implementation's
    greedy tokens; ``rlis perplexity`` scores a token file through the same step function."""
    from rust_llm_inference_server_amd import cli
    folder, cfg, stored = model_case("c", "float32", tmp_path_factory)
    prompt = rm.prompts(cfg["vocab"], [11], seed=20)[0]
    rc = cli.main(["generate", "--model", folder, "--dtype", "f32", "--max-seq-len", "128",
                   "--num-pages", "32", "--block-size", "8", "--max-num-seqs", "2",
                   "--max-tokens", "5", "--prompt-ids", ",".join(map(str, prompt))])
    out = capsys.readouterr()
    assert rc == 0
    got = [int(t) for t in out.out.split()]
    tokens = list(prompt)
    for g in got:
        last = rm.plain_logits(plain, cfg, stored, tokens)[-1]
        best = int(torch.argmax(last))
        assert g == best or float(last[best] - last[g]) < 1e-3
        tokens.append(g)
    assert len(got) == 5 and "output 5 tok (length)" in out.err
    ids = tmp_path / "ids.txt"
    ids.write_text(" ".join(map(str, rm.prompts(cfg["vocab"], [96], seed=21)[0])))
    rc = cli.main(["perplexity", "--model", folder, "--dtype", "f32", "--max-seq-len", "128",
                   "--ids-file", str(ids), "--ctx", "32"])
    out = capsys.readouterr()
    assert rc == 0 and json.loads(out.out.strip().splitlines()[-1])["ppl"] > 1.0
