"""The Nililix architecture in the engine against the plain implementation of its equations
(tests/plain_nililix.py): each mechanism alone, every way of cutting the work, pages and state slots
used again, captured steps, long decoding, generation through the entry point, and keys that a
crafted query singles out at the places where an index can be off by one."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import plain_nililix as plain
import traces
from nililix_util import CONFIGS, MIX_A, as_double, every_expert, make_folder, random_config, rounded, row_err
from util import random_tokens

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
# float32: everything is computed in 32 bits, what is left is the order of sums (the plain model itself, run in
# float32, differs from its float64 run by up to 7e-6 of a row on these models).  bfloat16: weights are rounded for the
# plain model too; the products' inputs and outputs are rounded in the engine only, the models are made tame so that
# this rounding is not amplified, and a row's limit grows with what rounding nothing but the products' operands does to
# it in the plain model (`round_operands`, the worst of four samples; 1e-2 as a rule), and every token uses every expert
# (a score that bfloat16 moves past its neighbour would otherwise choose another expert; the router's choices are compared
# in float32 and, with scores that are apart, at the part itself).  A fault of a mechanism (a key off by one, a lost
# convolution input, a sink left out) moves a row by its whole size in either precision.
TOL = {"float32": 1e-4, "bfloat16": 5e-2}
LENGTHS = {"A": [70, 133, 33, 200, 97, 64], "B": [1, 9, 40, 100, 150, 57], "odd": [31, 2, 77, 50], "wide": [50, 7, 101],
           "loop_end": [40, 75, 130, 9], "loop_once": [40, 75, 130, 9], "plain": [24, 121, 48, 5], "moe": [24, 61, 5]}


class Limits(dict):
    """{request: the plain model's logits}, with the rounding noise of every row beside them."""

    def __init__(self, cfg, w64, reqs, dtype):
        super().__init__({rid: plain.forward(cfg, w64, toks) for rid, toks in reqs.items()})
        self.noise = {}
        if dtype == "bfloat16":
            for rid, toks in reqs.items():
                cuts = [plain.forward(cfg, w64, toks, round_operands=torch.bfloat16, round_scale=s) for s in (1.0, 1.23, 1.51, 1.77)]
                self.noise[rid] = [max(row_err(c[i], self[rid][i]) for c in cuts) for i in range(len(toks))]

    def limit(self, rid, pos, tol):
        return tol + (4.0 * self.noise[rid][pos] if rid in self.noise else 0.0)


_cache = {}


def config_for(name, dtype):
    cfg, block = CONFIGS[name]
    return (every_expert(cfg) if dtype == "bfloat16" else cfg), block


def material(name, dtype, tmp_path_factory):
    key = (name, dtype)
    if key not in _cache:
        cfg, block = config_for(name, dtype)
        folder, w = make_folder(tmp_path_factory.mktemp(f"nililix_{name}_{dtype}"), cfg, seed=11,
                                store=torch.bfloat16 if dtype == "bfloat16" else torch.float32,
                                sharpen=1.0 if dtype == "bfloat16" else 3.0)
        w64 = rounded(w) if dtype == "bfloat16" else as_double(w)
        reqs = {f"r{i}": random_tokens(n, cfg["vocab"], 100 * i + len(name)) for i, n in enumerate(LENGTHS[name])}
        ref = Limits(cfg, w64, reqs, dtype)
        _cache[key] = (folder, cfg, w64, reqs, ref, block)
    return _cache[key]


def make_runner(folder, dtype, block_size, max_tokens, max_seqs=4):
    from tiny_llm_amd.config import EngineConfig
    from tiny_llm_amd.engine.loading import build_runner, load_model
    engine = EngineConfig(dtype=dtype, kv_block_size=block_size, max_cache_tokens=max_tokens, max_num_seqs=max_seqs,
                          max_num_batched_tokens=1 << 16, use_graphs=False)
    _, dec = load_model(folder, engine)
    runner = build_runner(dec, engine)
    for g in runner.cache.groups:               # stale or unwritten pages must never reach a result
        for t in g.tensors.values():
            t.fill_(float("nan"))
    for st in runner.cache.states.values():     # a state slot is cleared when a request takes it
        st.fill_(12345)
    return runner


def replay(runner, steps, use_graph=False):
    from tiny_llm_amd.engine.step import StepEntry
    out = {}
    for s in steps:
        logits = runner.step([StepEntry(e["id"], e["tokens"], e["want"]) for e in s["entries"]], use_graph=use_graph)
        if logits.shape[0]:
            out[s["step"]] = logits.cpu()
        for rid in s["end"]:
            runner.finish(rid)
        runner.cache.audit()
    return out


def check(out, steps, ref, tol):
    rows = traces.rows_of(steps)
    assert set(rows) == set(out)
    worst = 0.0
    for step, where in rows.items():
        got = out[step]
        assert got.shape[0] == len(where)
        for i, (rid, pos) in enumerate(where):
            assert torch.isfinite(got[i]).all(), (step, rid, pos)
            e = row_err(got[i], ref[rid][pos])
            limit = ref.limit(rid, pos, tol)
            worst = max(worst, e)
            assert e < limit, f"step {step}: request {rid} position {pos}: err {e:.3e}, limit {limit:.3e}"
    return worst


def r64(n):
    return -(-n // 64) * 64


def all_free(runner):
    return runner.cache.free_blocks() == [g.pool.num_blocks for g in runner.cache.groups] and \
        runner.cache.free_slots == runner.cache.max_seqs


CASES = [(n, "float32") for n in ("plain", "moe", "loop_end", "loop_once", "wide", "A", "B", "odd")] + \
        [(n, "bfloat16") for n in ("plain", "moe", "loop_end", "loop_once", "wide", "A", "B")]


@pytest.mark.parametrize("name,dtype", CASES)
def test_whole_tail_portions(name, dtype, tmp_path_factory):
    """Each request alone: whole, its tail token by token (windows pass over decoded tokens), and in
    portions down to two tokens (small models of one mechanism each, then the mixed models)."""
    folder, cfg, w, reqs, ref, block = material(name, dtype, tmp_path_factory)
    biggest = max(r64(len(t)) for t in reqs.values())
    for build in (traces.whole, traces.tail_one_by_one, traces.portions):
        steps = build(reqs)
        runner = make_runner(folder, dtype, block, biggest, max_seqs=1)
        worst = check(replay(runner, steps), steps, ref, TOL[dtype])
        print(f"{name} {dtype} {build.__name__}: worst {worst:.2e}")
        assert all_free(runner)


def test_odd_sizes_in_a_bfloat16_engine(tmp_path_factory):
    """A checkpoint stored in bfloat16 whose sizes are multiples of nothing, asked for in bfloat16: the float32
    kernels serve it (with a warning), mixed batches and portions agree with the plain model to float32's limit."""
    cfg, block = CONFIGS["odd"]
    folder, w = make_folder(tmp_path_factory.mktemp("nililix_odd_bf16"), cfg, seed=4, store=torch.bfloat16)
    reqs = {f"r{i}": random_tokens(n, cfg["vocab"], 50 + i) for i, n in enumerate(LENGTHS["odd"])}
    ref = Limits(cfg, rounded(w), reqs, "float32")
    steps, peak = traces.mixed(reqs, seed=3)
    with pytest.warns(RuntimeWarning, match="served in float32"):
        runner = make_runner(folder, "bfloat16", block, max(peak, max(r64(len(t)) for t in reqs.values())))
    assert runner.decoder.dtype == torch.float32
    for st in (steps, traces.portions(reqs)):
        check(replay(runner, st), st, ref, TOL["float32"])
        assert all_free(runner)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B"])
def test_mixed_batches_reuse_pages_and_slots(name, dtype, tmp_path_factory):
    """Up to four live requests of unequal length in one step, six requests through four state slots
    and a pool smaller than their sum; every row against the request run alone by the plain model."""
    folder, cfg, w, reqs, ref, block = material(name, dtype, tmp_path_factory)
    for seed in (0, 1):
        steps, peak = traces.mixed(reqs, seed=seed)
        assert peak < sum(r64(len(t)) for t in reqs.values())
        runner = make_runner(folder, dtype, block, peak, max_seqs=4)
        worst = check(replay(runner, steps), steps, ref, TOL[dtype])
        print(f"{name} {dtype} mixed {seed}: worst {worst:.2e}, pool {peak}")
        assert all_free(runner)


@pytest.mark.parametrize("seed", range(10))
def test_configurations_drawn_at_random(seed, tmp_path):
    """Sizes nobody chose: width, head counts and sizes with and without a matrix-core kernel, keys wider and
    narrower than values, windows from one position to more than the prompt and none, rotated dims, frequency scaling, taps,
    dense layers, groups of experts, layers without feed-forward, repeated runs, pages of 4 to 32 tokens; mixed batches,
    portions and whole prompts in both precisions."""
    import random
    drawn = random_config(seed)
    rng = random.Random(1000 + seed)
    block = rng.choice([4, 8, 16, 32])
    for dtype in ("float32", "bfloat16"):
        cfg = every_expert(drawn) if dtype == "bfloat16" else drawn
        folder, w = make_folder(tmp_path / dtype, cfg, seed=seed, store=torch.bfloat16 if dtype == "bfloat16" else torch.float32,
                                sharpen=1.0 if dtype == "bfloat16" else 3.0)
        w64 = rounded(w) if dtype == "bfloat16" else as_double(w)
        reqs = {f"r{i}": random_tokens(n, cfg["vocab"], 7 * seed + i) for i, n in enumerate([rng.randrange(1, 140) for _ in range(5)])}
        ref = Limits(cfg, w64, reqs, dtype)
        steps, peak = traces.mixed(reqs, seed=seed)
        runner = make_runner(folder, dtype, block, max(peak, max(r64(len(t)) for t in reqs.values())))
        for st in (steps, traces.portions(reqs), traces.whole(reqs)):
            worst = check(replay(runner, st), st, ref, TOL[dtype])
            assert all_free(runner)
        print(f"seed {seed} {dtype}: worst {worst:.2e}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_layer_sizes_of_a_larger_model(dtype, tmp_path):
    """Two layers, repeated, with heads of the sizes a model of some billions of weights has (heads of 128, a window that a
    prompt of 300 tokens leaves, experts of 64 hidden units): a whole prompt (the kernels for many rows), the same in
    portions, and a tail decoded token by token beside a second request."""
    from nililix_util import attention, dense, layer, model, moe
    big = model(512, 1031, [
        layer(attention(16, 4, 128, 128, 4, 130, 64, (8.0, 1.0, 4.0, 128), 500000.0), moe(16, 4, 64, (4, 2))),
        layer(attention(8, 8, 128, 64, 3, 96, 128), dense(1408)),
    ], loop=(0, 2, 2), mult=0.6)
    cfg = every_expert(big) if dtype == "bfloat16" else big
    folder, w = make_folder(tmp_path, cfg, seed=5, store=torch.bfloat16 if dtype == "bfloat16" else torch.float32,
                            sharpen=1.0 if dtype == "bfloat16" else 3.0)
    w64 = rounded(w) if dtype == "bfloat16" else as_double(w)
    reqs = {"long": random_tokens(300, cfg["vocab"], 1), "short": random_tokens(45, cfg["vocab"], 2)}
    ref = Limits(cfg, w64, reqs, dtype)
    runner = make_runner(folder, dtype, 16, 384 + 64)
    for st in (traces.whole(reqs), traces.portions(reqs), traces.mixed(reqs, seed=1)[0]):
        worst = check(replay(runner, st), st, ref, TOL[dtype])
        assert all_free(runner)
        print(f"larger sizes {dtype}: worst {worst:.2e}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_captured_steps(dtype, tmp_path_factory):
    """The same cuttings with every step as a HIP graph of its shape (padding tokens, requests and
    rows), twice over so that the second pass replays what the first captured."""
    folder, cfg, w, reqs, ref, block = material("A", dtype, tmp_path_factory)
    steps, peak = traces.mixed(reqs, seed=2)
    runner = make_runner(folder, dtype, block, max(peak, max(r64(len(t)) for t in reqs.values())))
    for st in (steps, traces.portions(reqs), traces.tail_one_by_one(reqs)):
        for again in range(2):
            check(replay(runner, st, use_graph=True), st, ref, TOL[dtype])
            assert all_free(runner)
    assert runner.graph_steps > runner.eager_steps
    assert not any(g.capture_failed for g in runner._graphs.values())
    assert runner.decoder.graph_safe


def test_first_tokens(tmp_path_factory):
    """One to four tokens: the convolutions reach back into zeros, a softmax holds one key and the sink."""
    for name in ("A", "B"):
        folder, cfg, w, reqs, ref, block = material(name, "float32", tmp_path_factory)
        runner = make_runner(folder, "float32", block, 64)
        from tiny_llm_amd.engine.step import StepEntry
        for n in (1, 2, 3, 4):
            logits = runner.step([StepEntry("x", reqs["r3"][:n], list(range(n)))]).cpu()
            runner.finish("x")
            for i in range(n):
                assert row_err(logits[i], ref["r3"][i]) < TOL["float32"]


def test_long_decoding(tmp_path_factory):
    """Several hundred single-token steps: the convolutions' inputs are carried from step to step in every pass, every page
    edge is crossed by decoded tokens, the windows leave the first tokens behind."""
    folder, cfg, w, reqs, ref, block = material("A", "float32", tmp_path_factory)
    toks = random_tokens(330, cfg["vocab"], 4242)
    want = plain.forward(cfg, w, toks)
    runner = make_runner(folder, "float32", block, r64(330))
    from tiny_llm_amd.engine.step import StepEntry
    got = [runner.step([StepEntry("long", toks[:6], list(range(6)))]).cpu()]
    for i in range(6, 330):
        got.append(runner.step([StepEntry("long", [toks[i]], [0])]).cpu())
    got = torch.cat(got)
    worst = max(row_err(got[i], want[i]) for i in range(330))
    print(f"long decoding: worst {worst:.2e}")
    assert worst < TOL["float32"]


@pytest.mark.parametrize("graphs", [False, True])
def test_greedy_generation_through_the_engine(graphs, tmp_path_factory):
    """Engine.generate (scheduler, portions, captured steps, runs of chained decode steps) against
    greedy decoding with the plain model."""
    folder, cfg, w, reqs, ref, block = material("A", "float32", tmp_path_factory)
    from tiny_llm_amd import Engine, SamplingParams
    prompts = [reqs["r2"][:21], reqs["r3"][:5], reqs["r4"][:34]]
    eng = Engine(folder, dtype="float32", kv_block_size=block, max_num_seqs=2, max_num_batched_tokens=24,
                 max_model_len=256, use_graphs=graphs)
    out = eng.generate(prompts, SamplingParams.greedy(40, ignore_eos=True))
    for p, o in zip(prompts, out):
        seq = list(p)
        for _ in range(40):
            seq.append(int(plain.forward(cfg, w, seq)[-1].argmax()))
        assert o == seq[len(p):]
    eng.runner.cache.audit()
    if graphs:
        assert eng.runner.graph_steps > 0


def test_preempted_requests_are_computed_again(tmp_path_factory):
    """A pool so small that requests are preempted and recomputed from their first token: their state slots start
    empty again and the tokens are the same."""
    folder, cfg, w, reqs, ref, block = material("A", "float32", tmp_path_factory)
    from tiny_llm_amd import Engine, SamplingParams
    prompts = [reqs["r0"][:60], reqs["r1"][:50], reqs["r3"][:40]]
    big = Engine(folder, dtype="float32", kv_block_size=block, max_num_seqs=3, max_num_batched_tokens=64, max_model_len=256)
    want = big.generate(prompts, SamplingParams.greedy(30, ignore_eos=True))
    small = Engine(folder, dtype="float32", kv_block_size=block, max_num_seqs=3, max_num_batched_tokens=64,
                   max_model_len=256, num_kv_blocks=11)
    assert small.generate(prompts, SamplingParams.greedy(30, ignore_eos=True)) == want
    small.runner.cache.audit()


def test_trace_run_program(tmp_path_factory, tmp_path):
    folder, cfg, w, reqs, ref, block = material("A", "bfloat16", tmp_path_factory)
    steps, peak = traces.mixed(reqs, seed=3)
    out_dir = tmp_path / "out"
    proc = subprocess.run(
        [sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", "bfloat16",
         "--out", str(out_dir), "--max-tokens", str(peak)],
        input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=600)
    assert proc.returncode == 0, proc.stderr[-3000:]
    assert [l for l in proc.stdout.splitlines() if l.startswith("done ")] == [f"done {s['step']}" for s in steps]
    out = {}
    for step, where in traces.rows_of(steps).items():
        arr = np.fromfile(out_dir / f"{step}.f32", dtype="<f4")
        assert arr.size == len(where) * cfg["vocab"]
        out[step] = torch.from_numpy(arr.reshape(len(where), cfg["vocab"]))
    check(out, steps, ref, TOL["bfloat16"])


def test_command_line_and_seeded_sampling(tmp_path_factory):
    """bin/tiny_llm serves a Nililix folder as it serves any other (config.json chooses the model);
    seeded sampling through the engine does not depend on what else is in the batch."""
    folder, cfg, w, reqs, ref, block = material("A", "float32", tmp_path_factory)
    prompt = reqs["r2"][:12]
    proc = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "tiny_llm"), "--model_path", folder,
                           "--nodo_sample", "--max_new_tokens=5", "--dtype", "float32", "--ignore_eos",
                           "--prompt_ids", ",".join(map(str, prompt))], capture_output=True, text=True, timeout=300)
    assert proc.returncode == 0, proc.stderr[-2000:]
    got = [int(t) for t in proc.stdout.strip().splitlines()[-1].split()]
    seq = list(prompt)
    for _ in range(5):
        seq.append(int(plain.forward(cfg, w, seq)[-1].argmax()))
    assert got == seq[len(prompt):]
    from tiny_llm_amd import Engine, SamplingParams
    eng = Engine(folder, dtype="float32", kv_block_size=block, max_num_seqs=4, max_num_batched_tokens=64, max_model_len=256)
    params = SamplingParams(max_new_tokens=12, do_sample=True, temperature=0.9, top_k=40, top_p=0.95, seed=7,
                            ignore_eos=True)
    alone = eng.generate([prompt], params)[0]
    among = eng.generate([reqs["r0"][:30], prompt, reqs["r1"][:7]], params)[1]
    assert alone == among


def test_random_weights_from_a_configuration():
    """A configuration written by hand runs with seeded random weights (no files), as the measurements do."""
    from tiny_llm_amd import Engine, SamplingParams
    eng = Engine(config=MIX_A, dtype="bfloat16", kv_block_size=16, max_num_seqs=2, max_num_batched_tokens=32,
                 max_model_len=128, weights_seed=3, init_std=0.05)
    out = eng.generate([random_tokens(20, MIX_A["vocab"], 1), random_tokens(3, MIX_A["vocab"], 2)],
                       SamplingParams.greedy(8, ignore_eos=True))
    assert [len(o) for o in out] == [8, 8] and all(0 <= t < MIX_A["vocab"] for o in out for t in o)


# ------------------------------------------------------------------ mechanisms alone
def _paged(rows: torch.Tensor, table, block, n_blocks, dtype):
    """rows [n, kv_heads, d] laid into pages [n_blocks, kv_heads, block, d] at the blocks `table` names; NaN elsewhere."""
    n, g, d = rows.shape
    pages = torch.full((n_blocks, g, block, d), float("nan"), dtype=dtype, device="cuda")
    for j in range(n):
        pages[table[j // block], :, j % block] = rows[j].to(dtype)
    return pages


def _attend(kernel, qd, k_pages, v_pages, bt, pos_dev, heads, kvh, d, scale, window, vdim, opts):
    """Every row of qd a request of its own over the same pages, by the named attention kernel."""
    from tiny_llm_amd.kernels import ops
    T, dtype = qd.shape[0], qd.dtype
    out = torch.full((T, heads * vdim), float("nan"), dtype=torch.float32 if "float32 result" in kernel else dtype, device="cuda")
    tables = bt.repeat(T, 1).contiguous()
    each = torch.arange(T, dtype=torch.int32, device="cuda")
    opts = dict(opts, value_dim=vdim)
    if kernel.startswith("general"):
        return ops.paged_attention(qd, k_pages, v_pages, bt, torch.zeros_like(each), pos_dev, out, heads, kvh, d, scale, window, **opts)
    if "float32" in kernel and "many rows" in kernel:
        reps = -(-1024 // (T * kvh)) + 1
        n_t = T * reps
        big = torch.empty(n_t, heads * vdim, dtype=dtype, device="cuda")
        tiles = (torch.arange(n_t, dtype=torch.int32, device="cuda"),) * 2 + (torch.ones(n_t, dtype=torch.int32, device="cuda"),)
        ops.attention_f32(qd.repeat(reps, 1), k_pages, v_pages, bt.repeat(n_t, 1).contiguous(), tiles, pos_dev.repeat(reps),
                          big, heads, kvh, d, scale, window, **dict(opts, gate=opts["gate"].repeat(reps, 1)))
        assert all(torch.equal(big[:T], big[r * T:(r + 1) * T]) for r in range(1, reps))
        return big[:T]
    if kernel.startswith("matrix cores float32"):
        chunks = -(-bt.shape[1] * k_pages.shape[2] // ops.F32_CHUNK_KEYS) if "chunks" in kernel else 1
        part = torch.empty(chunks * T * heads * (d + 2), device="cuda") if chunks > 1 else None
        return ops.attention_f32(qd, k_pages, v_pages, tables, None, pos_dev, out, heads, kvh, d, scale, window, chunks, part, **opts)
    splits = 3 if "split" in kernel else 17 if "many parts" in kernel else 1
    part = torch.empty(splits * T * heads * (d + 2), device="cuda") if splits > 1 else None
    if "prompt" in kernel:
        waves = 8 if "eight waves" in kernel else 4
        return ops.flash_prefill(qd, k_pages, v_pages, tables, (each, each.clone(), torch.ones_like(each)), pos_dev, out, heads,
                                 kvh, d, scale, window, waves, splits, part, **opts)
    return ops.flash_attention(qd, k_pages, v_pages, tables, None, pos_dev, out, heads, kvh, d, scale, window, splits, part, **opts)


ATTENTION_KERNELS = ["general float32", "general bfloat16", "matrix cores float32", "matrix cores float32, chunks",
                     "matrix cores float32, many rows", "matrix cores bfloat16", "matrix cores bfloat16, split keys",
                     "matrix cores bfloat16, many parts", "matrix cores bfloat16, prompt", "matrix cores bfloat16, prompt, split keys",
                     "matrix cores bfloat16, prompt, eight waves", "matrix cores bfloat16, float32 result",
                     "matrix cores bfloat16, prompt, float32 result"]


@pytest.mark.parametrize("kernel", ATTENTION_KERNELS)
@pytest.mark.parametrize("window,heads,kvh,d,vdim,opts", [
    (37, 6, 2, 32, 20, {}), (1, 4, 4, 48, 48, {}), (64, 16, 1, 64, 24, {}), (150, 5, 1, 16, 12, {}), (0, 3, 3, 112, 96, {}),
    (50, 6, 2, 32, 32, {"keep": 7}), (50, 6, 2, 32, 16, {"softcap": 8.0, "out_scale": 0.6})])
def test_a_sink_a_gate_and_one_key(kernel, window, heads, kvh, d, vdim, opts):
    """One query per place of interest is aligned with one key (its score stands out from the others, and the sink's
    score, near it, takes a visible share): the result must be that key's value times what the sink leaves, times the
    gate, in the head's first `vdim` columns.  Keys at the window's first place, at both sides of a page's and a tile's
    edge, the query's own; the keys just outside the window and the one behind the query are far louder, and the mask must
    hide them.  The last head's sink lies far above every score: its result is nearly nothing."""
    if "float32 result" in kernel and vdim % 4:
        pytest.skip("float32 rows of heads that are no multiple of four are another kernel's case")
    dtype = torch.float32 if kernel.startswith(("general float32", "matrix cores float32")) else torch.bfloat16
    g = torch.Generator().manual_seed(5)
    n, block = 560, 16
    keys = torch.randn(n, kvh, d, generator=g)
    keys = keys / keys.norm(dim=-1, keepdim=True)
    vals = torch.randn(n, kvh, d, generator=g)
    table = torch.randperm(64, generator=g)[: -(-n // block)].tolist()
    k_pages, v_pages = _paged(keys, table, block, 64, dtype), _paged(vals, table, block, 64, dtype)
    keep, cap, out_scale = opts.get("keep", 0), opts.get("softcap", 0.0), opts.get("out_scale", 1.0)
    first = lambda pos: max(0, pos - window + 1) if window else 0
    seen = lambda pos: sorted(set(range(first(pos), pos + 1)) | set(range(min(keep, pos + 1))))
    places = {559, 512, 511, 400, 257, 256, 255, 199, 130, 129, 128, 64, 63, 48, 16, 15, 7, 1, 0, window, max(window - 1, 0)}
    cases = sorted({(pos, key) for pos in places if 0 <= pos < n
                    for key in (first(pos), pos, min(first(pos) + 1, pos), seen(pos)[len(seen(pos)) // 2])})
    T = len(cases)
    sinks = torch.randn(heads, generator=g) * 2.0 + 6.0
    sinks[heads - 1] = 300.0
    gate = torch.randn(T, heads + 3, generator=g) * 2.0
    q = torch.zeros(T, heads, d)
    for i, (pos, key) in enumerate(cases):
        vis = seen(pos)
        for h in range(heads):
            kv = h // (heads // kvh)
            # head 0 aims at the case's key, the others at keys of their own among the visible ones
            target = key if h == 0 else vis[(vis.index(key) + 3 * h) % len(vis)]
            q[i, h] = 9.0 * keys[target, kv]
            for hidden in (pos + 1, first(pos) - 1):       # would win if they were seen
                if 0 <= hidden < n and hidden not in vis:
                    q[i, h] += 40.0 * keys[hidden, kv]
    pos_dev = torch.tensor([c[0] for c in cases], dtype=torch.int32, device="cuda")
    bt = torch.tensor([table + [0] * (64 - len(table))], dtype=torch.int32, device="cuda")
    opts = dict(opts, sinks=sinks.cuda(), gate=gate.cuda()[:, :heads])
    out = _attend(kernel, q.reshape(T, heads * d).to(dtype).cuda(), k_pages, v_pages, bt, pos_dev, heads, kvh, d, 0.9, window, vdim, opts)
    kr, vr, qr = keys.to(dtype).double(), vals.to(dtype).double(), q.to(dtype).double()
    out = out.double().cpu().reshape(T, heads, vdim)
    for i, (pos, _) in enumerate(cases):
        vis = torch.tensor(seen(pos))
        for h in range(heads):
            kv = h // (heads // kvh)
            s = kr[vis, kv] @ qr[i, h] * 0.9
            if cap:
                s = cap * torch.tanh(s / cap)
            p = torch.softmax(torch.cat([s, sinks[h:h + 1].double()]), dim=0)[:-1]
            want = p @ vr[vis, kv][:, :vdim] * out_scale * torch.sigmoid(gate[i, h].double())
            assert torch.isfinite(out[i, h]).all()
            assert (out[i, h] - want).abs().max() < (3e-5 if dtype == torch.float32 else 2e-2), (pos, h)
    assert out[:, heads - 1].abs().max() < 1e-12
    assert out[:, 0].abs().max() > 0.3


@pytest.mark.parametrize("kernel", ["general float32", "matrix cores float32", "matrix cores bfloat16, prompt"])
@pytest.mark.parametrize("window,heads,vdim", [(24, 4, 20), (100, 6, 32), (3, 16, 8), (64, 2, 28)])
def test_a_prompts_portion_with_sinks_and_gates(kernel, window, heads, vdim):
    """A portion of a prompt behind cached tokens, cut in the middle of a window and of a page: tiles that hold several
    tokens whose windows differ; the pages the first window has left are NaN, as pages that were given back may be."""
    from tiny_llm_amd.kernels import ops
    dtype = torch.float32 if "float32" in kernel else torch.bfloat16
    g = torch.Generator().manual_seed(8)
    n, d, block, kvh, start = 390, 32, 16, 2, 257
    keys, vals = torch.randn(n, kvh, d, generator=g) * 1.5, torch.randn(n, kvh, d, generator=g)
    T = n - start
    q = torch.randn(T, heads, d, generator=g) * 1.5
    sinks, gate = torch.randn(heads, generator=g) * 2.0, torch.randn(T, heads, generator=g)
    table = torch.randperm(32, generator=g)[: -(-n // block)].tolist()
    k_pages, v_pages = _paged(keys, table, block, 32, dtype), _paged(vals, table, block, 32, dtype)
    for b in range(max(0, start - window + 1) // block):
        k_pages[table[b]] = v_pages[table[b]] = float("nan")
    pos_dev = torch.arange(start, n, dtype=torch.int32, device="cuda")
    bt = torch.tensor([table + [0] * (32 - len(table))], dtype=torch.int32, device="cuda")
    out = torch.empty(T, heads * vdim, dtype=dtype, device="cuda")
    qd = q.reshape(T, heads * d).to(dtype).cuda()
    width, opts = 16 // (heads // kvh), {"sinks": sinks.cuda(), "gate": gate.cuda(), "value_dim": vdim}
    if kernel.startswith("general"):
        ops.paged_attention(qd, k_pages, v_pages, bt, torch.zeros(T, dtype=torch.int32, device="cuda"), pos_dev, out,
                            heads, kvh, d, d ** -0.5, window, **opts)
    else:
        if "prompt" in kernel:
            width *= 4
        tok0 = torch.arange(0, T, width, dtype=torch.int32, device="cuda")
        tiles = (torch.zeros_like(tok0), tok0, torch.clamp(T - tok0, max=width).to(torch.int32))
        if "prompt" in kernel:
            ops.flash_prefill(qd, k_pages, v_pages, bt, tiles, pos_dev, out, heads, kvh, d, d ** -0.5, window, 4, 1, None, **opts)
        else:
            ops.attention_f32(qd, k_pages, v_pages, bt, tiles, pos_dev, out, heads, kvh, d, d ** -0.5, window, **opts)
    kr, vr, qr = (x.to(dtype).double() for x in (keys, vals, q))
    k_all, v_all = kr.repeat_interleave(heads // kvh, 1), vr.repeat_interleave(heads // kvh, 1)[..., :vdim]
    q_all = torch.zeros((n, heads, d), dtype=torch.float64)
    q_all[start:] = qr
    want = plain.attend(q_all, k_all, v_all, plain.window_mask(torch.arange(n), window), d ** -0.5, sinks.double())[start:]
    want = want * torch.sigmoid(gate.double())[:, :, None]
    got = out.double().cpu().reshape(T, heads, vdim)
    assert (got - want).abs().max() < (2e-5 if dtype == torch.float32 else 3e-2)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("dim,vdim,rot,taps,scaling", [(24, 16, 8, 3, (4.0, 1.0, 4.0, 64.0)), (16, 40, 16, 4, None), (6, 11, 2, 2, None),
                                                       (80, 8, 0, 6, None), (8, 8, 4, 1, (3.0, 1.0, 2.0, 30.0)), (136, 72, 40, 5, None)])
def test_convolution_then_rotation_of_neighbours(dtype, dim, vdim, rot, taps, scaling):
    """The short convolution over time on q, k and v with the request's saved inputs, then the rotation of neighbouring
    dims, no norm and no bias between; three requests of unequal length in state slots out of order, cut into steps of
    several tokens and of single ones (which bring the saved inputs up to date themselves)."""
    from tiny_llm_amd.engine.step import tile_lists
    from tiny_llm_amd.kernels import ops
    from tiny_llm_amd.parts.rotary import angle_tables
    g = torch.Generator().manual_seed(3)
    H, G, block = 3, 1, 4
    D = -(-max(dim, vdim) // 16) * 16
    qc, kc, vc = H * dim, G * dim, G * vdim
    channels = qc + kc + vc
    conv_w = torch.randn(channels, taps, generator=g)
    lens, slots = [9, 5, 31], [2, 0, 3]
    ps = [torch.randn(n, channels + 3, generator=g) for n in lens]
    want, cos, sin = [], None, None
    for p in ps:
        a = plain.causal_conv(p[:, :channels].double(), conv_w.double())
        n = a.shape[0]
        q, k = a[:, :qc].reshape(n, H, dim), a[:, qc:qc + kc].reshape(n, G, dim)
        if rot:
            spec = {"dims": rot, "base": 777.0}
            if scaling:
                spec["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
            q, k = (plain.rotate_pairs(x, torch.arange(n), spec) for x in (q, k))
        want.append((q, k, a[:, qc + kc:].reshape(n, G, vdim)))
    if rot:
        llama3 = None if scaling is None else (scaling[0], scaling[3], scaling[1], scaling[2])
        cos, sin = angle_tables(rot, 777.0, 512, "cuda", llama3=llama3)
    state = torch.full((4, channels * (taps - 1) + 5), float("nan"), device="cuda")
    for s in slots:
        state[s].zero_()
    rel = 1e-5 if dtype == torch.float32 else 2.0 ** -8         # a bfloat16 result is its value rounded once
    close = lambda got, w: bool(((got - w).abs() <= rel * (w.abs() + 1.0)).all())
    at = [0, 0, 0]
    for take in ([3, 1, 2], [1, 1, 1], [1, 0, 1], [4, 2, 19], [0, 1, 8]):
        live = [r for r in (1, 2, 0) if take[r]]
        p = torch.cat([ps[r][at[r]:at[r] + take[r]] for r in live]).cuda()
        T = p.shape[0]
        counts = [take[r] for r in live]
        pos = torch.tensor([at[r] + i for r in live for i in range(take[r])], dtype=torch.int32, device="cuda")
        cu = torch.tensor([0] + list(np.cumsum(counts)), dtype=torch.int32, device="cuda")
        sl = torch.tensor([slots[r] for r in live], dtype=torch.int32, device="cuda")
        single = max(counts) == 1
        pages = [torch.full((10, G, block, D), float("nan"), dtype=dtype, device="cuda") for _ in range(2)]
        q = torch.full((T, H * D), float("nan"), dtype=dtype, device="cuda")
        where = torch.randperm(40, generator=g)[:T].to(torch.int32)
        runs = None if single else tuple(torch.tensor(x, dtype=torch.int32, device="cuda") for x in tile_lists(counts, ops.CONV_RUN))
        conv = ops.ShortConv(conv_w.cuda(), state, 0, cu, sl, runs)
        ops.conv_attn_prepare(p, None, pos, cos, sin, where.cuda(), q, pages[0], pages[1], H, G, dim, vdim, conv, None, rot,
                              "interleaved", 1e-5)
        if not single and taps > 1:
            ops.conv_state_update(p, 0, channels, state, 0, cu, sl, taps, None)
        t = 0
        for r in live:
            for i in range(at[r], at[r] + take[r]):
                wq, wk, wv = (x[i] for x in want[r])
                got = q[t].double().cpu().reshape(H, D)
                assert close(got[:, :dim], wq) and (got[:, dim:] == 0).all(), (r, i)
                s = int(where[t])
                row = pages[0][s // block, :, s % block].double().cpu()
                assert close(row[:, :dim], wk) and (row[:, dim:] == 0).all(), (r, i)
                row = pages[1][s // block, :, s % block].double().cpu()
                assert close(row[:, :vdim], wv) and (row[:, vdim:] == 0).all(), (r, i)
                t += 1
            at[r] += take[r]
    assert at == lens
    if taps > 1:
        assert torch.isnan(state[1]).all() and not state[slots][:, :channels * (taps - 1)].isnan().any()


@pytest.mark.parametrize("T,W", [(1, 64), (5, 96), (3, 50), (2, 2048), (7, 1030), (2, 4100), (1, 8192), (3, 8191)])
def test_norm_added_to_the_stream_and_the_next_norm(T, W):
    """x <- x + m * RMS norm of y + a vector, and the next RMS norm of the new rows in either precision, by one kernel;
    each of the vector and the next norm may be left out."""
    from tiny_llm_amd.kernels import ops
    g = torch.Generator().manual_seed(T * W)
    x, y = torch.randn(T, W, generator=g) * 2.0, torch.randn(T, W, generator=g) * 3.0 + 0.5
    w1, w2, sh = (1.0 + 0.3 * torch.randn(W, generator=g) for _ in range(3))
    new = x.double() + 0.7 * plain.rms_norm(y.double(), w1.double(), 1e-2)
    for shift in (None, sh):
        want = new if shift is None else new + shift.double()
        for dtype in (None, torch.float32, torch.bfloat16):
            xd = x.cuda()
            h = None if dtype is None else torch.empty(T, W, dtype=dtype, device="cuda")
            ops.rms_norm_add(y.cuda(), w1.cuda(), xd, 0.7, 1e-2, then=None if h is None else (w2.cuda(), 3e-3, h),
                             shift=None if shift is None else shift.cuda())
            assert (xd.double().cpu() - want).abs().max() < 2e-5
            if h is not None:
                normed = plain.rms_norm(want, w2.double(), 3e-3)
                assert ((h.double().cpu() - normed).abs() <= (2e-5 if dtype == torch.float32 else 2.0 ** -8) * (normed.abs() + 1.0)).all()
    xd = x.cuda()
    ops.add_row_vector(xd, sh.cuda())
    assert torch.equal(xd.cpu(), x + sh)
    from tiny_llm_amd.kernels import KernelError
    with pytest.raises(KernelError):
        ops.rms_norm_add(torch.zeros(T, W + 1, device="cuda"), w1.cuda(), xd, 1.0, 1e-5)


@pytest.mark.parametrize("M,K,N", [(1, 64, 40), (8, 2048, 520), (16, 72, 5632), (17, 4096, 96), (40, 176, 1030), (65, 96, 36), (300, 256, 1032),
                                   (70, 5632, 128), (2048, 64, 512)])
def test_squared_relu_in_a_products_epilogue(M, K, N):
    """The few-row product, the tiled one and the one whose inner size is split, each with the activation on its float32
    sums; other types are refused."""
    from tiny_llm_amd.kernels import KernelError, ops
    g = torch.Generator().manual_seed(M + N)
    a, w = torch.randn(M, K, generator=g).bfloat16(), (torch.randn(N, K, generator=g) / K ** 0.5 * 2).bfloat16()
    out = torch.empty(M, N, dtype=torch.bfloat16, device="cuda")
    ops.linear(a.cuda(), w.cuda(), out, epilogue="relu2")
    want = torch.clamp(a.double() @ w.double().T, min=0.0) ** 2
    assert (out.double().cpu() - want).abs().max() < 6e-3 * want.abs().max()
    assert (out >= 0).all()
    with pytest.raises(KernelError):
        ops.linear(a.float().cuda(), w.float().cuda(), out.float(), epilogue="relu2")


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("T", [1, 30, 200])
def test_dense_feed_forward(dtype, T):
    from tiny_llm_amd.parts.mlp import ActMLP
    g = torch.Generator().manual_seed(T)
    W, F = 72, 200
    w = {"m.up": (torch.randn(F, W, generator=g) / 8).to(dtype), "m.down": (torch.randn(W, F, generator=g) / 14).to(dtype)}
    h = torch.randn(T, W, generator=g).to(dtype)
    part = ActMLP("m", dtype, torch.device("cuda"), hidden_size=W, intermediate_size=F)
    part.bind({k: v.cuda() for k, v in w.items()})
    want = plain.dense(h.double(), {k[2:]: v.double() for k, v in w.items()})
    err = (part.forward(h.cuda(), None, None).double().cpu() - want).abs().max() / want.abs().max()
    assert err < (1e-5 if dtype == torch.float32 else 1e-2)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("tokens", [3, 50, 500])
def test_experts_by_every_route(dtype, tokens):
    """The mixture alone by each of its three routes, with scores that are apart, so that both precisions choose alike: a
    group with the best single expert but the worse pair stays out, and so does one that the correction shuts."""
    from tiny_llm_amd.parts.moe import RoutedMoE
    g = torch.Generator().manual_seed(tokens)
    W, E, top, F = 80, 8, 3, 32
    tdt = torch.float32 if dtype == "float32" else torch.bfloat16
    names = {}
    for e in range(E):
        names[f"m.e{e}.gate"], names[f"m.e{e}.up"] = torch.randn(F, W, generator=g) / 8, torch.randn(F, W, generator=g) / 8
        names[f"m.e{e}.down"] = torch.randn(W, F, generator=g) / 5
    router = torch.zeros(E, W)
    router[:, :E] = torch.eye(E) * 0.5
    names["m.router"] = router
    names["m.correction"] = torch.tensor([0.0, 0.0, -9.0, -9.0, 0.375, 0.0, -0.25, 0.0])
    h = torch.randn(tokens, W, generator=g) * 0.5
    h[:, :E] = torch.stack([torch.randperm(E, generator=g).float() * 1.5 - 5.0 for _ in range(tokens)])
    w = {k: v.to(tdt) for k, v in names.items()}
    part = RoutedMoE("m", tdt, torch.device("cuda"), hidden_size=W, num_experts=E, top=top, intermediate_size=F, groups=4,
                     keep=2, activation="swiglu", score="sigmoid", correction=True, group_score="top2", normalize=False)
    part.bind({k: v.cuda() for k, v in w.items()})
    out = part.forward(h.to(tdt).cuda(), None, None)
    want = plain.moe(h.to(tdt).double(), {k[2:]: v.double() for k, v in w.items()},
                     {"router": {"top": top, "experts": E, "groups": {"count": 4, "keep": 2}}})
    err = (out.double().cpu() - want).abs().max() / want.abs().max()
    assert err < (1e-5 if dtype == "float32" else 3e-2)


def _stream(dec, runner, toks):
    """The residual stream after every layer run of one prompt (ahead of a pass's vector), and the vectors that the blocks
    added themselves."""
    from tiny_llm_amd.engine.step import StepEntry
    seen, fused = [], 0
    for layer in dec.layers:
        inner = layer.block.forward_chained

        def watch(x, *args, _inner=inner, **kw):
            nonlocal fused
            out = _inner(x, *args, **kw)
            row = out[0].clone()
            if kw.get("shift") is not None:
                row -= kw["shift"]
                fused += 1
            seen.append(row.double().cpu())
            return out
        layer.block.forward_chained = watch
    runner.step([StepEntry("s", toks, [len(toks) - 1])])
    return seen, fused


@pytest.mark.parametrize("name", ["A", "B", "loop_end"])
def test_stream_after_every_layer_run(name, tmp_path_factory):
    """Layer by layer against the plain model; the vector ahead of a pass rides in the block in front wherever there is one."""
    folder, cfg, w, reqs, ref, block = material(name, "float32", tmp_path_factory)
    runner = make_runner(folder, "float32", block, 64)
    toks = reqs["r2"][:30]
    want = []
    plain.forward(cfg, w, toks, trace=want)
    got, fused = _stream(runner.decoder, runner, toks)
    assert len(got) == len(want) == len(plain.runs(cfg))
    assert fused == cfg["loop"]["times"] - (1 if cfg["loop"]["start"] == 0 else 0)
    for i, (a, b) in enumerate(zip(got, want)):
        assert (a - b).abs().max() < 1e-4 * b.abs().max(), i
