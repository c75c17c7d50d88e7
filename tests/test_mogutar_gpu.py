"""The Mogutar architecture in the engine against the plain implementation of its equations
(tests/plain_mogutar.py): each mechanism alone, every way of cutting the work, pages and state slots
used again, captured steps, long decoding, generation through the entry point, and keys that a
crafted query singles out at the places where an index can be off by one."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import plain_mogutar as plain
import traces
from mogutar_util import CONFIGS, MIX_A, as_double, every_expert, make_folder, random_config, rounded, row_err
from util import random_tokens

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
# float32: everything is computed in 32 bits, what is left is the order of sums (the plain model itself, run in
# float32, differs from its float64 run by up to 8e-6 of a row on these models).  bfloat16: weights are rounded for the
# plain model too; the products' inputs and outputs are rounded in the engine only, the models are made tame so that
# this rounding is not amplified, and a row's limit grows with what rounding nothing but the products' operands does to
# it in the plain model (`round_operands`, the worst of four samples: 1e-2 as a rule, ten times that where a head's eight
# numbers happen to be small ahead of their norm), and every token uses every expert (a score that bfloat16 moves past its neighbour would
# otherwise choose another expert; the router's choices are compared in float32 and, with scores that are apart, at the
# part itself).  A fault of a mechanism (a key off by one, a lost state, a kept token left out) moves a row by its
# whole size in either precision.
TOL = {"float32": 1e-4, "bfloat16": 5e-2}
LENGTHS = {"A": [70, 133, 33, 200, 97, 64], "B": [1, 9, 40, 100, 150, 57], "odd": [31, 2, 77, 50], "wide": [50, 7, 101],
           "lightning": [40, 75, 130, 9], "parallel": [40, 75, 130, 9], "moe": [24, 121, 48, 5], "side": [24, 61, 5]}



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
        folder, w = make_folder(tmp_path_factory.mktemp(f"mogutar_{name}_{dtype}"), cfg, seed=11,
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


CASES = [(n, "float32") for n in ("lightning", "parallel", "moe", "side", "wide", "A", "B", "odd")] + \
        [(n, "bfloat16") for n in ("lightning", "parallel", "moe", "side", "wide", "A", "B")]


@pytest.mark.parametrize("name,dtype", CASES)
def test_whole_tail_portions(name, dtype, tmp_path_factory):
    """Each request alone: whole, its tail token by token (windows pass over decoded tokens), and in
    portions down to two tokens (one-layer models of each sublayer, then the mixed models)."""
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
    folder, w = make_folder(tmp_path_factory.mktemp("mogutar_odd_bf16"), cfg, seed=4, store=torch.bfloat16)
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
    narrower than values, windows from one position to more than the prompt and none, kept tokens on less and more than
    a page, rotated dims, YaRN, caps, taps, decays of one, groups of experts, layers without feed-forward, pages of 4 to
    32 tokens; mixed batches, portions and whole prompts in both precisions."""
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
    """Three layers with heads of the sizes a model of some billions of weights has (heads of 128, states of 128 x 64
    with shared B and C, a window that a prompt of 300 tokens leaves, experts of 64 hidden units): a whole prompt (the
    kernels for many rows), the same in portions, and a tail decoded token by token beside a second request."""
    from mogutar_util import layer, left, lightning, model, moe, parallel, right
    big = model(256, 1031, [
        layer(parallel(left(16, 4, 128, 128, 4, 130, 9, 64, (8.0, 128, 32.0, 1.0), 30.0, 500000.0, 128 ** -0.5),
                       right(16, 2, 128, 64, 4, 2), 0.8, 1.1), moe(16, 4, 64, (4, 2))),
        layer(lightning(8, 128, 128), moe(12, 3, 32)),
        layer(lightning(4, 64, 256), moe(8, 2, 64, (2, 1))),
    ], side=64)
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
    """One to four tokens: the convolutions reach back into zeros, the state starts empty, a softmax holds one key."""
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
    """Several hundred single-token steps: the states and the convolutions' inputs are carried from step to step,
    every page edge is crossed by decoded tokens, the windows leave the first tokens behind and keep the kept ones."""
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
    """bin/tiny_llm serves a Mogutar folder as it serves any other (config.json chooses the model);
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
def _paged_kv(rows: torch.Tensor, table, block, n_blocks, dtype):
    """rows [n, kv_heads, d] laid into pages [n_blocks, kv_heads, block, d] at the blocks `table` names; NaN elsewhere."""
    n, g, d = rows.shape
    pages = torch.full((n_blocks, g, block, d), float("nan"), dtype=dtype, device="cuda")
    for j in range(n):
        pages[table[j // block], :, j % block] = rows[j].to(dtype)
    return pages


def _attend(kernel, qd, k_pages, v_pages, bt, pos_dev, heads, kvh, d, scale, window, keep, cap, out_scale=1.0):
    """Every row of qd a request of its own over the same pages, by the named attention kernel."""
    from tiny_llm_amd.kernels import ops
    T, dtype = qd.shape[0], qd.dtype
    out = torch.empty(T, heads * d, dtype=dtype, device="cuda")
    tables = bt.repeat(T, 1).contiguous()
    each = torch.arange(T, dtype=torch.int32, device="cuda")
    opts = {"keep": keep, "softcap": cap, "out_scale": out_scale}
    if kernel.startswith("general"):
        return ops.paged_attention(qd, k_pages, v_pages, bt, torch.zeros_like(each), pos_dev, out, heads, kvh, d, scale, window, **opts)
    if "float32" in kernel and "many rows" in kernel:
        reps = -(-1024 // (T * kvh)) + 1
        n_t = T * reps
        big = torch.empty(n_t, heads * d, dtype=dtype, device="cuda")
        tiles = (torch.arange(n_t, dtype=torch.int32, device="cuda"),) * 2 + (torch.ones(n_t, dtype=torch.int32, device="cuda"),)
        ops.attention_f32(qd.repeat(reps, 1), k_pages, v_pages, bt.repeat(n_t, 1).contiguous(), tiles, pos_dev.repeat(reps),
                          big, heads, kvh, d, scale, window, **opts)
        assert all(torch.equal(big[:T], big[r * T:(r + 1) * T]) for r in range(1, reps))
        return big[:T]
    if "float32" in kernel:
        chunks = -(-bt.shape[1] * k_pages.shape[2] // ops.F32_CHUNK_KEYS) if "chunks" in kernel else 1
        part = torch.empty(chunks * T * heads * (d + 2), device="cuda") if chunks > 1 else None
        return ops.attention_f32(qd, k_pages, v_pages, tables, None, pos_dev, out, heads, kvh, d, scale, window, chunks, part, **opts)
    splits = 3 if "split" in kernel else 1
    part = torch.empty(splits * T * heads * (d + 2), device="cuda") if splits > 1 else None
    if "prompt" in kernel:
        return ops.flash_prefill(qd, k_pages, v_pages, tables, (each, each.clone(), torch.ones_like(each)), pos_dev, out, heads,
                                 kvh, d, scale, window, 4, splits, part, **opts)
    return ops.flash_attention(qd, k_pages, v_pages, tables, None, pos_dev, out, heads, kvh, d, scale, window, splits, part, **opts)


ATTENTION_KERNELS = ["general float32", "general bfloat16", "matrix cores float32", "matrix cores float32, chunks",
                     "matrix cores float32, many rows", "matrix cores bfloat16", "matrix cores bfloat16, split keys",
                     "matrix cores bfloat16, prompt", "matrix cores bfloat16, prompt, split keys"]


@pytest.mark.parametrize("kernel", ATTENTION_KERNELS)
@pytest.mark.parametrize("window,keep,cap", [(40, 6, 0.0), (1, 1, 20.0), (17, 70, 12.0), (64, 64, 0.0), (150, 3, 20.0), (96, 0, 9.0),
                                             (5, 130, 0.0), (1000, 8, 15.0), (0, 0, 20.0)])
def test_window_with_kept_tokens_finds_one_key(kernel, window, keep, cap):
    """One query per place of interest is aligned with one key (and scaled so that this score stands out): the result
    must be that key's value.  Keys at the window's first place, among the kept tokens (the first, the last), the query's
    own position, far keys; the keys just OUTSIDE (the last one the window has left, the first one that is not kept) and
    the one behind the query are louder still, and the mask must hide them.  Window 0 is no window at all."""
    dtype = torch.float32 if "float32" in kernel else torch.bfloat16
    g = torch.Generator().manual_seed(5)
    n, d, block, heads, kvh = 700, 32, 16, 6, 2
    keys = torch.randn(n, kvh, d, generator=g)
    keys = keys / keys.norm(dim=-1, keepdim=True)
    vals = torch.randn(n, kvh, d, generator=g)
    table = torch.randperm(64, generator=g)[: -(-n // block)].tolist()
    k_pages, v_pages = _paged_kv(keys, table, block, 64, dtype), _paged_kv(vals, table, block, 64, dtype)
    first = lambda pos: max(0, pos - window + 1) if window else 0
    seen = lambda pos: sorted(set(range(first(pos), pos + 1)) | set(range(min(keep, pos + 1))))
    places = {699, 650, 640, 639, 400, 257, 256, 255, 199, 130, 129, 128, 71, 70, 64, 63, 48, 31, 16, 15, 7, 6, 1, 0, window,
              window + keep, window + keep - 1, keep}
    cases = sorted({(pos, key) for pos in places if 0 <= pos < n
                    for key in (first(pos), pos, min(first(pos) + 1, pos), 0, min(max(keep - 1, 0), pos), seen(pos)[len(seen(pos)) // 2])
                    if key in seen(pos)})
    T = len(cases)
    q = torch.zeros(T, heads, d)
    for i, (pos, key) in enumerate(cases):
        vis = seen(pos)
        for h in range(heads):
            kv = h // (heads // kvh)
            # head 0 aims at the case's key, the others at keys of their own among the visible ones
            target = key if h == 0 else vis[(vis.index(key) + 3 * h) % len(vis)]
            q[i, h] = 30.0 * keys[target, kv]
            for hidden in (pos + 1, first(pos) - 1, keep):       # would win if they were seen
                if 0 <= hidden < n and hidden not in vis:
                    q[i, h] += 50.0 * keys[hidden, kv]
    pos_dev = torch.tensor([c[0] for c in cases], dtype=torch.int32, device="cuda")
    bt = torch.tensor([table + [0] * (64 - len(table))], dtype=torch.int32, device="cuda")
    out = _attend(kernel, q.reshape(T, heads * d).to(dtype).cuda(), k_pages, v_pages, bt, pos_dev, heads, kvh, d, 0.9, window,
                  keep, cap, 0.75)
    kr, vr, qr = keys.to(dtype).double(), vals.to(dtype).double(), q.to(dtype).double()
    out = out.double().cpu().reshape(T, heads, d)
    for i, (pos, _) in enumerate(cases):
        vis = torch.tensor(seen(pos))
        for h in range(heads):
            kv = h // (heads // kvh)
            s = kr[vis, kv] @ qr[i, h] * 0.9
            want = torch.softmax(plain.softcap(s, cap) if cap else s, dim=-1) @ vr[vis, kv] * 0.75
            assert torch.isfinite(out[i, h]).all()
            assert (out[i, h] - want).abs().max() < (3e-5 if dtype == torch.float32 else 2e-2), (pos, h)


@pytest.mark.parametrize("kernel", ["general float32", "matrix cores float32", "matrix cores bfloat16, prompt"])
@pytest.mark.parametrize("window,keep", [(24, 5), (100, 70), (3, 1), (64, 20)])
def test_windowed_attention_of_a_prompts_portion(kernel, window, keep):
    """A portion of a prompt behind cached tokens, cut in the middle of a window and of a page: tiles that hold
    several tokens whose windows differ; the pages between the kept tokens and the first window are NaN, as pages that
    were given back may be."""
    from tiny_llm_amd.kernels import ops
    dtype = torch.float32 if "float32" in kernel else torch.bfloat16
    g = torch.Generator().manual_seed(8)
    n, d, block, heads, kvh, start, cap = 390, 32, 16, 4, 2, 257, 6.0
    keys, vals = torch.randn(n, kvh, d, generator=g) * 1.5, torch.randn(n, kvh, d, generator=g)
    q = torch.randn(n - start, heads, d, generator=g) * 1.5
    table = torch.randperm(32, generator=g)[: -(-n // block)].tolist()
    k_pages, v_pages = _paged_kv(keys, table, block, 32, dtype), _paged_kv(vals, table, block, 32, dtype)
    for b in range(-(-keep // block), max(0, start - window + 1) // block):
        k_pages[table[b]] = v_pages[table[b]] = float("nan")
    T = n - start
    pos_dev = torch.arange(start, n, dtype=torch.int32, device="cuda")
    bt = torch.tensor([table + [0] * (32 - len(table))], dtype=torch.int32, device="cuda")
    out = torch.empty(T, heads * d, dtype=dtype, device="cuda")
    qd = q.reshape(T, heads * d).to(dtype).cuda()
    width, opts = 16 // (heads // kvh), {"keep": keep, "softcap": cap}
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
    kr, vr, qr = keys.to(dtype).double(), vals.to(dtype).double(), q.to(dtype).double()
    allowed = plain.window_with_first(torch.arange(n), window, keep)[start:]
    s = torch.einsum("ihd,jhd->hij", qr, kr.repeat_interleave(heads // kvh, 1)) * d ** -0.5
    s = plain.softcap(s, cap).masked_fill(~allowed[None], float("-inf"))
    want = torch.einsum("hij,jhv->ihv", torch.softmax(s, -1), vr.repeat_interleave(heads // kvh, 1))
    got = out.double().cpu().reshape(T, heads, d)
    assert (got - want).abs().max() < (2e-5 if dtype == torch.float32 else 3e-2)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("dim,vdim,rot,taps,yarn", [(24, 16, 8, 3, (4.0, 64.0, 16.0, 1.0)), (16, 40, 16, 4, None), (6, 11, 2, 2, None),
                                                    (80, 8, 0, 6, None), (8, 8, 4, 1, (1.5, 2048.0, 32.0, 1.0))])
def test_conv_attn_prepare(dtype, dim, vdim, rot, taps, yarn):
    """Bias, the short convolution over time on q, k and v with the request's saved inputs, the norm per head with its
    weights and then the rotation (with YaRN's frequencies and magnitude); three requests of unequal length in state slots
    out of order, cut into steps of several tokens and of single ones (which bring the saved inputs up to date themselves)."""
    from tiny_llm_amd.engine.step import tile_lists
    from tiny_llm_amd.kernels import ops
    from tiny_llm_amd.parts.rotary import angle_tables
    g = torch.Generator().manual_seed(3)
    H, G, block, eps = 4, 2, 4, 1e-5
    D = -(-max(dim, vdim) // 16) * 16
    qc, kc, vc = H * dim, G * dim, G * vdim
    channels = qc + kc + vc
    bias, head_w = torch.randn(channels, generator=g), 1.0 + 0.3 * torch.randn(2 * dim, generator=g)
    conv_w = torch.randn(channels, taps, generator=g)
    lens, slots = [9, 5, 31], [2, 0, 3]
    ps = [torch.randn(n, channels + 3, generator=g) for n in lens]
    want = []
    for p in ps:
        a = plain.causal_conv(p[:, :channels].double() + bias.double(), conv_w.double())
        n = a.shape[0]
        q = plain.rms_norm(a[:, :qc].reshape(n, H, dim), head_w[:dim].double(), eps)
        k = plain.rms_norm(a[:, qc:qc + kc].reshape(n, G, dim), head_w[dim:].double(), eps)
        if rot:
            spec = {"dims": rot, "base": 777.0}
            if yarn:
                spec["scaling"] = dict(zip(("factor", "original", "fast", "slow"), yarn))
            q, k = plain.rotate(q, torch.arange(n), spec), plain.rotate(k, torch.arange(n), spec)
        want.append((q, k, a[:, qc + kc:].reshape(n, G, vdim)))
    cos = sin = None
    if rot:
        cos, sin = angle_tables(rot, 777.0, 512, "cuda", yarn=yarn)
    off = 8
    state = torch.full((4, off + channels * (taps - 1) + 5), float("nan"), device="cuda")
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
        q = torch.full((1, T, H * D), float("nan"), dtype=dtype, device="cuda")
        where = torch.randperm(40, generator=g)[:T].to(torch.int32)
        runs = None if single else tuple(torch.tensor(x, dtype=torch.int32, device="cuda") for x in tile_lists(counts, ops.CONV_RUN))
        conv = ops.ShortConv(conv_w.cuda(), state, off, cu, sl, runs)
        ops.conv_attn_prepare(p, bias.cuda(), pos, cos, sin, where.cuda(), q[0], pages[0], pages[1], H, G, dim, vdim, conv,
                              head_w.cuda(), rot, "half", eps)
        if not single and taps > 1:
            ops.conv_state_update(p, 0, channels, state, off, cu, sl, taps, bias.cuda())
        t = 0
        for r in live:
            for i in range(at[r], at[r] + take[r]):
                wq, wk, wv = (x[i] for x in want[r])
                got = q[0, t].double().cpu().reshape(H, D)
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
        assert torch.isnan(state[1]).all() and not state[slots].isnan().any()


@pytest.mark.parametrize("experts,top,groups,keep", [(6, 2, 2, 1), (16, 3, 4, 2), (64, 6, 8, 3), (5, 5, 1, 1), (130, 4, 10, 1), (8, 2, 8, 3),
                                                     (1, 1, 1, 1), (12, 5, 4, 4)])
def test_router_with_sigmoid_scores_and_a_correction(experts, top, groups, keep):
    """Sigmoid scores; the correction decides (most corrected scores are negative) and stays out of the weights; a group is
    ranked by its two best experts together (groups of one expert: that one); the weights keep their size."""
    from tiny_llm_amd.kernels import ops
    g = torch.Generator().manual_seed(experts * 7 + top)
    T = 37
    z = torch.randn(T, experts, generator=g) * 2.0
    correction = torch.randn(experts, generator=g) * 0.7 - 1.5
    ids = torch.empty(T, top, dtype=torch.int32, device="cuda")
    wts = torch.empty(T, top, device="cuda")
    ops.moe_route(z.cuda(), ids, wts, groups, keep, 1.0, score="sigmoid", correction=correction.cuda(), group_top2=True,
                  normalize=False)
    s = torch.sigmoid(z.double())
    for t in range(T):
        want = plain.choose(s[t], correction.double(), top, groups, keep)
        assert ids[t].tolist() == want
        assert (wts[t].double().cpu() - s[t, want]).abs().max() < 1e-6


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("tokens", [5, 40, 700])
def test_experts_by_every_route(dtype, tokens):
    """The feed-forward part alone by each of its three routes (rows against their own expert, tiles of one expert's
    rows, runs of rows through the tiled product), with scores that are apart, so that both precisions choose alike, and
    a group that the correction shuts out."""
    from tiny_llm_amd.parts.moe import RoutedMoE
    g = torch.Generator().manual_seed(tokens)
    W, E, top, F = 64, 6, 2, 24
    tdt = torch.float32 if dtype == "float32" else torch.bfloat16
    names = {}
    for e in range(E):
        names[f"m.e{e}.gate"], names[f"m.e{e}.up"] = torch.randn(F, W, generator=g) / 8, torch.randn(F, W, generator=g) / 8
        names[f"m.e{e}.down"] = torch.randn(W, F, generator=g) / 5
    # the router reads the first channels: channel e of h is expert e's logit, so the choice is plain to see
    router = torch.zeros(E, W)
    router[:, :E] = torch.eye(E) * 0.5
    names["m.router"], names["m.correction"] = router, torch.tensor([0.0, 0.0, -9.0, -9.0, 0.25, 0.0])
    h = torch.randn(tokens, W, generator=g) * 0.5
    h[:, :E] = torch.stack([torch.randperm(E, generator=g).float() * 2.0 - 5.0 for _ in range(tokens)])    # logits 1 apart
    w = {k: v.to(tdt) for k, v in names.items()}
    part = RoutedMoE("m", tdt, torch.device("cuda"), hidden_size=W, num_experts=E, top=top, intermediate_size=F, groups=3,
                     keep=2, activation="swiglu", score="sigmoid", correction=True, group_score="top2", normalize=False)
    part.bind({k: v.cuda() for k, v in w.items()})
    out = part.forward(h.to(tdt).cuda(), None, None)
    wd = {k[2:]: v.double() for k, v in w.items()}
    want = plain.moe(h.to(tdt).double(), wd, {"router": {"top": top, "experts": E, "groups": {"count": 3, "keep": 2}}})
    err = (out.double().cpu() - want).abs().max() / want.abs().max()
    assert err < (1e-5 if dtype == "float32" else 3e-2)


def test_table_rows_behind_a_gelu():
    """gelu(gate) times the token's part of a table, in rows filled up with zeros."""
    from tiny_llm_amd.kernels import ops
    g = torch.Generator().manual_seed(2)
    T, dim, off, wide, width, V = 19, 12, 24, 16, 60, 50
    gate, table = torch.randn(T, wide, generator=g) * 2, torch.randn(V, width, generator=g)
    tokens = torch.randint(0, V, (T,), generator=g)
    for dtype, tol in ((torch.float32, 1e-5), (torch.bfloat16, 3e-2)):
        out = torch.full((T, wide), float("nan"), dtype=dtype, device="cuda")
        ops.gelu_table_rows(gate.cuda(), tokens.to(torch.int32).cuda(), table.to(dtype).cuda(), off, dim, out)
        want = plain.gelu_tanh(gate[:, :dim].double()) * table.to(dtype).double()[tokens, off:off + dim]
        assert (out[:, :dim].double().cpu() - want).abs().max() < tol and (out[:, dim:] == 0).all()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("T,W,dim", [(1, 64, 16), (8, 2048, 64), (9, 40, 12), (32, 128, 5), (17, 50, 8)])
def test_token_gate_for_few_rows(dtype, T, W, dim):
    """The gate's product, the gelu and the token's table row in one kernel, rows in groups of eight and rests of them."""
    from tiny_llm_amd.kernels import ops
    g = torch.Generator().manual_seed(T)
    wide, off, V = -(-dim // 8) * 8, 7, 50
    h, w = torch.randn(T, W, generator=g).to(dtype), (torch.randn(wide, W, generator=g) / W ** 0.5 * 2).to(dtype)
    table, tokens = torch.randn(V, off + dim + 3, generator=g).to(dtype), torch.randint(0, V, (T,), generator=g)
    out = torch.full((T, wide), float("nan"), dtype=dtype, device="cuda")
    ops.token_gate(h.cuda(), w.cuda(), tokens.to(torch.int32).cuda(), table.cuda(), off, dim, out)
    want = plain.gelu_tanh(h.double() @ w[:dim].double().T) * table.double()[tokens, off:off + dim]
    assert ((out[:, :dim].double().cpu() - want).abs() <= (1e-5 if dtype == torch.float32 else 2.0 ** -8) * (want.abs() + 1.0)).all()
    assert (out[:, dim:] == 0).all()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width,groups,kind,first,scale", [(96, 1, "sigmoid", False, 1.0), (96, 6, "silu", True, 0.7), (2000, 4, "silu", True, 1.3),
                                                           (7000, 1, "sigmoid", False, 0.5), (35, 5, "silu", False, 1.0),
                                                           (9000, 1, "silu", True, 1.1)])
def test_group_norm_gate(dtype, width, groups, kind, first, scale):
    """A gate ahead of the norm or behind it, norms over equal parts of a row, parts from seven numbers to thousands."""
    from tiny_llm_amd.kernels import ops
    g = torch.Generator().manual_seed(width)
    T, eps = 7, 1e-5
    o, gate, w = torch.randn(T, width, generator=g) * 2, torch.randn(T, width + 3, generator=g), torch.randn(width, generator=g)
    out = torch.empty(T, width, dtype=dtype, device="cuda")
    ops.group_norm_gate(o.cuda(), w.cuda(), gate.cuda()[:, :width], out, groups, eps, kind, first, scale)
    a = torch.sigmoid(gate[:, :width].double()) if kind == "sigmoid" else plain.silu(gate[:, :width].double())
    norm = lambda x: plain.unit_rms(x.reshape(T, groups, -1), eps).reshape(T, width)
    want = (norm(o.double() * a) if first else norm(o.double()) * a) * w.double() * scale
    assert ((out.double().cpu() - want).abs() <= (1e-5 if dtype == torch.float32 else 2.0 ** -8) * (want.abs() + 1.0)).all()


class _Ctx:
    def __init__(self, counts, slots):
        self.cu_seqlens_q = torch.tensor([0] + list(np.cumsum(counts)), dtype=torch.int32, device="cuda")
        self.req_of_token = torch.tensor([i for i, n in enumerate(counts) for _ in range(n)], dtype=torch.int32, device="cuda")
        self.state_slots = torch.tensor(slots, dtype=torch.int32, device="cuda")
        self.max_q_len, self.num_requests, self.counts = max(counts), len(counts), counts

    def attention_tiles(self, width):
        from tiny_llm_amd.engine.step import tile_lists
        return tuple(torch.tensor(t, dtype=torch.int32, device="cuda") for t in tile_lists(self.counts, width))


def _mixer(kind, sizes, dtype, W, eps):
    """(part, plain function, its sizes, weights by name)"""
    from tiny_llm_amd.parts.linear_recurrence import DecayedAttention, StateSpace
    if kind == "state_space":
        H, G, N, V, taps, ng = sizes
        part = StateSpace("m", dtype, torch.device("cuda"), hidden_size=W, num_heads=H, groups=G, state_dim=N, value_dim=V,
                          conv_taps=taps, norm_groups=ng, eps=eps)
        return part, plain.mamba2, {"heads": H, "groups": G, "state": N, "vdim": V, "conv": taps, "norm_groups": ng}
    H, N, V, decay = sizes
    part = DecayedAttention("m", dtype, torch.device("cuda"), hidden_size=W, num_heads=H, head_dim=N, value_dim=V, decay=decay, eps=eps)
    return part, plain.lightning, {"heads": H, "dim": N, "vdim": V, "decay": decay}


RECURRENT = [("state_space", (4, 2, 24, 16, 4, 2)), ("state_space", (3, 1, 5, 9, 3, 3)), ("state_space", (2, 2, 128, 64, 2, 1)),
             ("state_space", (6, 3, 200, 12, 6, 1)), ("state_space", (1, 1, 1, 4, 1, 4)), ("state_space", (8, 1, 48, 96, 4, 8)),
             ("decayed_attention", (3, 16, 24, [0.5, 0.999, 1.0])), ("decayed_attention", (2, 7, 5, [0.0, 0.9])),
             ("decayed_attention", (1, 256, 128, [0.97])), ("decayed_attention", (5, 64, 256, [0.3, 0.6, 0.9, 0.99, 0.999]))]


@pytest.mark.parametrize("kind,sizes", RECURRENT)
def test_recurrent_state_over_slots_and_tiny_portions(kind, sizes):
    """The recurrent mixers alone: three requests of unequal length in slots out of order, fed in portions of 1 to 70
    tokens (single tokens take the one-token kernel, steps with a long portion the chunked form), against the plain scan over each whole sequence; a slot of another
    request stays untouched.  The state is a slice of wider rows, as it is beside another branch."""
    g = torch.Generator().manual_seed(9)
    W, eps = 40, 1e-5
    part, fn, m = _mixer(kind, sizes, torch.float32, W, eps)
    w = {}
    for s in part.weights():
        t = torch.randn(*s.shape, generator=g)
        w[s.name] = t * (1.5 / W ** 0.5 if len(s.shape) == 2 and s.shape[-1] == W else 0.5)
    part.bind({k: v.cuda() for k, v in w.items()})
    lens, slots = [23, 9, 180], [2, 0, 3]
    hs = [torch.randn(n, W, generator=g) for n in lens]
    wd = {k[2:]: v.double() for k, v in w.items()}
    want = [fn(h.double(), wd, m, eps) for h in hs]
    width = part.state_spec().shape[0]
    rows = torch.full((4, width + 12), float("nan"), device="cuda")
    state = rows[:, 8:8 + width]
    for s in slots:
        state[s].zero_()
    at, got = [0, 0, 0], [[], [], []]
    sizes_ = [3, 1, 7, 2, 70, 5, 2, 16, 1, 33, 1, 1, 17, 1]
    k = 0
    while any(a < n for a, n in zip(at, lens)):
        live = [r for r in (2, 0, 1) if at[r] < lens[r]]             # batch order differs from slot order
        take = []
        for r in live:
            take.append(min(sizes_[k % len(sizes_)], lens[r] - at[r]))
            k += 1
        if k % 5 == 0:
            take = [1] * len(live)                                    # a step of single tokens
        h = torch.cat([hs[r][at[r]:at[r] + n] for r, n in zip(live, take)]).cuda()
        out = part.forward(h, _Ctx(take, [slots[r] for r in live]), None, state, None).cpu()
        o = 0
        for r, n in zip(live, take):
            got[r].append(out[o:o + n].clone())
            o += n
            at[r] += n
    for r in range(3):
        err = (torch.cat(got[r]).double() - want[r]).abs().max() / want[r].abs().max()
        assert err < 1e-4, (r, float(err))
    assert torch.isnan(rows[1]).all() and torch.isnan(rows[:, :8]).all() and torch.isnan(rows[:, 8 + width:]).all()


@pytest.mark.parametrize("kind,sizes", [("state_space", (8, 2, 128, 64, 4, 2)), ("decayed_attention", (4, 64, 64, [0.5, 0.9, 0.999, 1.0]))])
def test_long_memory_of_a_recurrence(kind, sizes):
    """A prompt of 600 tokens in one step, in portions of 256, 200 and 144 and by single tokens behind 500: the same
    result to float32's rounding, whatever the cut, also where nothing is forgotten (a decay of one)."""
    g = torch.Generator().manual_seed(4)
    W, eps, n = 64, 1e-5, 600
    part, fn, m = _mixer(kind, sizes, torch.float32, W, eps)
    w = {s.name: torch.randn(*s.shape, generator=g) * (1.5 / W ** 0.5 if len(s.shape) == 2 and s.shape[-1] == W else 0.5)
         for s in part.weights()}
    if kind == "state_space":
        w["m.A_log"], w["m.dt_bias"] = torch.full((sizes[0],), -6.0), torch.zeros(sizes[0])     # forgets over hundreds of tokens
    part.bind({k: v.cuda() for k, v in w.items()})
    h = torch.randn(n, W, generator=g)
    want = fn(h.double(), {k[2:]: v.double() for k, v in w.items()}, m, eps)
    for cuts in ([600], [256, 200, 144], [500] + [1] * 100):
        state = torch.zeros(1, part.state_spec().shape[0], device="cuda")
        got, at = [], 0
        for c in cuts:
            got.append(part.forward(h[at:at + c].cuda(), _Ctx([c], [0]), None, state, None).cpu().clone())
            at += c
        err = (torch.cat(got).double() - want).abs().max() / want.abs().max()
        assert err < 1e-4, (cuts[:3], float(err))


@pytest.mark.parametrize("name", ["lightning", "parallel"])
def test_generation_of_models_with_one_kind_of_memory(name, tmp_path_factory):
    """A model without any paged cache (state slots alone), and one with a window and states, through the scheduler with
    more requests than slots, captured steps and chained decode steps."""
    folder, cfg, w, reqs, ref, block = material(name, "float32", tmp_path_factory)
    from tiny_llm_amd import Engine, SamplingParams
    prompts = [reqs["r0"][:17], reqs["r1"][:61], reqs["r3"][:3]]
    eng = Engine(folder, dtype="float32", kv_block_size=block, max_num_seqs=2, max_num_batched_tokens=64, max_model_len=256)
    out = eng.generate(prompts, SamplingParams.greedy(24, ignore_eos=True))
    for p, o in zip(prompts, out):
        seq = list(p)
        for _ in range(24):
            seq.append(int(plain.forward(cfg, w, seq)[-1].argmax()))
        assert o == seq[len(p):]
    steps, peak = traces.mixed(reqs, seed=5)
    runner = make_runner(folder, "float32", block, peak)
    for use_graph in (False, True, True):
        check(replay(runner, steps, use_graph=use_graph), steps, ref, TOL["float32"])
        assert all_free(runner)
