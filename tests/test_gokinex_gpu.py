"""The Gokinex decoder in the engine against the plain implementation (``plain_gokinex``).

Small configurations of their own (``gokinex_util``: other sizes, head counts, layer orders, states, expert counts
and constants than any served model; also values that are equal, 1 or absent), seeded weights with spread-out
scores.  Every schedule - whole prompts, token-by-token decoding, portions down to two tokens, mixed batches on a
pool so small that pages and seats come back - must give the logits of the plain whole-sequence forward pass, in
both number formats.
"""
import copy
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import gokinex_util as U
import plain_gokinex as plain
import replay_util as R
from kv_cache_optimization_for_llm_amd.engine.engine import Engine, EngineOptions
from kv_cache_optimization_for_llm_amd.engine.runner import LLM, ServeOptions

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    base = tmp_path_factory.mktemp("gokinex")
    return {name: (cfg, *U.write_model(str(base / name), cfg, seed)) for name, (cfg, seed) in U.CONFIGS.items()}


def engine_for(folder, dtype, **kw):
    opts = dict(dtype=dtype, page_size=16, cache_tokens=1024, max_seqs=4, max_seq_len=512, max_batch_tokens=1024,
                use_graphs=False)
    opts.update(kw)
    return Engine(folder, EngineOptions(**opts))


REQUESTS = {"A": [1, 2, 9, 40, 77], "B": [3, 33, 70], "C": [1, 5, 47, 150], "D": [2, 44, 101], "E": [1, 2, 35, 64]}


def requests_for(name, cfg):
    return {f"{name}{i}": U.prompt(cfg, n, 100 * i + n) for i, n in enumerate(REQUESTS[name])}


def check(eng, cfg, state, reqs, steps, dtype, what, tolerance=None):
    rows, routes = U.run_steps(eng, steps, cfg)
    U.assert_rows(rows, U.expected_rows(cfg, state, reqs, dtype, routes), dtype, what, tolerance)
    eng.cache.check()
    return rows


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(U.CONFIGS))
def test_whole_prompts_and_the_first_tokens(name, dtype, models, gpu):
    cfg, folder, state = models[name]
    reqs = requests_for(name, cfg)
    eng = engine_for(folder, dtype)
    rows = check(eng, cfg, state, reqs, R.whole(reqs), dtype, "whole")
    assert len(rows) == sum(len(t) for t in reqs.values())
    assert eng.cache.free_seats == 4


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(U.CONFIGS))
def test_prefill_against_token_by_token_decoding(name, dtype, models, gpu):
    """Most of a request in one step, the rest one token at a time; and a request decoded from its very first
    token on."""
    cfg, folder, state = models[name]
    reqs = {k: v for k, v in requests_for(name, cfg).items() if len(v) > 30}
    eng = engine_for(folder, dtype)
    check(eng, cfg, state, reqs, R.tail_decoded(reqs, tail=34 if name == "E" else 30), dtype, "decode")
    first = {"solo": U.prompt(cfg, 60, 9)}
    check(eng, cfg, state, first, R.tail_decoded(first, tail=59), dtype, "decode from the first token")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("sizes", [(2,), (7, 16, 5, 2, 33, 3, 64, 2), (17, 1, 1, 30), (24, 23, 1, 64, 65)])
@pytest.mark.parametrize("name", ["A", "B", "C", "D"])
def test_portions_of_any_size(name, sizes, dtype, models, gpu):
    """Down to two tokens (fewer than a convolution reads), on both sides of where a recurrence's kernels change."""
    cfg, folder, state = models[name]
    reqs = {k: v for k, v in requests_for(name, cfg).items() if len(v) > 8}
    eng = engine_for(folder, dtype, page_size=8 if name == "A" else 16)
    check(eng, cfg, state, reqs, R.chunked(reqs, sizes), dtype, f"portions {sizes}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name, seed", [("A", 0), ("B", 1), ("C", 2), ("C", 3), ("D", 4), ("E", 5)])
def test_mixed_batches_on_a_small_pool_reuse_pages_and_seats(name, seed, dtype, models, gpu):
    """Pages with other requests' keys, seats with other requests' states, convolution inputs and last tokens."""
    cfg, folder, state = models[name]
    lengths = [40, 3, 90, 25, 61, 2, 130, 47, 33]
    reqs = {f"m{i}": U.prompt(cfg, n, 7 * i + seed) for i, n in enumerate(lengths)}
    steps = R.mixed(reqs, seed=seed, max_live=3)
    pool = R.max_live_tokens(steps, unit=16)
    eng = engine_for(folder, dtype, cache_tokens=pool, max_seqs=3, max_seq_len=192)
    rows = check(eng, cfg, state, reqs, steps, dtype, "mixed")
    assert len(rows) == sum(lengths)
    stats = eng.cache.stats()
    assert stats["pages_reused"] > 0 and stats["running"] == 0
    assert all(g.free_pages() == g.num_pages for g in eng.cache.groups)


def test_one_seat_taken_again_and_again(models, gpu):
    cfg, folder, state = models["A"]
    reqs = {f"s{i}": U.prompt(cfg, n, 40 + i) for i, n in enumerate([50, 7, 31, 2, 1, 20])}
    eng = engine_for(folder, "float32", max_seqs=1, cache_tokens=64, max_seq_len=64)
    check(eng, cfg, state, reqs, R.chunked(reqs, (9, 4)), "float32", "one seat")


@pytest.mark.parametrize("name", ["A", "C"])
def test_a_request_alone_and_in_a_batch_give_the_same_logits(name, models, gpu):
    """Logits of a (request, position) do not depend on the cut, the batch, the pages or the seat, beyond
    rounding."""
    cfg, folder, state = models[name]
    reqs = {f"b{i}": U.prompt(cfg, n, 50 + i) for i, n in enumerate([70, 21, 44])}
    eng = engine_for(folder, "float32")
    alone = U.run_steps(eng, R.whole(reqs))
    together = U.run_steps(eng, R.mixed(reqs, seed=4, max_live=3, chunk_sizes=(2, 3, 16, 9)))
    assert alone.keys() == together.keys()
    for key in alone:
        assert U.row_error(together[key], alone[key]) <= 2e-5, str(key)


@pytest.mark.parametrize("name, dtype", [("A", "float32"), ("C", "bfloat16")])
def test_long_decoding(name, dtype, models, gpu):
    """Two to three hundred single-token steps behind a short prompt, two requests beside each other."""
    cfg, folder, state = models[name]
    n = 300 if name == "A" else 200
    reqs = {"l0": U.prompt(cfg, n, 1), "l1": U.prompt(cfg, n - 11, 2)}
    steps = [{"step": 0, "entries": [{"id": r, "tokens": t[:12], "want": [11]} for r, t in reqs.items()], "end": []}]
    for i in range(12, n):
        ent = [{"id": r, "tokens": t[i:i + 1], "want": [0]} for r, t in reqs.items() if i < len(t)]
        steps.append({"step": i, "entries": ent, "end": [r for r, t in reqs.items() if i == len(t) - 1]})
    check(engine_for(folder, dtype), cfg, state, reqs, steps, dtype, "long decoding")


def _sharp(cfg, gain):
    """Queries scaled up, so that every softmax is sharp: one key carries nearly all of a map's weight, and a key
    wrongly seen, wrongly hidden or taken from the other map moves a row by far more than rounding.  Slow decays, so
    that a state reaches back over whole portions."""
    def edit(state):
        for name in state:
            if name.endswith((".mix.q", ".mix.q.b")):
                state[name] = (state[name].float() * gain).to(torch.bfloat16)
            elif name.endswith(".A_log"):
                state[name] = torch.full_like(state[name], -4.0)
    return edit


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name, gain", [("A", 6.0), ("C", 3.0), ("D", 4.0)])
def test_sharp_scores_far_keys_page_borders_and_long_states(name, gain, dtype, tmp_path, gpu):
    """The first keys of a request from hundreds of positions away, keys on both sides of every page's border, states
    that remember whole portions, in whole prompts, in portions that start and end at a page's or a chunk's border and
    one off it, decoded one by one and side by side."""
    cfg = U.CONFIGS[name][0]
    if dtype == "bfloat16":
        gain = min(gain, 1.5)          # (in 16 bits a softmax four times as sharp turns rounding into other keys)
    folder, state = U.write_model(str(tmp_path / "sharp"), cfg, 21, edit=_sharp(cfg, gain))
    reqs = {"e0": U.prompt(cfg, 75, 1), "e1": U.prompt(cfg, 410, 2)}
    eng = engine_for(folder, dtype)
    tol = 5e-4                         # (sharp softmaxes multiply the rounding of what they read)
    check(eng, cfg, state, reqs, R.whole(reqs), dtype, "whole", tol)
    check(eng, cfg, state, reqs, R.chunked(reqs, (16, 15, 2, 33, 14, 48, 1, 31, 64, 63, 65)), dtype, "cuts at borders", tol)
    check(eng, cfg, state, {"e0": reqs["e0"]}, R.tail_decoded({"e0": reqs["e0"]}, tail=60), dtype, "decoded over page borders", tol)
    check(eng, cfg, state, {"e1": reqs["e1"]}, R.tail_decoded({"e1": reqs["e1"]}, tail=20), dtype, "decoded far from the start", tol)
    side = {f"s{i}": U.prompt(cfg, n, 30 + i) for i, n in enumerate([40, 65, 110, 129])}
    check(eng, cfg, state, side, R.mixed(side, seed=2, max_live=4, chunk_sizes=(31, 33, 17)), dtype, "side by side", tol)


def test_a_mistake_in_the_plain_model_shows(models, gpu):
    """The comparison sees each mechanism: the engine's rows against plain models with one thing wrong."""
    cfg, folder, state = models["C"]
    reqs = {"w": U.prompt(cfg, 60, 3)}
    rows = U.run_steps(engine_for(folder, "float32"), R.whole(reqs))

    def error(c, s):
        want = plain.forward(c, s, reqs["w"]).numpy()
        return max(U.row_error(rows["w", p], want[p]) for p in range(60))

    def with_weights(match, f):
        return {k: f(v.float()).to(v.dtype) if match(k) else v for k, v in state.items()}

    def with_config(f):
        c = copy.deepcopy(cfg)
        f(c)
        return c
    assert error(cfg, state) <= U.TOLERANCE["float32"]
    flat = torch.zeros_like
    for what, c, s in [
            ("the pairs' table", with_config(lambda c: c["embedding"]["bigram"].update(mul_prev=0)), state),
            ("the first token's row", cfg, with_weights(lambda k: k == "bigram", lambda v: torch.cat([v[:-1], 0 * v[-1:]]))),
            ("a norm's slope", cfg, with_weights(lambda k: k.endswith("norm1b.alpha"), lambda v: v * 1.3)),
            ("a norm's bias", cfg, with_weights(lambda k: k.endswith("norm2b.b"), flat)),
            ("a projection's bias", cfg, with_weights(lambda k: k.endswith("mix.o.b"), flat)),
            ("the keys' bias", cfg, with_weights(lambda k: k.endswith("mix.q.b"), flat)),
            ("the second map's weight", cfg, with_weights(lambda k: k.endswith("lq2"), flat)),
            ("the frequencies' scaling", with_config(lambda c: [c["layers"][i]["mixer"]["rot"].pop("scaling") for i in (0, 2, 5)]), state),
            ("the convolution's bias", cfg, with_weights(lambda k: k.endswith("conv.b"), flat)),
            ("the skip", cfg, with_weights(lambda k: k.endswith(".D"), flat)),
            ("the step's bias", cfg, with_weights(lambda k: k.endswith("dt_bias"), flat)),
            ("the norm's parts", with_config(lambda c: c["layers"][1]["mixer"].update(norm_groups=1)), state),
            ("the shared expert's gate", cfg, with_weights(lambda k: k.endswith("shared.sg"), flat))]:
        assert error(c, s) > 5e-3, what


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_the_trace_runner_replays_a_mixed_schedule(dtype, models, tmp_path, gpu):
    """``bin/trace_run`` (graphs and all) on a mixed schedule."""
    cfg, folder, state = models["C"]
    reqs = {f"t{i}": U.prompt(cfg, n, 11 + i) for i, n in enumerate([30, 2, 75, 18, 52])}
    steps = R.mixed(reqs, seed=5, max_live=4)
    pool = R.max_live_tokens(steps)
    rows = R.run_trace(folder, dtype, steps, pool, str(tmp_path / "out"), cfg["vocab"])
    assert R.cache_stats(str(tmp_path / "out"))["pages_reused"] > 0
    if dtype == "float32":
        U.assert_rows(rows, U.expected_rows(cfg, state, reqs, dtype), dtype, "trace")
    else:       # (16 bits may tip a close choice of experts: the same engine in this process is what must come out)
        same = U.run_steps(engine_for(folder, dtype, cache_tokens=pool, max_seq_len=pool, max_batch_tokens=8192, use_graphs=True), steps)
        for key in same:
            np.testing.assert_array_equal(rows[key], same[key], err_msg=str(key))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "C"])
def test_greedy_generation_through_the_entry_point(name, dtype, models, gpu):
    """Scheduler, sampler and run-ahead (pairs of tokens of which one is still on the device)."""
    cfg, folder, state = models[name]
    prompts = [U.prompt(cfg, n, 3 + n) for n in (1, 12, 37, 64, 5, 90)]
    llm = LLM(folder, EngineOptions(dtype=dtype, max_seqs=3, max_seq_len=160, cache_tokens=480),
              ServeOptions(chunk_size=16, max_batch_tokens=48))
    got, reasons = llm.generate(prompts, max_new_tokens=24, ignore_eos=True, return_reasons=True)
    assert reasons == ["length"] * len(prompts)
    for p, g in zip(prompts, got):
        assert len(g) == 24
        logits = plain.forward(cfg, state, list(p) + list(g)).numpy()
        for i, tok in enumerate(g):
            row = logits[len(p) + i - 1]
            slack = (1e-3 if dtype == "float32" else 0.1) * (row.max() - row.mean())
            assert row[tok] >= row.max() - slack, f"token {i} behind a prompt of {len(p)} is not the best one"
    llm.engine.cache.check()
    assert llm.engine.cache.free_seats == 3


def test_a_preempted_request_starts_again_from_an_empty_state(models, gpu):
    """A pool too small for what is admitted: whoever is sent back to the queue computes its tokens again in another
    seat, from a state, convolution inputs and a previous token that are its own."""
    cfg, folder, state = models["A"]
    prompts = [U.prompt(cfg, n, 60 + n) for n in (30, 26, 22, 28)]
    big = LLM(folder, EngineOptions(dtype="float32", max_seqs=4, max_seq_len=96, cache_tokens=4 * 96)).generate(
        prompts, max_new_tokens=30, ignore_eos=True)
    llm = LLM(folder, EngineOptions(dtype="float32", max_seqs=4, max_seq_len=96, cache_tokens=128))
    assert llm.generate(prompts, max_new_tokens=30, ignore_eos=True) == big
    assert llm.last_runner.scheduler.preemptions > 0


@pytest.fixture
def eager_steps_see_the_context_bucket(monkeypatch):
    """A graph cuts the keys into ranges by its context bucket, an eager step by the context it sees: eager steps
    that are given the bucket too are what a replay has to equal bit for bit."""
    import kv_cache_optimization_for_llm_amd.engine.engine as engine_module
    from kv_cache_optimization_for_llm_amd.engine.graphs import context_bucket
    plain_build = engine_module.build_batch

    def build_with_bucket(*args, **kwargs):
        batch = plain_build(*args, **kwargs)
        batch.max_context = context_bucket(batch.max_context)
        return batch
    monkeypatch.setattr(engine_module, "build_batch", build_with_bucket)


@pytest.mark.parametrize("name", ["A", "C", "D"])
def test_decode_steps_from_graphs_equal_eager_steps(name, models, eager_steps_see_the_context_bucket, gpu):
    """Replay after replay: states, convolution inputs and the token before are carried by the graph's own kernels."""
    cfg, folder, state = models[name]
    reqs = {f"g{i}": U.prompt(cfg, n, 31 + i) for i, n in enumerate([48, 80])}
    steps = R.tail_decoded(reqs, tail=20)
    eager = U.run_steps(engine_for(folder, "bfloat16"), steps)
    eng = engine_for(folder, "bfloat16", use_graphs=True)
    assert eng.graphs is not None
    replayed = U.run_steps(eng, steps)
    assert eng.graphs.replays > 0
    for key in eager:
        np.testing.assert_array_equal(eager[key], replayed[key], err_msg=str(key))


def test_portion_steps_from_graphs_equal_eager_steps(models, eager_steps_see_the_context_bucket, gpu):
    """Portions of two requests beside a decoded token whose shape comes back, four times over."""
    cfg, folder, state = models["C"]
    steps = []
    for rep in range(4):
        reqs = {f"a{rep}": U.prompt(cfg, 112, 60 + rep), f"b{rep}": U.prompt(cfg, 32, 70 + rep), f"c{rep}": U.prompt(cfg, 4, 80 + rep)}
        cuts = {f"a{rep}": 28, f"b{rep}": 8, f"c{rep}": 1}
        for k in range(4):
            steps.append({"step": len(steps), "entries": [{"id": rid, "tokens": toks[k * cuts[rid]:(k + 1) * cuts[rid]],
                                                           "want": [cuts[rid] - 1]} for rid, toks in reqs.items()],
                          "end": list(reqs) if k == 3 else []})
    eager = U.run_steps(engine_for(folder, "bfloat16"), steps)
    eng = engine_for(folder, "bfloat16", use_graphs=True)
    replayed = U.run_steps(eng, steps)
    assert eng.portion_graphs is not None and eng.portion_graphs.replays > 0
    for key in eager:
        np.testing.assert_array_equal(eager[key], replayed[key], err_msg=str(key))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_contiguous_cache_mode_gives_the_logits_of_the_plain_model(dtype, models, gpu):
    cfg, folder, state = models["C"]
    reqs = {f"c{i}": U.prompt(cfg, n, 90 + i) for i, n in enumerate([70, 33, 121])}
    eng = engine_for(folder, dtype, cache_mode="contiguous", cache_tokens=4 * 128, max_seq_len=128)
    check(eng, cfg, state, reqs, R.mixed(reqs, seed=9, max_live=3), dtype, "contiguous")


def test_the_serving_process_serves_the_model(models, tmp_path, gpu):
    """``cli.client`` starts ``cli.serve`` on the model folder: every sequence emits its budget."""
    cfg, folder, state = models["A"]
    out = tmp_path / "paged.json"
    env = dict(os.environ, IGNORE_EOS="1", ORCA_POLICY="oracle", PYTHONPATH=ROOT)
    cmd = [sys.executable, "-m", "kv_cache_optimization_for_llm_amd.cli.client", folder, "5", "--prompt-len", "37",
           "--max-new-tokens", "10", "--num-seqs", "2", "--out", str(out), "--", "--dtype", "float32",
           "--cache-mode", "paged", "--max-seqs", "4", "--max-seq-len", "64", "--cache-tokens", "384",
           "--chunk-size", "8", "--max-batch-tokens", "24"]
    proc = subprocess.run(cmd, env=env, cwd=ROOT, capture_output=True, text=True, timeout=110)
    assert proc.returncode == 0, proc.stdout + proc.stderr
    r = json.load(open(out))
    assert r["status"] == "ok" and r["sequences_done"] == 10 and r["tokens"] == 100
    assert r["count_mismatches"] == 0 and r["budget_mismatches"] == 0 and r["errors"] == []


def test_the_sweep_command_runs_a_configuration_file_of_this_architecture(models, tmp_path, gpu):
    from kv_cache_optimization_for_llm_amd.cli import sweep
    cfg, folder, state = models["C"]
    out = tmp_path / "sweep.jsonl"
    assert sweep.main(["--shapes", os.path.join(folder, "config.json"), "--batches", "3", "--cache-modes", "paged",
                       "--prompt-len", "40", "--prompt-min", "5", "--workload", "mixed", "--new-tokens", "9",
                       "--max-seqs", "2", "--out", str(out)]) == 0
    line, = [json.loads(l) for l in out.read_text().splitlines()]
    assert line["requests_done"] == 3 and line["tokens_emitted"] == 27 and line["finish_reasons"] == {"length": 3}
    assert line["pages_reused"] > 0
