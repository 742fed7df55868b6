"""Girolorn models through the engine against the plain implementation (``plain_girolorn``): whole prompts, prompts
with their last tokens one by one, portions down to two tokens, mixed batches in pools so small that pages are used
again, long decoding through recorded steps, and greedy generation through the engine's own entry point and
scheduler.  Seven configurations that differ in every size and constant (``girolorn_tiny``)."""
import io
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import plain_girolorn as P
import traces
from girolorn_tiny import CONFIGS, make_model
from plain_llama import load_folder
from tiny import logit_error, prompt_ids

pytestmark = pytest.mark.gpu

# fraction of the mean logit range: (max, mean)
TOL = {"float32": (2e-5, 2e-6), "bfloat16": (5e-2, 6e-3)}
# In bfloat16 a token whose last chosen expert's logit and the next one's lie within rounding of each other may take the
# other expert: that token's row then differs by what the two experts differ, which no tolerance on rounding covers,
# and the layers behind carry the difference on to every later row of the request.  The plain implementation says by
# how much every choice is decided (``choice_margin``): in bfloat16 the bounds hold for a request's rows before its first
# choice that is decided by less than CLOSE_CALL of a logit; a close call in the last layer changes its own row alone, and
# a few rows (8 in 100, or one) may lie over the bound for it, none far over.  The rows behind are only asked to be
# numbers.  In 32 bits every row is held to the bounds, and so is every row of the configurations that choose every expert.
BF16_ROWS_OVER, BF16_FAR, CLOSE_CALL = 0.08, 0.5, 0.06
# prompt lengths (the rest of every request is given "decoded" tokens) and how many of those
WORKLOAD = {
    "G1": ([1, 4, 23, 64, 150], 30),
    "G2": ([2, 9, 31, 100], 26),
    "G3": ([3, 63, 129, 200], 40),          # prompts that end beside a page's edge
    "G4": ([2, 65, 99], 30),
    "G5": ([2, 90, 128, 330], 60),
    "G6": ([1, 30, 90], 50),
    "G7": ([3, 420], 40),
}


def first_close_call(cfg, calls, n_tokens):
    """``calls``: what ``forward`` recorded of every routed token, layer run by layer run, each over all tokens."""
    if not calls:
        return n_tokens
    runs = len(calls) // n_tokens
    last_routes = cfg["layers"][-1].get("mlp") is not None
    first = n_tokens
    for run in range(runs - 1 if last_routes else runs):
        for t in range(n_tokens):
            if calls[run * n_tokens + t][2] < CLOSE_CALL:
                first = min(first, t)
                break
    return first


FIRST_CLOSE = {}        # (configuration, request) -> the first row whose choice of experts a rounding may change


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    out = {}
    for which in WORKLOAD:
        d = make_model(which, str(tmp_path_factory.mktemp("girolorn" + which)))
        cfg, w = load_folder(d)
        lens, extra = WORKLOAD[which]
        reqs = {f"r{i}": prompt_ids(n + extra, cfg["vocab"], 1300 + i) for i, n in enumerate(lens)}
        plens = {f"r{i}": n for i, n in enumerate(lens)}
        want = {}
        for rid, toks in reqs.items():
            calls = []
            want[rid] = P.forward(cfg, w, toks, choices=calls)
            FIRST_CLOSE[(which, rid)] = first_close_call(cfg, calls, len(toks))
        out[which] = (d, cfg, w, reqs, plens, want)
    return out


def run_replay(model_dir, dtype, steps, tmp_path, page_size, max_requests=4, max_tokens=None, use_graphs=True):
    from xyntetik_runner_amd.engine.runner import ModelRunner
    from xyntetik_runner_amd.trace import replay
    mt = max_tokens or traces.max_live_tokens(steps, max(64, page_size))
    runner = ModelRunner.from_folder(model_dir, dtype=dtype, max_tokens=mt, page_size=page_size, max_requests=max_requests,
                                     use_graphs=use_graphs)
    for lc in runner.storage.layers:            # old keys must never show: they start as NaN
        lc.k.fill_(float("nan")); lc.v.fill_(float("nan"))
    out = str(tmp_path / "out")
    replay(runner, traces.to_lines(steps), out, report=io.StringIO())
    runner.manager.check()
    assert not runner.manager.requests and runner.manager.all_free()
    return out, runner


def check(got, want, dtype, what, which=None, upto=None):
    """``which``: the configuration whose requests' first close calls bound the rows that are compared in bfloat16
    (``upto``: the same as a mapping request -> row)."""
    assert set(got) == set(want)
    for rid in want:
        assert np.isfinite(got[rid]).all(), f"{what} {rid}: a logit is not finite"
        rng = float(np.mean(want[rid].max(axis=-1) - want[rid].min(axis=-1)))
        n = len(want[rid])
        if dtype == "bfloat16":
            n = upto[rid] if upto is not None else FIRST_CLOSE.get((which, rid), n)
        if n == 0:
            continue
        d = np.abs(np.asarray(got[rid][:n], dtype=np.float64) - want[rid][:n]) / rng
        mx, mean = float(d.max()), float(d.mean())
        if dtype == "bfloat16" and mx > TOL[dtype][0]:
            rows = d.max(axis=-1)
            over = int((rows > TOL[dtype][0]).sum())
            assert over <= max(1, BF16_ROWS_OVER * len(rows)) and mx <= BF16_FAR and mean <= TOL[dtype][1], \
                f"{what} {rid} ({dtype}): {over} of {len(rows)} rows over, max {mx:.3g} mean {mean:.3g}"
            continue
        assert mx <= TOL[dtype][0] and mean <= TOL[dtype][1], f"{what} {rid} ({dtype}): max {mx:.3g} mean {mean:.3g} ({n} rows)"


SCHEDULES = ["whole", "tail", "portions", "mixed"]


def steps_for(schedule, reqs, plens, extra):
    if schedule == "whole":
        return traces.whole(reqs)
    if schedule == "tail":
        return traces.tail_one_by_one(reqs, tail=extra)
    if schedule == "portions":
        return traces.portions(reqs)
    return traces.mixed(reqs, plens, max_live=min(3, len(reqs)), seed=5)


@pytest.mark.parametrize("schedule", SCHEDULES)
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which,page_size", [("G1", 16), ("G2", 8), ("G3", 64), ("G4", 16), ("G5", 64), ("G6", 4), ("G7", 64)])
def test_every_way_of_cutting_gives_the_plain_logits(models, tmp_path, which, page_size, dtype, schedule):
    d, cfg, w, reqs, plens, want = models[which]
    steps = steps_for(schedule, reqs, plens, WORKLOAD[which][1])
    out, runner = run_replay(d, dtype, steps, tmp_path, page_size, max_requests=3)
    check(traces.collect(steps, out, cfg["vocab"]), want, dtype, f"{which} {schedule}", which)
    if schedule == "tail":
        assert runner.graphs.replays > 0, "single tokens went through no recorded step"


def test_enough_rows_are_compared_in_bfloat16(models):
    """Close calls must not swallow the comparison: the configurations that choose every expert keep all their rows,
    the others a part."""
    for which in ("G2", "G6", "G7"):
        for rid, toks in models[which][3].items():
            assert FIRST_CLOSE[(which, rid)] == len(toks), (which, rid)
    for which in ("G1", "G3", "G5"):
        assert sum(FIRST_CLOSE[(which, rid)] for rid in models[which][3]) >= 10, which


def test_mixed_batch_equals_each_request_alone(models, tmp_path):
    """What a request's logits are does not depend on its neighbours in the batch beyond rounding:
    the mixed schedule against the same requests alone, engine against engine, in 32-bit."""
    d, cfg, w, reqs, plens, want = models["G5"]
    alone, _ = run_replay(d, "float32", traces.portions(reqs), tmp_path / "a", 64)
    steps = traces.mixed(reqs, plens, max_live=4, seed=9)
    mixed, _ = run_replay(d, "float32", steps, tmp_path / "m", 64)
    a = traces.collect(traces.portions(reqs), alone, cfg["vocab"])
    m = traces.collect(steps, mixed, cfg["vocab"])
    for rid in reqs:
        mx, _ = logit_error(m[rid], a[rid])
        assert mx <= 1e-5, f"{rid}: {mx:.3g}"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_slots_and_pages_are_used_again(models, tmp_path, dtype):
    """Two slots and a pool for the two longest requests: every request after the first two runs in pages that
    another has used, which hold its keys, for every run of a layer that shares its tensors."""
    d, cfg, w, reqs, plens, want = models["G6"]
    again = {f"{rid}.{i}": toks for i in range(2) for rid, toks in reqs.items()}
    plens = {f"{rid}.{i}": n for i in range(2) for rid, n in plens.items()}
    steps = traces.mixed(again, plens, max_live=2, seed=3)
    out, runner = run_replay(d, dtype, steps, tmp_path, 16, max_requests=2)
    assert runner.manager.slots.size == 2
    check(traces.collect(steps, out, cfg["vocab"]), {k: want[k.split(".")[0]] for k in again}, dtype, "reuse")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which", ["G6", "G2"])
def test_long_decoding_through_recorded_steps(models, tmp_path, dtype, which):
    """A short prompt and 300 tokens one by one over pages of 16."""
    d, cfg, w, reqs, plens, want = models[which]
    toks = prompt_ids(310, cfg["vocab"], 77)
    wanted = P.forward(cfg, w, toks)
    steps = traces.tail_one_by_one({"long": toks}, tail=300)
    out, runner = run_replay(d, dtype, steps, tmp_path, 16)
    assert runner.graphs.replays >= 290
    check(traces.collect(steps, out, cfg["vocab"]), {"long": wanted}, dtype, "long decoding")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_long_prompt_whole_and_in_portions(models, tmp_path, dtype):
    """900 tokens in one step (attention in whole tiles, the experts' rows sorted), the same in two long portions
    around a short one, and 20 more one by one."""
    d, cfg, w, *_ = models["G7"]
    toks = prompt_ids(920, cfg["vocab"], 78)
    wanted = {"long": P.forward(cfg, w, toks)}
    whole = traces.tail_one_by_one({"long": toks}, tail=20)
    out, _ = run_replay(d, dtype, whole, tmp_path / "w", 64)
    check(traces.collect(whole, out, cfg["vocab"]), wanted, dtype, "long prompt")
    cut = traces.portions({"long": toks}, sizes=(600, 2, 298, 1, 1, 18))
    out, _ = run_replay(d, dtype, cut, tmp_path / "c", 16)
    check(traces.collect(cut, out, cfg["vocab"]), wanted, dtype, "long prompt in portions")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_eager_and_recorded_steps_agree(models, tmp_path, dtype):
    d, cfg, w, reqs, plens, want = models["G1"]
    steps = traces.tail_one_by_one(reqs, tail=30)
    a, _ = run_replay(d, dtype, steps, tmp_path / "g", 16, use_graphs=True)
    b, _ = run_replay(d, dtype, steps, tmp_path / "e", 16, use_graphs=False)
    ga, gb = traces.collect(steps, a, cfg["vocab"]), traces.collect(steps, b, cfg["vocab"])
    for rid in reqs:
        if dtype == "float32":
            assert np.array_equal(ga[rid], gb[rid]), rid
        else:           # (a recorded step may cut a request's keys into other ranges)
            n = FIRST_CLOSE[("G1", rid)]
            assert n == 0 or logit_error(ga[rid][:n], gb[rid][:n])[0] <= TOL[dtype][0], rid


def test_every_run_of_a_shared_layer_has_a_cache_of_its_own(models):
    """Three layers' runs share tensors with two layers: five entries, each with pages of its own, and the
    residual stream after every entry is the plain one."""
    from xyntetik_runner_amd.engine.batch import StepEntry
    from xyntetik_runner_amd.engine.runner import ModelRunner
    d, cfg, w, reqs, plens, want = models["G1"]
    toks = reqs["r2"]
    plain_layers = []
    P.forward(cfg, w, toks, taps=plain_layers)
    r = ModelRunner.from_folder(d, dtype="float32", max_tokens=128, page_size=16, max_requests=2, use_graphs=False)
    assert len(r.storage.layers) == 5 and all(lc.owns for lc in r.storage.layers)
    assert len({lc.k.data_ptr() for lc in r.storage.layers}) == 5 and len(r.model.blocks) == 2
    taps = []
    r.model.tap = lambda i, x: taps.append(x.detach().float().cpu().numpy().copy())
    cut = 11            # a portion, then the rest: the taps of both steps side by side are the whole sequence's
    r.step([StepEntry("a", toks[:cut], [])])
    r.step([StepEntry("a", toks[cut:], [])])
    r.finish("a")
    assert len(taps) == 10
    for i in range(5):
        got = np.concatenate([taps[i], taps[5 + i]], axis=0)
        assert np.abs(got - plain_layers[i]).max() <= 2e-5 * max(1.0, np.abs(plain_layers[i]).max()), f"entry {i}"


def greedy(cfg, w, prompt, n_new):
    toks, out = list(prompt), []
    for _ in range(n_new):
        t = int(np.argmax(P.forward(cfg, w, toks)[-1]))
        out.append(t)
        toks.append(t)
    return out


@pytest.mark.parametrize("which", ["G1", "G2", "G6"])
def test_greedy_generation_through_the_entry_point(models, which):
    """``LLM.generate``: scheduler, portions under a token budget, sampling on the device."""
    from xyntetik_runner_amd import LLM, SamplingParams
    d, cfg, w, reqs, plens, want = models[which]
    prompts = [prompt_ids(n, cfg["vocab"], 500 + n) for n in (3, 21, 40)]
    wanted = [greedy(cfg, w, p, 8) for p in prompts]
    llm = LLM(d, dtype="float32", max_tokens=512, page_size=16, max_batched_tokens=16, max_running=2)
    got = llm.generate(prompts, SamplingParams(temperature=0.0, max_new_tokens=8))
    assert got == wanted
    assert llm.runner.manager.all_free()


ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def test_command_line(models):
    d, cfg, w, *_ = models["G3"]
    prompt = prompt_ids(9, cfg["vocab"], 21)
    wanted = greedy(cfg, w, prompt, 5)
    cmd = [sys.executable, os.path.join(ROOT, "bin", "runner"), "-m", d, "--ids", ",".join(map(str, prompt)), "-n", "5",
           "--temp", "0", "--dtype", "float32", "-c", "128", "-b", "4"]
    p = subprocess.run(cmd, capture_output=True, text=True, timeout=120)
    assert p.returncode == 0, p.stderr
    assert p.stdout.strip() == ",".join(map(str, prompt + wanted))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_run_program(models, tmp_path, dtype):
    """bin/trace_run as a user runs it: a child process, steps on stdin, 'done <step>' lines back,
    four slots and pools for the tokens that are live."""
    d, cfg, w, reqs, plens, want = models["G3"]
    steps = traces.mixed(reqs, plens, max_live=4, seed=2)
    out = str(tmp_path / "out")
    p = subprocess.Popen([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", d, "--dtype", dtype,
                          "--out", out, "--max-tokens", str(traces.max_live_tokens(steps, 64))],
                         stdin=subprocess.PIPE, stdout=subprocess.PIPE, text=True)
    for st in steps:
        p.stdin.write(json.dumps(st) + "\n")
        p.stdin.flush()
        assert p.stdout.readline().strip() == f"done {st['step']}"
    p.stdin.close()
    assert p.wait(timeout=60) == 0
    check(traces.collect(steps, out, cfg["vocab"]), want, dtype, "trace_run", "G3")
