"""Pevolorn models through the engine against the plain implementation (``plain_pevolorn``): whole prompts, prompts
with their last tokens one by one, portions down to two tokens, mixed batches in pools so small that pages are used
again, long decoding through recorded steps, and greedy generation through the engine's own entry point and
scheduler.  Eight configurations that differ in every size and constant (``pevolorn_tiny``)."""
import io
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import plain_pevolorn as P
import traces
from pevolorn_tiny import CONFIGS, make_model
from plain_llama import load_folder
from tiny import logit_error, prompt_ids

pytestmark = pytest.mark.gpu

# fraction of the mean logit range: (max, mean)
TOL = {"float32": (2e-5, 2e-6), "bfloat16": (5e-2, 6e-3)}
# In bfloat16 a token whose last chosen expert (or last kept group) and the next one lie within rounding of each other may
# take the other one: that token's row then differs by what the two experts differ, which no tolerance on rounding
# covers, and the layers behind carry the difference on to every later row of the request.  The plain implementation says
# by how much every choice is decided (``route_margin``): in bfloat16 the bounds hold for a request's rows before its first
# choice that is decided by less than CLOSE_CALL; a close call in the last layer changes its own row alone, and a few rows
# (8 in 100, or one) may lie over the bound for it, none far over.  The rows behind are only asked to be numbers.  In 32
# bits every row is held to the bounds, and so is every row of the configurations that choose every expert.
BF16_ROWS_OVER, BF16_FAR, CLOSE_CALL = 0.08, 0.5, 0.02
# prompt lengths (the rest of every request is given "decoded" tokens) and how many of those
WORKLOAD = {
    "P1": ([1, 4, 23, 64, 150], 30),
    "P2": ([2, 9, 31, 100], 26),
    "P3": ([3, 63, 129, 200], 40),          # prompts that end beside a page's edge
    "P4": ([2, 65, 99], 30),
    "P5": ([2, 90, 128, 330], 60),          # and prompts of whole chunks of the state space
    "P6": ([1, 30, 90], 50),
    "P7": ([3, 420], 40),
    "P8": ([2, 70], 20),
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
        d = make_model(which, str(tmp_path_factory.mktemp("pevolorn" + which)))
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
    for lc in runner.storage.layers:            # what an earlier request left must never show: it starts as NaN
        if lc.owns and lc.k is not None:
            lc.k.fill_(float("nan")); lc.v.fill_(float("nan"))
        for st in lc.states.values():
            st.fill_(float("nan"))
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
@pytest.mark.parametrize("which,page_size", [("P1", 16), ("P2", 8), ("P3", 64), ("P4", 16), ("P5", 64), ("P6", 4), ("P7", 64), ("P8", 16)])
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
    for which in ("P2", "P4", "P6", "P7", "P8"):
        for rid, toks in models[which][3].items():
            assert FIRST_CLOSE[(which, rid)] == len(toks), (which, rid)
    for which, rows in (("P1", 150), ("P3", 20), ("P5", 300)):
        assert sum(FIRST_CLOSE[(which, rid)] for rid in models[which][3]) >= rows, which


def test_mixed_batch_equals_each_request_alone(models, tmp_path):
    """What a request's logits are does not depend on its neighbours in the batch beyond rounding:
    the mixed schedule against the same requests alone, engine against engine, in 32-bit."""
    d, cfg, w, reqs, plens, want = models["P5"]
    alone, _ = run_replay(d, "float32", traces.portions(reqs), tmp_path / "a", 64)
    steps = traces.mixed(reqs, plens, max_live=4, seed=9)
    mixed, _ = run_replay(d, "float32", steps, tmp_path / "m", 64)
    a = traces.collect(traces.portions(reqs), alone, cfg["vocab"])
    m = traces.collect(steps, mixed, cfg["vocab"])
    for rid in reqs:
        mx, _ = logit_error(m[rid], a[rid])
        assert mx <= 1e-5, f"{rid}: {mx:.3g}"


@pytest.mark.parametrize("which", ["P2", "P6"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_slots_and_pages_are_used_again(models, tmp_path, dtype, which):
    """Two slots and a pool for the two longest requests: every request after the first two runs in pages and slots that
    another has used, which hold its latents, its keys and its state."""
    d, cfg, w, reqs, plens, want = models[which]
    again = {f"{rid}.{i}": toks for i in range(2) for rid, toks in reqs.items()}
    plens = {f"{rid}.{i}": n for i in range(2) for rid, n in plens.items()}
    steps = traces.mixed(again, plens, max_live=2, seed=3)
    out, runner = run_replay(d, dtype, steps, tmp_path, 16, max_requests=2)
    assert runner.manager.slots.size == 2
    check(traces.collect(steps, out, cfg["vocab"]), {k: want[k.split(".")[0]] for k in again}, dtype, "reuse")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which", ["P6", "P2", "P4"])
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
    """900 tokens in one step (attention in whole tiles, the state space in chunks, the experts' rows sorted), the same in
    two long portions around a short one, and 20 more one by one."""
    d, cfg, w, *_ = models["P7"]
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
    d, cfg, w, reqs, plens, want = models["P1"]
    steps = traces.tail_one_by_one(reqs, tail=30)
    a, _ = run_replay(d, dtype, steps, tmp_path / "g", 16, use_graphs=True)
    b, _ = run_replay(d, dtype, steps, tmp_path / "e", 16, use_graphs=False)
    ga, gb = traces.collect(steps, a, cfg["vocab"]), traces.collect(steps, b, cfg["vocab"])
    for rid in reqs:
        if dtype == "float32":
            assert np.array_equal(ga[rid], gb[rid]), rid
        else:           # (a recorded step may cut a request's keys into other ranges)
            n = FIRST_CLOSE[("P1", rid)]
            assert n == 0 or logit_error(ga[rid][:n], gb[rid][:n])[0] <= TOL[dtype][0], rid


def test_layers_that_read_another_layers_rows(models):
    """The readers own no pages, the owner's are written once; the residual stream after every layer is the plain one,
    across a cut."""
    from xyntetik_runner_amd.engine.batch import StepEntry
    from xyntetik_runner_amd.engine.runner import ModelRunner
    for which, owners in (("P1", [0, 1, 3, 4]), ("P5", [0, 2, 4]), ("P6", [0])):
        d, cfg, w, reqs, plens, want = models[which]
        toks = reqs["r2"][:60]
        plain_layers = []
        P.forward(cfg, w, toks, taps=plain_layers)
        r = ModelRunner.from_folder(d, dtype="float32", max_tokens=128, page_size=16, max_requests=2, use_graphs=False)
        n = len(cfg["layers"])
        layers = r.storage.layers
        assert [i for i, lc in enumerate(layers) if lc.owns] == owners and len(layers) == n
        for i, layer in enumerate(cfg["layers"]):
            j = layer["mixer"].get("kv_from")
            if j is not None:
                assert layers[i].k.data_ptr() == layers[j].k.data_ptr() and layers[i].group == layers[j].group
        taps = []
        r.model.tap = lambda i, x: taps.append(x.detach().float().cpu().numpy().copy())
        cut = 11        # a portion, then the rest: the taps of both steps side by side are the whole sequence's
        r.step([StepEntry("a", toks[:cut], [])])
        r.step([StepEntry("a", toks[cut:], [])])
        r.finish("a")
        assert len(taps) == 2 * n
        for i in range(n):
            got = np.concatenate([taps[i], taps[n + i]], axis=0)
            assert np.abs(got - plain_layers[i]).max() <= 2e-5 * max(1.0, np.abs(plain_layers[i]).max()), f"{which} layer {i}"


def test_a_pair_of_mixers_without_the_joint_products(models):
    """The two sides by products of their own, summed by the pair's own kernel, are the joint pair: the same part built
    without ``joint``."""
    import dataclasses
    from xyntetik_runner_amd.config import config_from_dict
    from xyntetik_runner_amd.engine.batch import StepEntry
    from xyntetik_runner_amd.engine.runner import ModelRunner
    from xyntetik_runner_amd.weights import SafetensorsStore
    for which in ("P1", "P4"):
        d, cfg, w, reqs, plens, want = models[which]
        arch, typed = config_from_dict(json.load(open(os.path.join(d, "config.json"))))
        spec = arch.build_spec(typed)
        layers = [dataclasses.replace(l, mixer=dataclasses.replace(l.mixer, params=dict(l.mixer.params, joint=False)))
                  if l.mixer.kind == "parallel_mixers" else l for l in spec.layers]
        store = SafetensorsStore.open_folder(d)
        r = ModelRunner(dataclasses.replace(spec, layers=layers), store, "float32", max_tokens=256, page_size=16, max_requests=2)
        store.close()
        toks = reqs["r1"]
        got = r.step([StepEntry("a", toks, list(range(len(toks))))]).cpu().numpy()
        check({"r1": got}, {"r1": want["r1"]}, "float32", f"{which} by four products")


def greedy(cfg, w, prompt, n_new):
    toks, out = list(prompt), []
    for _ in range(n_new):
        t = int(np.argmax(P.forward(cfg, w, toks)[-1]))
        out.append(t)
        toks.append(t)
    return out


@pytest.mark.parametrize("which", ["P1", "P2", "P4", "P6"])
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
    d, cfg, w, *_ = models["P3"]
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
    d, cfg, w, reqs, plens, want = models["P3"]
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
    check(traces.collect(steps, out, cfg["vocab"]), want, dtype, "trace_run", "P3")
