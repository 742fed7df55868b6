"""The serving benchmark: decode tokens a second for the Llama-3.1-8B shape with random
weights on one MI355X, plus the prefill rate at 2,048 tokens and the decode step's
fraction of the HBM roofline.

    python bench.py --gpus 1 --steps K --warmup W

A "step" is one decode step of the engine (schedule, model step, sampling) for a batch of
8 requests, each with a 2,048-token prompt already in the cache.  One JSON line goes to
stdout.  The reference's own bench times a 512-token prompt and 128 greedy tokens of one
sequence and ignores end-of-text while it does (src/main.c:1435-1515).
"""
import argparse
import json
import os
import sys
import time

ROOT = os.path.dirname(os.path.abspath(__file__))
sys.path.insert(0, ROOT)

LLAMA_3_1_8B = {
    "architectures": ["LlamaForCausalLM"], "model_type": "llama",
    "num_hidden_layers": 32, "hidden_size": 4096, "num_attention_heads": 32, "num_key_value_heads": 8,
    "head_dim": 128, "intermediate_size": 14336, "vocab_size": 128256, "rope_theta": 500000.0,
    "rope_scaling": {"rope_type": "llama3", "factor": 8.0, "low_freq_factor": 1.0, "high_freq_factor": 4.0,
                     "original_max_position_embeddings": 8192},
    "rms_norm_eps": 1e-5, "tie_word_embeddings": False, "max_position_embeddings": 8192, "hidden_act": "silu",
}
# other sizes of the same architecture (--shape); the default and the contract's line are the 8B shape
LLAMA_2_7B = dict(LLAMA_3_1_8B, num_key_value_heads=32, intermediate_size=11008, vocab_size=32000, rope_theta=10000.0,
                  rope_scaling=None, max_position_embeddings=4096)
LLAMA_3_1_70B = dict(LLAMA_3_1_8B, num_hidden_layers=80, hidden_size=8192, num_attention_heads=64, intermediate_size=28672)
# a small shape of the same architecture with heads of 64 and tied embeddings (the sizes of a 1B-class Llama)
LLAMA_1B = dict(LLAMA_3_1_8B, num_hidden_layers=16, hidden_size=2048, head_dim=64, intermediate_size=8192,
                tie_word_embeddings=True, max_position_embeddings=131072,
                rope_scaling={"rope_type": "llama3", "factor": 32.0, "low_freq_factor": 1.0, "high_freq_factor": 4.0,
                              "original_max_position_embeddings": 8192})
SHAPES = {"llama-3.1-8b": ("Llama-3.1-8B shape", LLAMA_3_1_8B), "llama-2-7b": ("Llama-2-7B shape", LLAMA_2_7B),
          "llama-3.1-70b": ("Llama-3.1-70B shape", LLAMA_3_1_70B), "llama-1b-head64": ("Llama 1B-class shape, heads of 64", LLAMA_1B)}
PEAK = {"hbm_gbs": 8000.0, "bf16_flops": 2.5e15, "fp32_flops": 157.3e12}


def log(msg):
    sys.stderr.write(f"[bench] {msg}\n")
    sys.stderr.flush()


def build_runner(cfg, dtype, max_tokens, max_requests, seed=0):
    import torch
    from xyntetik_runner_amd.config import config_from_dict
    from xyntetik_runner_amd.engine import ModelRunner
    from xyntetik_runner_amd.engine.model import Model
    from xyntetik_runner_amd.weights import random_state
    arch, typed = config_from_dict(cfg)
    spec = arch.build_spec(typed)
    t0 = time.time()
    state = random_state(Model.expected_tensors(spec), seed, device=torch.device("cuda:0"))
    runner = ModelRunner(spec, state, dtype, max_tokens=max_tokens, page_size=64, max_requests=max_requests,
                         consume_state=True)      # the 70B shape is half the card: it must not stand there twice
    del state
    torch.cuda.synchronize()
    log(f"model with {len(spec.layers)} layers on the GPU in {time.time() - t0:.1f} s")
    return spec, runner


def matmul_params(cfg, layers):
    E, H, Hk, D, F, V = (cfg["hidden_size"], cfg["num_attention_heads"], cfg["num_key_value_heads"], cfg["head_dim"],
                         cfg["intermediate_size"], cfg["vocab_size"])
    per_layer = E * (H * D + 2 * Hk * D) + H * D * E + 3 * E * F
    return per_layer * layers, V * E


def decode_bytes(cfg, layers, batch, ctx_tokens, elt=2):
    """Bytes one decode step has to read: every weight it uses once, and the cache of the live requests."""
    body, head = matmul_params(cfg, layers)
    norms = (2 * layers + 1) * cfg["hidden_size"]
    weights = (body + head + norms) * elt + batch * cfg["hidden_size"] * elt     # + one embedding row per request
    kv = ctx_tokens * 2 * cfg["num_key_value_heads"] * cfg["head_dim"] * layers * elt
    return weights + kv


def prefill_flops(cfg, layers, T):
    body, head = matmul_params(cfg, layers)
    attn = 4 * cfg["num_attention_heads"] * cfg["head_dim"] * layers * (T * (T + 1) // 2)
    return 2 * body * T + 2 * head * 1 + attn


def measure_achievable(runner):
    """What this GPU delivers to kernels with nothing else to do, as yardsticks beside the nominal
    peaks: bytes a second to a kernel that only reads (every workgroup a range of its own, 8 GB in
    all), and bfloat16 products a second of the matrix kernel on one large product of random data
    (8192 x 28672 x 4096).  The best of five each."""
    import torch
    ops = runner.ops
    dev = runner.device

    def best_ms(fn, reps=5):
        fn()
        best = None
        for _ in range(reps):
            a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
            a.record()
            fn()
            b.record()
            b.synchronize()
            t = a.elapsed_time(b)
            best = t if best is None else min(best, t)
        return best
    n_bytes = 8 << 30
    buf = torch.empty((n_bytes,), dtype=torch.uint8, device=dev)
    buf.zero_()
    read_ms = best_ms(lambda: ops.stream_read(buf))
    del buf
    M, N, K = 8192, 28672, 4096
    a = (torch.randn((M, K), device=dev) * 0.5).bfloat16()
    w = ops.pack_weight((torch.randn((N, K), device=dev) * 0.02).bfloat16())
    out = torch.empty((M, N), dtype=torch.bfloat16, device=dev)
    mm_ms = best_ms(lambda: ops.linear(a, w, out=out))
    del a, w, out
    torch.cuda.empty_cache()
    return n_bytes / (read_ms * 1e-3) / 1e9, 2.0 * M * N * K / (mm_ms * 1e-3)


def measure_decode(runner, cfg, batch, prompt_len, steps, warmup, seed, alone=False):
    """tokens/s of `steps` decode steps with `batch` requests whose prompts are already cached;
    afterwards one more step's logits are checked (`check_decode_logits`)."""
    import numpy as np
    import torch
    from xyntetik_runner_amd.engine import Engine
    from xyntetik_runner_amd.sampling import SamplingParams
    # (prompts up to 8,192 tokens go in one step each, longer ones in portions of 2,048)
    budget = max(2048, prompt_len) if prompt_len <= 8192 else 2048
    eng = Engine(runner, max_batched_tokens=budget, max_running=batch,
                 max_model_len=cfg["max_position_embeddings"], stop_ids=[])
    rng = np.random.default_rng(seed)
    # a request admitted first decodes while the others' prompts are still computed (a step for
    # every portion of every prompt): nobody may finish before the last timed step
    sp = SamplingParams(temperature=0.0, max_new_tokens=batch * -(-prompt_len // budget) + warmup + steps + 8, ignore_eos=True)
    ids = [eng.add_request([int(t) for t in rng.integers(0, cfg["vocab_size"], size=prompt_len)], sp) for _ in range(batch)]
    def step():
        for o in eng.step():
            if o.finished:
                raise RuntimeError(f"decode batch {batch}: request {o.req_id!r} ended before the last timed step ({o.finish_reason})")
    while any(eng.requests[i].n_computed < prompt_len for i in ids):
        step()
    for _ in range(warmup):
        step()
    ctx0 = sum(eng.requests[i].n_tokens for i in ids)
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    for _ in range(steps):
        eng.step()
    torch.cuda.synchronize()
    dt = time.perf_counter() - t0
    if len(eng.scheduler.running) != batch or any(i not in eng.requests for i in ids):
        raise RuntimeError(f"decode batch {batch}: a request ended or waited during the timed steps")
    ctx1 = sum(eng.requests[i].n_tokens for i in ids)
    if ctx1 - ctx0 != batch * steps:
        raise RuntimeError(f"decode batch {batch}: {ctx1 - ctx0} tokens decoded in {steps} steps")
    replays = runner.graphs.replays if runner.graphs is not None else 0
    check = check_decode_logits(runner, eng, ids, batch, alone)
    if runner.graphs is not None:
        if runner.graphs.replays <= replays:
            raise RuntimeError(f"decode batch {batch}: the checked step did not go through a recorded graph")
        log(f"  graphs: {runner.graphs.captures} captured, {runner.graphs.replays} replays so far")
    return batch * steps / dt, dt / steps, (ctx0 + ctx1) / 2, check


def sane_logits(rows, what):
    """The reference's rule for a run that computed nothing: all-zero logits fail
    (tests/test_gpu_identity.c:190-201); so do logits that are not finite, and rows that are constant."""
    import torch
    if not bool(torch.isfinite(rows).all()):
        raise RuntimeError(f"{what}: logits are not finite")
    if bool((rows.abs().amax(dim=-1) == 0).any()) or bool((rows.std(dim=-1) == 0).any()):
        raise RuntimeError(f"{what}: a row of logits is all zero or all equal")


def check_decode_logits(runner, eng, ids, batch, alone):
    """One more decode step of the timed batch, through the same recorded graph, with its logits
    looked at: every row finite, not zero, not constant.  With ``alone``, the first request's row is
    also compared with the same tokens run as a request of its own (its prompt in portions of 2,048,
    the last token as a decode step of one): (max, mean) difference as fractions of the mean logit
    range.  Ends the requests."""
    import torch
    from xyntetik_runner_amd.engine.batch import StepEntry
    eng.run_ahead = False
    eng.step()                       # the step that was queued ahead, if any: now the host knows every token
    reqs = [eng.requests[i] for i in ids]
    if any(r.remaining != 1 for r in reqs):
        raise RuntimeError(f"decode batch {batch}: a request is not decoding")
    logits = runner.step([StepEntry(r.id, [r.output[-1]], [0]) for r in reqs])
    sane_logits(logits, f"decode batch {batch}")
    row = logits[0].clone()
    tokens = list(reqs[0].prompt) + list(reqs[0].output)
    for i in ids:
        eng.abort(i)
    if not alone:
        return None
    for a in range(0, len(tokens) - 1, 2048):
        runner.step([StepEntry("alone", tokens[a:min(a + 2048, len(tokens) - 1)], [])])
    single = runner.step([StepEntry("alone", tokens[-1:], [0])])[0]
    runner.finish("alone")
    sane_logits(single[None], f"decode batch {batch}, the first request alone")
    span = float((single.max() - single.min()))
    d = (row - single).abs()
    return {"max": round(float(d.max()) / span, 5), "mean": round(float(d.mean()) / span, 6),
            "same_top": bool(int(row.argmax()) == int(single.argmax()))}


def measure_mixed(runner, cfg, n_requests, steps_each, seed):
    """A scheduler workload: `n_requests` prompts of 128..2048 tokens admitted at once, `steps_each`
    tokens decoded for each, portions of prompts beside decoded tokens under a 2048-token budget.
    Returns (prompt tokens, decoded tokens, seconds, steps)."""
    import numpy as np
    import torch
    from xyntetik_runner_amd.engine import Engine
    from xyntetik_runner_amd.sampling import SamplingParams
    eng = Engine(runner, max_batched_tokens=2048, max_running=n_requests,
                 max_model_len=cfg["max_position_embeddings"], stop_ids=[])
    rng = np.random.default_rng(seed)
    lens = [int(n) for n in rng.integers(128, 2049, size=n_requests)]
    sp = SamplingParams(temperature=0.0, max_new_tokens=steps_each, ignore_eos=True)
    for n in lens:
        eng.add_request([int(t) for t in rng.integers(0, cfg["vocab_size"], size=n)], sp)
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    n_steps = 0
    done = []
    while eng.has_work():
        done += [o.request for o in eng.step() if o.finished]
        n_steps += 1
    torch.cuda.synchronize()
    secs = time.perf_counter() - t0
    if len(done) != n_requests or any(len(r.output) != steps_each for r in done):
        raise RuntimeError("mixed workload: a request ended early")
    return sum(lens), n_requests * steps_each, secs, n_steps


def measure_prefill(runner, cfg, T, repeats, seed):
    import numpy as np
    import torch
    from xyntetik_runner_amd.engine.batch import StepEntry
    """Seconds for a prompt of T tokens in one step, up to the logits of its last position on the
    host: the median of ``repeats`` runs after one that is not counted (the reference reports
    medians, docs/benchmarks.md:16)."""
    rng = np.random.default_rng(seed)
    times = []
    for r in range(repeats + 1):
        toks = [int(t) for t in rng.integers(0, cfg["vocab_size"], size=T)]
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        out = runner.step([StepEntry(("prefill", r), toks, [T - 1])])
        last = out.cpu()
        dt = time.perf_counter() - t0
        sane_logits(last, "prefill")
        runner.finish(("prefill", r))
        if r > 0:
            times.append(dt)
    times.sort()
    return times[len(times) // 2]


def measure_prefill_in_portions(runner, cfg, T, portion, seed):
    """Seconds for a prompt of T tokens run in portions of ``portion`` (each step reads the cache
    the portions before it left), up to the logits of its last position."""
    import numpy as np
    import torch
    from xyntetik_runner_amd.engine.batch import StepEntry
    rng = np.random.default_rng(seed)
    best = None
    for r in range(2):
        toks = [int(t) for t in rng.integers(0, cfg["vocab_size"], size=T)]
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        for a in range(0, T, portion):
            b = min(T, a + portion)
            out = runner.step([StepEntry(("long prefill", r), toks[a:b], [b - a - 1] if b == T else [])])
        out.cpu()
        dt = time.perf_counter() - t0
        runner.finish(("long prefill", r))
        best = dt if best is None else min(best, dt)
    return best


def suripel_config(width, layers, vocab=32000):
    """A Suripel model of real layer sizes: heads of 128, four query heads a key/value head, a
    window of 1,024 with blocks of 64, the mixers in turn (of every six layers: retention, attention,
    delta, an attention that reads the first one's keys and values, retention, delta), a dense
    feed-forward with as many weights as a gated one of 3.5 x width."""
    H = width // 128
    ff = {"kind": "dense", "ff": int(width * 5.25)}

    def attn(kv_from=None):
        m = {"heads": H, "kv_heads": max(1, H // 4), "dim": 128, "vdim": 128, "conv": 4, "scale": 128 ** -0.5,
             "mask": {"size": 1024, "pool": 64}}
        if kv_from is not None:
            m["kv_from"] = kv_from
        return {"type": "attention", "mixer": m, "mlp": ff}
    delta = {"type": "delta", "mixer": {"heads": H, "kv_heads": max(1, H // 2), "dim": 128, "vdim": 128, "conv": 4}, "mlp": ff}
    ret = {"type": "retention", "mixer": {"heads": H, "dim": 128, "vdim": 128, "decay": [1 - 0.06 * 0.75 ** (8 * i / H) for i in range(H)],
                                          "rot": {"dims": 128, "base": 1e6}}, "mlp": ff}
    out = []
    for i in range(layers):
        k = i % 6
        out.append(attn() if k == 1 else attn(kv_from=i - 2) if k == 3 else delta if k in (2, 5) else ret)
    return {"architecture": "Suripel", "vocab": vocab, "width": width, "norm": {"eps": 1e-5}, "canon": {"taps": 4}, "layers": out}


def sugosun_config(width, layers, vocab=32000):
    """A Sugosun model of real layer sizes: two residual streams, a pair table of 100,003 rows, heads of 128 in the
    lightning layers; latent attention with a cached row of 192 + 64 channels, 64 unrotated and 64 rotated query
    channels a head, values of 128, a query latent of 3/8 width and a window of 1,024; of every four layers
    lightning with a dense feed-forward of 3.5 x width, latent attention with 16 experts of width / 2 (2 a token),
    lightning with such experts, latent attention with the dense feed-forward."""
    H = width // 128
    dense = {"kind": "dense", "ff": int(width * 3.5), "limit": 7.0}
    moe = {"kind": "moe", "expert": {"ff": width // 2}, "router": {"experts": 16, "top": 2}}
    light = {"heads": H, "dim": 128, "vdim": 128, "decay": [1 - 0.06 * 0.75 ** (8 * i / H) for i in range(H)]}
    latent = {"heads": H, "dim": 64, "rot_dim": 64, "vdim": 128, "q_rank": width * 3 // 8, "kv_rank": 192, "scale": 128 ** -0.5,
              "rot": {"dims": 64, "base": 1e4}, "mask": {"size": 1024}}
    out = []
    for i in range(layers):
        k = i % 4
        out.append({"type": "lightning" if k in (0, 2) else "latent_attention", "mixer": light if k in (0, 2) else latent,
                    "mlp": dense if k in (0, 3) else moe})
    return {"architecture": "Sugosun", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "streams": 2,
            "embedding": {"bigram": {"buckets": 100003, "mul_prev": 1000003, "mul_cur": 999983}}, "layers": out}


def dinasun_config(width, layers, vocab=32000):
    """A Dinasun model of real layer sizes whose layer runs are ``layers``: time mixing with heads of 64 and
    attention with heads of 128 (four query heads a key/value head, a temperature step every 1,024 positions) in
    turn, every layer with 16 gated experts of width / 2 (2 a token, by the table) and a shared expert of the
    model's width; a third of the runs are the second pass over a span in the middle."""
    again = layers // 3
    distinct = layers - again
    moe = {"kind": "moe", "expert": {"ff": width // 2}, "router": {"experts": 16, "top": 2}, "shared": {"ff": width}}
    H = width // 128
    wkv = {"type": "wkv", "mixer": {"heads": width // 64, "dim": 64}, "mlp": moe}
    att = {"type": "attention", "mixer": {"heads": H, "kv_heads": max(1, H // 4), "dim": 128, "vdim": 128, "scale": 128 ** -0.5,
                                          "q_temp": {"coef": 0.1, "every": 1024}}, "mlp": moe}
    cfg = {"architecture": "Dinasun", "vocab": vocab, "width": width, "norm": {"eps": 1e-5}, "residual_mult": 0.8,
           "embedding": {"scale": 1.0}, "layers": [wkv if i % 2 == 0 else att for i in range(distinct)]}
    if again:
        start = (distinct - again) // 2
        cfg["loop"] = {"start": start, "stop": start + again, "times": 2}
    return cfg


def kegorax_config(width, layers, vocab=32000):
    """A Kegorax model of real layer sizes whose layer runs are ``layers``: of every three layers the gated delta rule
    with a decay a key channel (heads of 128, two heads a key head, four taps), chunked attention with a sink and a gate a
    head (heads of 128, four query heads a key/value head, chunks of 1,024, half the head rotated) beside gated linear
    attention (half as many heads of 128), and windowed attention that keeps four tokens (a window of 1,024) beside
    retention; a gated dense feed-forward of 3.5 x width, but 16 experts of width / 2 (2 a token, from 2 of 4 groups) in
    the chunked layers; a third of the runs are the second pass over a span in the middle."""
    again = layers // 3
    distinct = layers - again
    H = width // 128
    dense = {"kind": "dense", "ff": int(width * 3.5)}
    moe = {"kind": "moe", "expert": {"ff": width // 2}, "router": {"experts": 16, "top": 2, "scale": 2.0, "groups": {"count": 4, "keep": 2}}}
    att = {"heads": H, "kv_heads": max(1, H // 4), "dim": 128, "vdim": 128, "scale": 128 ** -0.5}
    half = max(1, H // 2)
    delta = {"type": "channel_delta", "mixer": {"heads": H, "kv_heads": half, "dim": 128, "vdim": 128, "conv": 4}, "mlp": dense}
    par = {"type": "parallel", "mixer": {"left": dict(att, mask={"size": 1024}, rot={"base": 5e5, "dims": 64}),
                                         "right": {"heads": half, "dim": 128, "vdim": 128, "tau": 8.0}}, "mlp": moe}
    par2 = {"type": "parallel_2", "mixer": {"left": dict(att, mask={"size": 1024, "keep_first": 4}),
                                            "right": {"heads": half, "dim": 128, "vdim": 128,
                                                      "decay": [1 - 0.06 * 0.75 ** (8 * i / half) for i in range(half)]},
                                            "left_scale": 0.5, "right_scale": 1.0}, "mlp": dense}
    cfg = {"architecture": "Kegorax", "vocab": vocab, "width": width, "norm": {"eps": 1e-5}, "embedding": {"scale": 1.0},
           "layers": [(delta, par, par2)[i % 3] for i in range(distinct)]}
    if again:
        start = (distinct - again) // 2
        cfg["loop"] = {"start": start, "stop": start + again, "times": 2}
    return cfg


def girolorn_config(width, layers, vocab=32000):
    """A Girolorn model of real layer sizes: soft-capped attention whose values are its keys (heads of 128, four query
    heads a key/value head, the whole head rotated with YaRN for four times 4,096 positions, a learned sink a head), every
    layer with 16 experts of width / 2 (2 a token) and a gated shared expert of the model's width; the last third of the
    layers runs with the tensors of the first."""
    again = layers // 3
    H = width // 128
    layer = {"type": "attention",
             "mixer": {"heads": H, "kv_heads": max(1, H // 4), "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "softcap": 30.0,
                       "rot": {"base": 1e6, "dims": 128, "scaling": {"factor": 4.0, "original": 4096, "fast": 32.0, "slow": 1.0}}},
             "mlp": {"kind": "moe", "expert": {"ff": width // 2, "limit": 7.0}, "router": {"experts": 16, "top": 2},
                     "shared": {"ff": width, "limit": 7.0}}}
    return {"architecture": "Girolorn", "vocab": vocab, "width": width, "norm": {"eps": 1e-5}, "logit_softcap": 20.0,
            "layers": [dict(layer) for _ in range(layers - again)] + [dict(layer, weights_of=i) for i in range(again)]}


def pevolorn_config(width, layers, vocab=32000):
    """A Pevolorn model of real layer sizes: of every four layers latent attention with a cached row of 192 + 64 channels
    (128 unrotated and 64 rotated query channels a head, values of 128), such a layer that reads the rows of the one before,
    and two of soft-capped attention (heads of 128, four query heads a key/value head, half the head rotated) beside a state
    space of twice the width (heads of 64, states of 128, 8 groups, four taps); every layer with 14 experts of width / 2 and
    2 identity experts (2 a token, from 2 of 4 groups) and a shared expert of the model's width."""
    H = width // 128
    moe = {"kind": "moe", "expert": {"ff": width // 2}, "router": {"experts": 14, "identity": 2, "top": 2, "groups": {"count": 4, "keep": 2}},
           "shared": {"ff": width}}
    latent = {"heads": H, "dim": 128, "rot_dim": 64, "vdim": 128, "kv_rank": 192, "scale": 192 ** -0.5, "rot": {"base": 1e4, "dims": 64}}
    both = {"left": {"heads": H, "kv_heads": max(1, H // 4), "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "softcap": 40.0,
                     "rot": {"base": 1e5, "dims": 64}},
            "right": {"heads": width // 32, "vdim": 64, "state": 128, "groups": 8, "conv": 4, "norm_groups": 8},
            "left_scale": 0.7, "right_scale": 0.7}
    out = []
    for i in range(layers):
        k = i % 4
        mixer = latent if k == 0 else dict(latent, kv_from=i - 1) if k == 1 else both
        out.append({"type": "latent_attention" if k < 2 else "parallel", "mixer": mixer, "mlp": moe})
    return {"architecture": "Pevolorn", "vocab": vocab, "width": width, "norm": {"eps": 1e-5}, "postln_alpha": 2.0, "layers": out}


DESIGNS = {"suripel": ("Suripel", suripel_config), "sugosun": ("Sugosun", sugosun_config), "dinasun": ("Dinasun", dinasun_config),
           "kegorax": ("Kegorax", kegorax_config), "girolorn": ("Girolorn", girolorn_config),
           "pevolorn": ("Pevolorn", pevolorn_config)}


def llama_like(width, layers, vocab=32000):
    """The closest existing model at equal size: the Llama decoder with the same width, layers, heads and weights a layer."""
    return dict(LLAMA_3_1_8B, num_hidden_layers=layers, hidden_size=width, num_attention_heads=width // 128,
                num_key_value_heads=max(1, width // 512), head_dim=128, intermediate_size=int(width * 3.5), vocab_size=vocab,
                rope_scaling=None, max_position_embeddings=8192)


def measure_design(runner, vocab, prompt_len, batches, steps, seed):
    """(seconds for a prompt of ``prompt_len`` tokens in one step, {batch: seconds a decode step}) through the
    step function: the median of five prompts, and ``steps`` steps of single tokens (recorded graphs) behind
    ``prompt_len`` cached tokens a request."""
    import numpy as np
    import torch
    from xyntetik_runner_amd.engine.batch import StepEntry
    rng = np.random.default_rng(seed)
    toks = lambda n: [int(t) for t in rng.integers(0, vocab, size=n)]
    times = []
    for r in range(6):
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        out = runner.step([StepEntry(("p", r), toks(prompt_len), [prompt_len - 1])])
        sane_logits(out.cpu(), "prefill")
        times.append(time.perf_counter() - t0)
        runner.finish(("p", r))
    pre = sorted(times[1:])[2]
    dec = {}
    for b in batches:
        ids = [("d", b, i) for i in range(b)]
        for i in ids:
            runner.step([StepEntry(i, toks(prompt_len), [])])
        step = lambda: runner.step([StepEntry(i, toks(1), [0]) for i in ids])
        for _ in range(4):
            step()
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        for _ in range(steps):
            out = step()
        torch.cuda.synchronize()
        dec[b] = (time.perf_counter() - t0) / steps
        sane_logits(out, f"decode batch {b}")
        for i in ids:
            runner.finish(i)
    return pre, dec


def bench_design(args):
    """``--design NAME``: prefill and decode of that design at a few real layer sizes beside the Llama
    decoder of equal size, both with random weights through the same step function.  One JSON line."""
    import torch
    title, make_config = DESIGNS[args.design]
    sizes = [int(x) for x in args.design_sizes.split(",")]
    batches = [1, 8, 64]
    rows = []
    for width in sizes:
        row = {"width": width, "layers": args.design_layers}
        for name, cfg in ((args.design, make_config(width, args.design_layers)), ("llama", llama_like(width, args.design_layers))):
            if name == "llama" and args.design_alone:
                continue
            spec, runner = build_runner(cfg, args.dtype, max_tokens=66 * (args.prompt_len + 256), max_requests=64)
            pre, dec = measure_design(runner, 32000, args.prompt_len, batches, min(args.steps, 64), seed=width)
            row[name] = {"prefill_ms": round(pre * 1e3, 3), "prefill_tok_s": round(args.prompt_len / pre, 1),
                         **{f"decode_b{b}_ms": round(t * 1e3, 4) for b, t in dec.items()},
                         **{f"decode_b{b}_tok_s": round(b / t, 1) for b, t in dec.items()}}
            log(f"width {width}, {name}: {row[name]}")
            del runner
            torch.cuda.empty_cache()
        rows.append(row)
    line = {"metric": f"prefill and decode of the {title} design beside the Llama decoder of equal size ({args.prompt_len}-token prompts, random weights)",
            "unit": "ms and tokens/s", "n_gpus": 1, "dtype": "bf16" if args.dtype == "bfloat16" else "fp32", "data": "synthetic",
            "sizes": rows}
    print(json.dumps(line), flush=True)
    if args.record:
        with open(args.record, "w") as f:
            f.write(f"# bench.py --design {args.design}\n\nCommand:\n\n    python {' '.join(['bench.py'] + sys.argv[1:])}\n\n"
                    f"Result (one MI355X, random weights, synthetic tokens):\n\n```json\n{json.dumps(line, indent=1)}\n```\n")
    return 0


def main():
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=256, help="decode steps that are timed (the configuration decodes 256 tokens)")
    ap.add_argument("--warmup", type=int, default=16)
    ap.add_argument("--layers", type=int, default=0, help="run fewer layers than the configuration has (named in config)")
    ap.add_argument("--batch", type=int, default=8)
    ap.add_argument("--prompt-len", type=int, default=2048)
    ap.add_argument("--no-points", action="store_true", help="skip decode at batch 1 and 64")
    ap.add_argument("--dtype", default="bfloat16")
    ap.add_argument("--shape", default="llama-3.1-8b", choices=sorted(SHAPES), help="sizes of the model (same architecture)")
    ap.add_argument("--max-context", type=int, default=0, metavar="N",
                    help="the model's context length (max_position_embeddings) instead of the shape's own")
    ap.add_argument("--contexts", default="", metavar="LIST",
                    help="decode points at these context lengths (comma separated) instead of the points at the model's limit")
    ap.add_argument("--context-batches", default="1,8", metavar="LIST", help="batch sizes of the --contexts points")
    ap.add_argument("--long-prefill", type=int, default=0, metavar="T",
                    help="length of the prompt that is run in portions of 2,048 (default: the model's context)")
    ap.add_argument("--record", default="", metavar="FILE",
                    help="also write the command and the JSON line into FILE (markdown)")
    ap.add_argument("--mixed", type=int, default=0, metavar="N",
                    help="also run N requests with prompts of 128..2048 tokens and 128 decoded tokens each through the scheduler")
    ap.add_argument("--design", default="", choices=["", *DESIGNS],
                    help="instead of the serving benchmark: this design at real layer sizes beside the Llama decoder of equal size")
    ap.add_argument("--design-sizes", default="2048,4096", metavar="LIST", help="widths of the --design models")
    ap.add_argument("--design-layers", type=int, default=12, help="layers of the --design models")
    ap.add_argument("--design-alone", action="store_true", help="the --design model without the Llama decoder beside it")
    args = ap.parse_args()
    if args.design:
        if args.gpus != 1:
            print("bench.py measures one GPU only", flush=True)
            return 2
        return bench_design(args)
    if args.gpus != 1:
        print(f"bench.py measures one GPU only: --gpus {args.gpus} is not supported by this engine", flush=True)
        return 2
    shape_name, shape_cfg = SHAPES[args.shape]
    cfg = {k: v for k, v in shape_cfg.items() if v is not None}
    layers_full = cfg["num_hidden_layers"]
    layers = args.layers or layers_full
    cfg["num_hidden_layers"] = layers
    if args.max_context:
        cfg["max_position_embeddings"] = args.max_context
    P, B = args.prompt_len, args.batch
    elt = 2 if args.dtype == "bfloat16" else 4
    ctx_max = cfg["max_position_embeddings"]
    long_steps, long_warmup = 32, 4
    span = P + args.warmup + args.steps + 80 + max(64, B)
    pool = max(max(64, B) * (-(-span // 64) * 64) + 4096, args.mixed * (2048 + 128 + 64))
    # The points away from the tuned one: (context, batch) pairs.  By default the model's limit at
    # batch 8 and, if the card has room for 64 requests of that length beside the weights, at batch 64.
    import torch
    kv_per_token = 2 * cfg["num_key_value_heads"] * cfg["head_dim"] * layers * elt
    body, head = matmul_params(cfg, layers)
    weight_bytes = (body + (1 if cfg.get("tie_word_embeddings") else 2) * head) * elt
    total_mem = torch.cuda.get_device_properties(0).total_memory

    def pool_for(ctx, b):
        return b * (-(-(ctx + 128) // 64) * 64) + 4096
    if args.contexts:
        ctx_points = [(int(c), int(b)) for c in args.contexts.split(",") for b in args.context_batches.split(",")]
    else:
        ctx_points = [(ctx_max, 8), (ctx_max, 64)]
    left_out = [cb for cb in ctx_points if weight_bytes + pool_for(*cb) * kv_per_token >= 0.8 * total_mem or cb[0] > ctx_max]
    ctx_points = [cb for cb in ctx_points if cb not in left_out]
    long_T = args.long_prefill or min(ctx_max, 32768)
    if not args.no_points:
        pool = max([pool, long_T + 4096] + [pool_for(*cb) for cb in ctx_points])
    spec, runner = build_runner(cfg, args.dtype, max_tokens=pool, max_requests=max(64, args.mixed))

    read_gbs, mm_flops = measure_achievable(runner) if args.dtype == "bfloat16" else (None, None)
    if read_gbs:
        log(f"achievable on this GPU: {read_gbs:.0f} GB/s to a kernel that only reads, "
            f"{mm_flops / 1e12:.0f} TFLOP/s bfloat16 on a 8192 x 28672 x 4096 product")
    peak_flops = PEAK["bf16_flops" if args.dtype == "bfloat16" else "fp32_flops"]
    pre_s = measure_prefill(runner, cfg, 2048, repeats=5, seed=1)
    pre_rate = prefill_flops(cfg, layers, 2048) / pre_s
    log(f"prefill 2048 tokens: {pre_s * 1e3:.1f} ms (the median of 5)")

    # the decode figure: the median of three repetitions of the whole workload (fresh requests,
    # prompts computed again), as the reference reports a median of its runs
    # (docs/benchmarks.md:16)
    runs = []
    for rep in range(3):
        tps, step_s, ctx, _ = measure_decode(runner, cfg, B, P, args.steps, args.warmup, seed=2 + 100 * rep)
        runs.append((step_s, tps, ctx))
        log(f"decode batch {B}, repetition {rep + 1}: {tps:.1f} tok/s, {step_s * 1e3:.3f} ms/step, "
            f"{decode_bytes(cfg, layers, B, ctx, elt) / step_s / 1e9:.0f} GB/s")
    runs.sort()
    step_s, tps, ctx = runs[1]
    achieved = decode_bytes(cfg, layers, B, ctx, elt) / step_s / 1e9
    points, checks = {}, {}
    if not args.no_points:
        def point(name, b, prompt_len, n, warm, seed, alone=False):
            t, sec, c, chk = measure_decode(runner, cfg, b, prompt_len, n, warm, seed=seed, alone=alone)
            points[name] = round(t, 1)
            log(f"{name}: {t:.1f} tok/s, {sec * 1e3:.3f} ms/step, {decode_bytes(cfg, layers, b, c, elt) / sec / 1e9:.0f} GB/s")
            if chk is not None:
                # One request's logits must not depend on the 63 beside it beyond the rounding of bfloat16
                # operands summed in another order.  That rounding grows with the root of the depth:
                # measured on this shape against the engine's 32-bit path, bfloat16 differs by a mean of
                # 0.95e-3 of the logit range at 2 layers and 3.6e-3 at 32 (maximum 2.3e-2), a row in a
                # batch of 64 from the same row alone by 2.7e-3 (1.6e-2); a row computed from another
                # request's keys differs by its whole range.
                checks[f"{name}_row0_vs_alone"] = chk
                log(f"{name}: the first request's logits against the same request alone: {chk}")
                bound = 5e-3 * (max(layers, 2) / 32.0) ** 0.5
                if args.dtype == "bfloat16" and not (chk["mean"] <= bound and chk["max"] <= 10 * bound):
                    raise RuntimeError(f"{name}: a request's logits in the batch differ from the same request alone: {chk} "
                                       f"(allowed: mean {bound:.1e}, max {10 * bound:.1e} of the logit range)")
        for b in (1, 64):
            point(f"decode_b{b}", b, P, max(8, min(args.steps, 64)), min(args.warmup, 8), 3 + b, alone=b == 64)
        # away from the tuned point: long contexts (they end 128 tokens under the named length), and
        # a long prompt in portions
        for i, (c, b) in enumerate(ctx_points):
            # (the request admitted first decodes a token for every portion of the others' prompts;
            # it must not reach the model's limit before the last timed step)
            ahead = (b - 1) * -(-c // 2048) if c > 8192 else 0
            point(f"decode_b{b}_ctx{c}", b, c - 128 - ahead, long_steps if c <= 8192 else 16, long_warmup, 21 + i)
        for c, b in left_out:
            log(f"decode_b{b}_ctx{c}: left out, the cache of {b} such requests does not fit beside the weights "
                f"or the context is beyond the model's {ctx_max}")
        # short prompts (time to the first token's logits): steps of 128 and of 512 rows
        for T in (128, 512):
            short_s = measure_prefill(runner, cfg, T, repeats=5, seed=30 + T)
            points[f"prefill_{T}_tokens_ms"] = round(short_s * 1e3, 3)
            log(f"prefill {T} tokens: {short_s * 1e3:.2f} ms (the median of 5)")
        long_s = measure_prefill_in_portions(runner, cfg, long_T, 2048, seed=23)
        points[f"prefill_{long_T}_in_2048_portions"] = round(long_T / long_s, 1)
        log(f"prefill of {long_T} tokens in portions of 2048: {long_s * 1e3:.1f} ms, {long_T / long_s:.0f} tok/s")
    if args.mixed:
        # the workload twice: the first pass also records the decode graphs of its batch sizes (as the
        # warm-up steps do for the decode figures), the second is the figure; both are reported
        for name in ("mixed_first_pass_tok_s", "mixed_total_tok_s"):
            n_prompt, n_dec, secs, n_steps = measure_mixed(runner, cfg, args.mixed, 128, seed=9)
            log(f"mixed ({name}): {args.mixed} requests, {n_prompt} prompt + {n_dec} decoded tokens in {secs:.3f} s "
                f"({n_steps} steps): {(n_prompt + n_dec) / secs:.0f} tok/s in all, {n_dec / secs:.0f} decoded tok/s")
            points[name] = round((n_prompt + n_dec) / secs, 1)
    line = {
        "metric": f"decode tokens/s, {shape_name}, batch {B}, {P}-token prompts (random weights)",
        "value": round(tps, 1), "unit": "tokens/s", "n_gpus": 1, "steps": args.steps, "warmup": args.warmup,
        "ms_per_step": round(step_s * 1e3, 4), "higher_is_better": True, "scaling": "weak", "vs_baseline": None,
        "dtype": "bf16" if args.dtype == "bfloat16" else "fp32", "data": "synthetic",
        "config": {"model": shape_name, "layers": layers, "layers_in_config": layers_full,
                   "hidden_size": cfg["hidden_size"], "heads": cfg["num_attention_heads"],
                   "kv_heads": cfg["num_key_value_heads"], "head_dim": cfg["head_dim"],
                   "intermediate_size": cfg["intermediate_size"], "vocab_size": cfg["vocab_size"],
                   "global_batch": B, "seq_len": P, "max_context": cfg["max_position_embeddings"],
                   "decode_tokens": args.steps, "parallelism": "single GPU"},
        "prefill": {"value": round(2048 / pre_s, 1), "tokens": 2048, "ms": round(pre_s * 1e3, 3),
                    "frac": round(pre_rate / peak_flops, 4)},
        "roofline": {"bound": "hbm", "achieved": round(achieved, 1), "peak": PEAK["hbm_gbs"], "unit": "GB/s",
                     "frac": round(achieved / PEAK["hbm_gbs"], 4)},
        "points": points, "checks": checks,
        "repetitions_ms_per_step": [round(r[0] * 1e3, 4) for r in runs],
    }
    if read_gbs:
        # the same two figures against what this GPU gave a kernel that only reads, and the matrix
        # kernel on one large product, in this very run
        line["roofline"]["measured_peak"] = round(read_gbs, 1)
        line["roofline"]["frac_of_measured"] = round(achieved / read_gbs, 4)
        # no roofline, and it can exceed 1: the step's rate over that of this engine's own matrix
        # kernel on one large product
        line["prefill"]["own_gemm_tflops"] = round(mm_flops / 1e12, 1)
        line["prefill"]["frac_of_own_gemm"] = round(pre_rate / mm_flops, 4)
    text = json.dumps(line)
    print(text, flush=True)
    if args.record:
        with open(args.record, "w") as f:
            f.write(f"# bench.py, {shape_name}\n\nCommand:\n\n    python {' '.join(['bench.py'] + sys.argv[1:])}\n\n"
                    f"Result (one MI355X, random weights, synthetic tokens):\n\n```json\n{json.dumps(line, indent=1)}\n```\n")
    return 0


if __name__ == "__main__":
    sys.exit(main())
