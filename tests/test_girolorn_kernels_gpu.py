"""Every mechanism of the Girolorn parts alone: the kernel against the plain function of ``plain_girolorn`` (or a few
lines of float64 written here), with inputs made so that a fault shows: scores several times the soft cap, a sink that
outweighs every key beside one that none feels, pages handed out in shuffled order that start as NaN, rows whose mean
is far larger than what they vary by, branches on both sides of a clamp, biases that change the choice, and one key
that stands out hundreds of tokens back at page borders."""
import math

import numpy as np
import pytest
import torch

import plain_girolorn as P
from test_dinasun_kernels_gpu import close, dev
from test_kegorax_kernels_gpu import fill_pages
from test_kernels_gpu import FakeCtx, scatter_pages

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DT = {"float32": torch.float32, "bfloat16": torch.bfloat16}


@pytest.fixture(scope="module")
def ops():
    from xyntetik_runner_amd.csrc.ops import load_ops
    return load_ops()


# ----------------------------------------------------------------------------- attention with a soft cap
def plain_rows(q, k, v, start, scale, cap, sink, lo=None, keep=0, slopes=None):
    """Rows ``start ..`` of a request; ``lo(p)``: the first key position p may read; the first ``keep`` keys are always read."""
    T, H, _ = q.shape
    G, Dv = v.shape[1:]
    out = np.zeros((T, H, Dv))
    for t in range(T):
        p = start + t
        first = lo(p) if lo is not None else 0
        js = np.array(sorted(set(range(min(keep, p + 1))) | set(range(first, p + 1))))
        for h in range(H):
            g = h // (H // G)
            s = P.softcap((k[js, g] @ q[t, h]) * scale, cap)
            if slopes is not None:
                s = s - slopes[h] * (p - js)
            m = max(s.max(), sink[h])
            e = np.exp(s - m)
            out[t, h] = (e / (e.sum() + np.exp(sink[h] - m))) @ v[js, g]
    return out


MASKS = [(None, None, 0), (24, None, 0), (None, 20, 0), (None, 20, 3), (None, 70, 20)]          # chunk, window, kept first keys
SHAPES = [(4, 2, 32, 16), (8, 2, 64, 64), (3, 1, 10, 8), (2, 2, 16, 4), (5, 5, 80, 16), (4, 1, 128, 64), (2, 1, 24, 32)]   # H, Hk, D, page


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
@pytest.mark.parametrize("mask", MASKS)
@pytest.mark.parametrize("shape", SHAPES)
def test_attention_with_a_soft_cap(ops, dt, mask, shape):
    """A long portion from 0, a portion behind 150 keys, decoded tokens behind 37, 129 and 300 keys, in one batch;
    scores of about three times the cap, so that a cap that is left out, applied to the sink or applied behind the
    softmax's maximum shows."""
    H, Hk, D, ps = shape
    chunk, window, keep = mask
    rng = np.random.default_rng(H * 1000 + D + (chunk or 0) + 7 * (window or 0) + keep)
    starts, q_lens = [0, 150, 37, 129, 300], [140, 45, 1, 1, 1]
    lens = [s + n for s, n in zip(starts, q_lens)]
    tables, n_pages = scatter_pages(lens, ps, D + keep)
    ctx = FakeCtx(starts, q_lens, tables, ps)
    ks = [torch.tensor(rng.normal(size=(n, Hk, D))).to(DT[dt]) for n in lens]
    vs = [torch.tensor(rng.normal(size=(n, Hk, D))).to(DT[dt]) for n in lens]
    qs = [torch.tensor(rng.normal(size=(n, H, D)) * 3).to(DT[dt]) for n in q_lens]
    kc, vc = fill_pages(ks, vs, tables, n_pages, ps, DT[dt])
    sinks = rng.normal(size=H)
    sinks[0], sinks[-1] = 30.0, -30.0           # one that outweighs every key, one that none feels
    scale, cap = 1.1 / math.sqrt(D), 1.3
    q = torch.cat(qs).reshape(-1, H * D).contiguous().to(DEV)
    run = lambda c: ops.attention(q, kc, vc, ctx, 0, H, Hk, D, ps, scale, window, chunk=chunk, keep_first=keep,
                                  sinks=dev(sinks), softcap=c).float().cpu().numpy()
    lo = (lambda p: p - p % chunk) if chunk else ((lambda p: max(0, p - window + 1)) if window else None)
    want = np.concatenate([plain_rows(qs[b].double().numpy(), ks[b].double().numpy(), vs[b].double().numpy(), starts[b], scale, cap,
                                      sinks, lo, keep) for b in range(len(starts))]).reshape(-1, H * D)
    close(run(cap), want, 2e-5 if dt == "float32" else 2e-2, f"{shape} {mask}")
    assert np.abs(run(0.0) - want).max() > 0.2, "the inputs do not show the cap"


@pytest.mark.parametrize("D,ps", [(64, 64), (128, 64), (128, 32), (48, 64)])
@pytest.mark.parametrize("cap", [0.7, 5.0, 1000.0])
def test_long_portions_with_a_soft_cap(ops, D, ps, cap):
    """Portions of hundreds of rows behind and without earlier keys (whole tiles in the middle of an item, masked ones at
    its edges) in bfloat16: a cap that bends most scores, one that bends the largest, and one so wide that the scores
    come back as they are."""
    H, Hk = 4, 2
    rng = np.random.default_rng(D + int(cap))
    starts, q_lens = [0, 333], [520, 290]
    lens = [s + n for s, n in zip(starts, q_lens)]
    tables, n_pages = scatter_pages(lens, ps, D)
    ctx = FakeCtx(starts, q_lens, tables, ps)
    ks = [torch.tensor(rng.normal(size=(n, Hk, D))).to(torch.bfloat16) for n in lens]
    vs = [torch.tensor(rng.normal(size=(n, Hk, D))).to(torch.bfloat16) for n in lens]
    qs = [torch.tensor(rng.normal(size=(n, H, D)) * 2).to(torch.bfloat16) for n in q_lens]
    kc, vc = fill_pages(ks, vs, tables, n_pages, ps, torch.bfloat16)
    sinks = rng.normal(size=H)
    q = torch.cat(qs).reshape(-1, H * D).contiguous().to(DEV)
    scale = 1.0 / math.sqrt(D)
    got = ops.attention(q, kc, vc, ctx, 0, H, Hk, D, ps, scale, sinks=dev(sinks), softcap=cap).float().cpu().numpy()
    rows = np.concatenate([np.arange(0, n, 17) + o for n, o in zip(q_lens, (0, q_lens[0]))])
    want = []
    for b in range(2):
        full = P.attend(qs[b].double().numpy(), ks[b].double().numpy(), vs[b].double().numpy(), scale, cap, sinks)
        want.append(full.reshape(q_lens[b], -1))
    want = np.concatenate(want)
    close(got[rows], want[rows], 2e-2, f"{D} {cap}")
    close(got, want, 3e-2, f"{D} {cap}, every row")


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
def test_a_soft_cap_beside_slopes(ops, dt):
    """The bias of the distance is taken off the capped score."""
    H, Hk, D, ps = 4, 2, 32, 16
    rng = np.random.default_rng(3)
    starts, q_lens = [0, 80], [40, 1]
    lens = [s + n for s, n in zip(starts, q_lens)]
    tables, n_pages = scatter_pages(lens, ps, 1)
    ctx = FakeCtx(starts, q_lens, tables, ps)
    ks = [torch.tensor(rng.normal(size=(n, Hk, D))).to(DT[dt]) for n in lens]
    vs = [torch.tensor(rng.normal(size=(n, Hk, D))).to(DT[dt]) for n in lens]
    qs = [torch.tensor(rng.normal(size=(n, H, D)) * 2).to(DT[dt]) for n in q_lens]
    kc, vc = fill_pages(ks, vs, tables, n_pages, ps, DT[dt])
    sinks, slopes = rng.normal(size=H), np.array([0.5, 0.1, 0.02, 0.004])
    got = ops.attention(torch.cat(qs).reshape(-1, H * D).contiguous().to(DEV), kc, vc, ctx, 0, H, Hk, D, ps, 0.3, slopes=dev(slopes),
                        sinks=dev(sinks), softcap=1.5).float().cpu().numpy()
    want = np.concatenate([plain_rows(qs[b].double().numpy(), ks[b].double().numpy(), vs[b].double().numpy(), starts[b], 0.3, 1.5,
                                      sinks, slopes=slopes) for b in range(2)]).reshape(-1, H * D)
    close(got, want, 2e-5 if dt == "float32" else 2e-2, "cap and slopes")


@pytest.mark.parametrize("shape", [(1, 7), (3, 1000), (64, 4099)])
@pytest.mark.parametrize("cap", [0.5, 30.0])
def test_soft_cap_of_logits(ops, shape, cap):
    rng = np.random.default_rng(shape[1])
    z = rng.normal(size=shape) * 40
    x = torch.full((shape[0], shape[1] + 5), 7.0, device=DEV)
    x[:, 2:2 + shape[1]] = dev(z)
    ops.softcap_(x[:, 2:2 + shape[1]], cap)
    close(x[:, 2:2 + shape[1]].cpu().numpy(), P.softcap(z, cap), 3e-6, "soft cap")
    assert (x[:, :2] == 7.0).all() and (x[:, 2 + shape[1]:] == 7.0).all()


# ----------------------------------------------------------------------------- norm over all heads, rotation, cache write
@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
@pytest.mark.parametrize("case", [
    # H, Hk, D, rot, interleaved, page, rows of the requests: (start, length)
    (4, 2, 32, 16, True, 16, [(0, 20), (5, 1), (13, 30)]),
    (3, 1, 10, 6, True, 8, [(0, 1), (7, 9)]),
    (2, 2, 14, 14, True, 4, [(3, 6)]),
    (16, 4, 128, 128, True, 64, [(0, 1), (100, 1), (63, 1), (2047, 1)]),
    (16, 16, 64, 64, True, 64, [(0, 150), (61, 70)]),
    (3, 3, 6, 0, True, 16, [(2, 17)]),
    (4, 2, 32, 24, False, 16, [(0, 33), (9, 1)]),
    (8, 1, 20, 20, True, 2, [(1, 11)]),
])
def test_row_norm_rotation_and_cache_write(ops, dt, case):
    """Against the plain functions: all heads' queries over their one root mean square, the keys likewise, neighbouring
    or half-split pairs, the factor on cosines and sines on the rotated part only; the cached values are the keys
    before both, or rows of their own; aligned groups of eight positions and single tokens."""
    H, Hk, D, rot, inter, ps, reqs = case
    rng = np.random.default_rng(H * D + rot)
    starts, q_lens = [r[0] for r in reqs], [r[1] for r in reqs]
    lens = [s + n for s, n in zip(starts, q_lens)]
    tables, n_pages = scatter_pages(lens, ps, D)
    ctx = FakeCtx(starts, q_lens, tables, ps)
    T, Q, K = sum(q_lens), H * D, Hk * D
    proj = rng.normal(size=(T, Q + 2 * K)) * np.exp(rng.normal(size=(T, 1)))      # rows of different sizes
    wq, wk = 1 + 0.3 * rng.normal(size=Q), 1 + 0.3 * rng.normal(size=K)
    eps, mult = 1e-2, 1.37
    freq = 50.0 ** (-2.0 * np.arange(rot // 2) / max(rot, 1))
    pos = np.concatenate([np.arange(s, s + n) for s, n in zip(starts, q_lens)])

    def turned(x, w, heads):
        y = P.rms_norm(x, w, eps).reshape(T, heads, D)
        if not rot:
            return y
        order = np.arange(D)
        if not inter:           # pairs (j, j + rot/2): the neighbours of the permuted channels
            order[:rot] = np.arange(rot).reshape(2, rot // 2).T.reshape(-1)
        out = np.zeros_like(y)
        for t in range(T):
            # (the angle is the 32-bit product of the position and a 32-bit frequency)
            angle = (np.float32(pos[t]) * freq.astype(np.float32)).astype(np.float64)
            out[t:t + 1][..., order] = P.rotate_neighbours(y[t:t + 1][..., order], angle / max(1, pos[t]), mult, first=int(pos[t]))
        return out

    p = dev(proj)
    for values_are_keys in (True, False):
        kc = torch.full((n_pages, Hk, ps, D), float("nan"), dtype=DT[dt], device=DEV)
        vc = torch.full((n_pages, Hk, D, ps), float("nan"), dtype=DT[dt], device=DEV)
        v_in = p[:, Q:Q + K] if values_are_keys else p[:, Q + K:]
        q = ops.row_norm_rope_write(p[:, :Q], p[:, Q:Q + K], v_in, dev(wq), dev(wk), eps, kc, vc, ctx, 0,
                                    dev(freq) if rot else None, H, Hk, D, rot, inter, mult, ps, DT[dt])
        tol = 3e-6 if dt == "float32" else 6e-3
        close(q.float().cpu().numpy(), turned(proj[:, :Q], wq, H).reshape(T, Q), tol, "queries")
        got_k, got_v, t = np.zeros((T, Hk, D)), np.zeros((T, Hk, D)), 0
        kh, vh = kc.float().cpu().numpy(), vc.float().cpu().numpy()
        for b, (s, n) in enumerate(reqs):
            for x in range(s, s + n):
                pg = tables[b][x // ps]
                got_k[t], got_v[t] = kh[pg, :, x % ps, :], vh[pg, :, :, x % ps]
                t += 1
        close(got_k, turned(proj[:, Q:Q + K], wk, Hk), tol, "keys")
        raw = proj[:, Q:Q + K] if values_are_keys else proj[:, Q + K:]
        close(got_v, raw.reshape(T, Hk, D), 1e-7 if dt == "float32" else 4e-3, "values")
        assert np.isfinite(kh).sum() == T * K and np.isfinite(vh).sum() == T * K, "something else was written"
    close(ops.row_norm_rope_write(p[:, :Q], None, None, dev(wq), None, eps, None, None, ctx, 0, dev(freq) if rot else None, H, 0, D,
                                  rot, inter, mult, ps, DT[dt]).float().cpu().numpy(),
          turned(proj[:, :Q], wq, H).reshape(T, Q), tol, "queries alone")


@pytest.mark.parametrize("H,Hk,D", [(4, 2, 16), (3, 1, 10)])
def test_row_norm_as_a_transform_of_its_own(ops, H, Hk, D):
    """The transform in place, as an attention runs it whose values have another size than its keys."""
    from xyntetik_runner_amd.parts import RowRMSNorm, Runtime
    rng = np.random.default_rng(D)
    T = 9
    wq, wk = rng.normal(size=H * D), rng.normal(size=Hk * D)
    part = RowRMSNorm(H * D, Hk * D, 1e-3)
    part.bind({"q_norm": dev(wq), "k_norm": dev(wk)}, Runtime(torch.device(DEV), torch.float32, ops))
    x = rng.normal(size=(T, (H + Hk) * D))
    d = dev(x)
    part.apply(None, d[:, :H * D].unflatten(1, (H, D)), d[:, H * D:].unflatten(1, (Hk, D)))
    close(d[:, :H * D].cpu().numpy(), P.rms_norm(x[:, :H * D], wq, 1e-3), 3e-6, "queries")
    close(d[:, H * D:].cpu().numpy(), P.rms_norm(x[:, H * D:], wk, 1e-3), 3e-6, "keys")


# ----------------------------------------------------------------------------- layer norms
@pytest.mark.parametrize("out", ["float32", "bfloat16"])
@pytest.mark.parametrize("R,E", [(1, 4), (5, 30), (3, 1024), (200, 1024), (2, 4096), (130, 2052), (129, 8192), (4, 8192), (3, 9000), (7, 1027)])
def test_layer_norm(ops, R, E, out):
    """Rows whose mean is fifty times what they vary by: a variance made of the squares' mean loses it."""
    rng = np.random.default_rng(E)
    x = (rng.normal(size=(R + 2, E)) + 50.0 * rng.normal(size=(R + 2, 1))).astype(np.float32).astype(np.float64)
    w = 1 + 0.3 * rng.normal(size=E)
    rows = [int(r) for r in rng.permutation(R + 2)[:R]]
    tol = 2e-5 if out == "float32" else 5e-3
    close(ops.layernorm(dev(x), dev(w), 1e-5, DT[out]).float().cpu().numpy(), P.layer_norm(x, w, 1e-5), tol, "all rows")
    got = ops.layernorm(dev(x), None, 1e-5, DT[out], rows=dev(rows, torch.int32)).float().cpu().numpy()
    close(got, P.layer_norm(x[rows], np.ones(E), 1e-5), tol, "chosen rows without a weight")


@pytest.mark.parametrize("M", [1, 8, 16, 17, 40, 64, 65, 200, 512, 1100])
@pytest.mark.parametrize("N,K", [(256, 512), (2048, 1024), (100, 64)])
@pytest.mark.parametrize("centred", [True, False])
def test_product_into_the_stream_with_the_norm_behind_it(ops, M, N, K, centred):
    rng = np.random.default_rng(M + N)
    a = dev(rng.normal(size=(M, K)), torch.bfloat16)
    w = dev(rng.normal(size=(N, K)) / math.sqrt(K), torch.bfloat16)
    x0 = rng.normal(size=(M, N)) + (5.0 * rng.normal(size=(M, 1)) if centred else 0.0)
    x = dev(x0)
    nw = 1 + 0.2 * rng.normal(size=N)
    h = ops.linear_add_rmsnorm(a, ops.pack_weight(w), x, dev(nw), 1e-5, torch.bfloat16, centred=centred)
    want = x0 + a.double().cpu().numpy() @ w.double().cpu().numpy().T
    close(x.cpu().numpy(), want, 1e-5, "stream")
    close(h.float().cpu().numpy(), (P.layer_norm if centred else P.rms_norm)(want, nw, 1e-5), 6e-3, "norm")


# ----------------------------------------------------------------------------- experts
@pytest.mark.parametrize("T,n,top", [(1, 1, 1), (5, 3, 3), (33, 8, 2), (300, 17, 5), (4, 130, 64), (9, 1024, 8)])
def test_choice_by_the_logits(ops, T, n, top):
    """The router's bias enters the choice and the weights; the softmax is over the chosen logits alone; the column
    behind the experts' is no expert, however large, and its sigmoid comes back."""
    rng = np.random.default_rng(n + top)
    z = rng.normal(size=(T, n + 1)) * 3
    z[:, n] = np.where(np.arange(T) % 2, 50.0, -1.0)
    b = rng.normal(size=n) * 3
    wide = torch.zeros((T, n + 4), device=DEV)
    wide[:, 2:n + 3] = dev(z)
    idx, wts, side = ops.route_logits(wide[:, 2:n + 3], dev(b), top, scores="logits", side_gate=True)
    i2, w2 = ops.route_logits(wide[:, 2:n + 2], dev(b), top, scores="logits")
    assert torch.equal(idx, i2) and torch.equal(wts, w2)
    close(side.cpu().numpy(), P.sigmoid(z[:, n]), 1e-6, "the gate beside")
    zf = (z[:, :n].astype(np.float32) + b.astype(np.float32)).astype(np.float64)
    for t in range(T):
        chosen, want = P.choose(zf[t], top)
        assert list(idx[t].cpu().numpy()) == list(chosen), f"row {t}"
        close(wts[t].cpu().numpy(), want, 3e-6, f"weights of row {t}")


def test_choice_by_the_logits_at_ties_and_no_numbers(ops):
    z = torch.tensor([[1.0, 2.0, 2.0, 2.0], [float("nan"), 1.0, float("nan"), 3.0], [float("nan")] * 4,
                      [-float("inf"), -1e30, 0.0, -float("inf")]], device=DEV)
    idx, wts = ops.route_logits(z, torch.zeros(4, device=DEV), 3, scores="logits")
    assert idx[0].tolist() == [1, 2, 3] and idx[1].tolist()[:2] == [3, 1]
    assert sorted(set(idx[2].tolist())) == [0, 1, 2] and (idx >= 0).all() and (idx < 4).all()
    assert torch.isfinite(wts).all() and torch.allclose(wts.sum(dim=1), torch.ones(4, device=DEV))
    assert idx[3].tolist()[:2] == [2, 1] and wts[3, 0] == 1.0


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
@pytest.mark.parametrize("T,E,F,n,top", [(1, 64, 24, 8, 2), (3, 40, 12, 3, 3), (7, 30, 9, 4, 1), (40, 96, 64, 5, 2), (64, 256, 128, 16, 2),
                                         (700, 128, 96, 4, 2), (500, 136, 40, 2, 1), (90, 64, 8, 40, 5), (300, 1028, 72, 3, 2)])
def test_clamped_experts_with_a_gated_row_beside_and_the_norm_behind(ops, dt, T, E, F, n, top):
    """Both paths (a few choices; sorted on the matrix cores with the gate in the first product's epilogue): branches well
    beyond the limit on both sides, the shared rows times the token's gate, the sum into rows that are already there,
    and the norm of what then stands."""
    rng = np.random.default_rng(E + F)
    h = dev(rng.normal(size=(T, E)), DT[dt])
    up = dev(rng.normal(size=(n, 2 * F, E)) * 1.2 / math.sqrt(E), DT[dt])
    down = dev(rng.normal(size=(n, E, F)) / math.sqrt(F), DT[dt])
    idx = dev(np.stack([rng.permutation(n)[:top] for _ in range(T)]), torch.int32)
    wts = rng.random((T, top))
    side, gate = rng.normal(size=(T, E)), rng.random(T)
    limit = 0.6
    hd, ud, dd = (x.double().cpu().numpy() for x in (h, up, down))
    want = np.zeros((T, E))
    for t in range(T):
        for j in range(top):
            e = int(idx[t, j])
            w = {"gate": ud[e, :F], "up": ud[e, F:], "down": dd[e]}
            want[t] += wts[t, j] * P.clamped_expert(hd[t], w, "", limit)
    tol = 5e-6 if dt == "float32" else 1.5e-2
    close(ops.moe_experts(h, up, down, idx, dev(wts), activation="clamped_swish", param=limit).cpu().numpy(), want, tol, "experts")
    base = rng.normal(size=(T, E)) + 2.0
    want = base + want + gate[:, None] * side
    nw = 1 + 0.2 * rng.normal(size=E)
    for centred in (True, False):
        x = dev(base)
        got = ops.moe_experts(h, up, down, idx, dev(wts), out=x, accumulate=True, activation="clamped_swish", param=limit,
                              beside=(dev(side), dev(gate)), norm=(dev(nw), 1e-5, centred))
        close(x.cpu().numpy(), want, tol, "stream")
        assert got.dtype == DT[dt]
        close(got.float().cpu().numpy(), (P.layer_norm if centred else P.rms_norm)(want, nw, 1e-5), 2 * tol, "norm")


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
@pytest.mark.parametrize("act", ["swiglu", "gelu_tanh", "clamped_swish"])
def test_every_gate_in_the_experts(ops, dt, act):
    """The same gates by both paths, and as ``gate_mul`` makes them."""
    rng = np.random.default_rng(11)
    E, F, n = 64, 48, 3
    up, down = dev(rng.normal(size=(n, 2 * F, E)) * 0.3, DT[dt]), dev(rng.normal(size=(n, E, F)) * 0.3, DT[dt])
    for T in (2, 60):
        h = dev(rng.normal(size=(T, E)), DT[dt])
        idx, wts = dev(rng.integers(0, n, size=(T, 1)), torch.int32), torch.ones((T, 1), device=DEV)
        got = ops.moe_experts(h, up, down, idx, wts, activation=act, param=0.9).cpu().numpy()
        for t in range(T):
            e = int(idx[t, 0])
            gu = (h[t].float() @ up[e].float().T)[None]
            z = ops.gate_mul(gu, {"swiglu": "silu"}.get(act, act), 0.9).double().cpu().numpy()[0]
            close(got[t], down[e].double().cpu().numpy() @ z, 1e-5 if dt == "float32" else 1.5e-2, f"{act} {T} row {t}")


# ----------------------------------------------------------------------------- a one-layer model with made weights
def needle_model(cap, sinks):
    """One layer of attention, two heads on two key heads of four channels of which the first two turn, no feed-forward.
    Every query lies along channel 3 of both heads, whatever the token; a filler's key (token 0) has nothing there and the
    needle's (token 1) has, so that the norm over both heads makes its score the same wherever it stands.  The needle's
    value, its key as projected, is brought by head 0 to stream channel 5, which row 3 of the head reads."""
    E, V, H, D = 8, 4, 2, 4
    rng = np.random.default_rng(4)
    m = {"heads": H, "kv_heads": H, "dim": D, "vdim": D, "scale": 1.0, "rot": {"base": 100.0, "dims": 2}}
    if cap is not None:
        m["softcap"] = cap
    cfg = {"architecture": "Girolorn", "vocab": V, "width": E, "norm": {"eps": 1e-6}, "layers": [{"type": "attention", "mixer": m, "mlp": None}]}
    emb = np.zeros((V, E)); emb[0, :2] = 1.0, -1.0; emb[1, :2] = -1.0, 1.0; emb[2, 4] = 1.0; emb[3, 5] = 1.0
    emb[:, 2] = 0.5; emb[:, 3] = -0.5                   # alike in every token: what the queries read
    p = "l0.mix."
    wq, wk = np.zeros((H * D, E)), rng.normal(size=(H * D, E)) * 0.01
    for c in (0, D):
        wq[c + 3, 2:4] = 1.0, -1.0
        wk[c + 2, :2] = 1.0, -1.0
        wk[c + 3, :4] = 1.0, 2.0, 1.0, -1.0             # a filler: 1 - 2 + 1/2 + 1/2 = 0, the needle: -1 + 2 + 1/2 + 1/2 = 2
    o = rng.normal(size=(E, H * D)) * 0.01
    o[5, 3] = 4.0
    w = {"embed": emb, "l0.norm1": np.ones(E), "final.norm": np.ones(E), "head": emb.copy(), p + "q": wq, p + "k": wk,
         p + "q.norm": np.full(H * D, 3.0), p + "k.norm": np.full(H * D, 2.0), p + "sink": np.asarray(sinks, dtype=np.float64), p + "o": o}
    return cfg, w


@pytest.mark.parametrize("page", [16, 64])
@pytest.mark.parametrize("decode_from", [None, 30])
@pytest.mark.parametrize("cap,sink", [(None, -2.0), (9.0, -2.0), (9.0, 12.0)])
def test_a_far_token_that_stands_out_through_the_engine(tmp_path, page, decode_from, cap, sink):
    """The needle 600 tokens back at a page's first and last place: read whole without a cap, among hundreds of fillers
    with one, and drowned by a large sink; in a prompt's portions and with all but 30 positions decoded one by one."""
    import io
    import traces
    from xyntetik_runner_amd.config import config_from_dict
    from xyntetik_runner_amd.engine.runner import ModelRunner
    from xyntetik_runner_amd.trace import replay
    cfg, w = needle_model(cap, [sink, sink])
    n = 680
    for jstar in (63, 64):
        toks = [0] * n
        toks[jstar] = 1
        want = P.forward(cfg, w, toks)
        without = P.forward(cfg, w, [0] * n)
        if sink < 0:
            assert abs(want[-1, 3] - without[-1, 3]) > 0.05, "the made weights do not show the needle"
        if decode_from is None:
            steps = traces.portions({"a": toks}, sizes=(17, 2, 40, 3, 400, 64))
        else:
            steps = traces.tail_one_by_one({"a": toks}, tail=n - decode_from)
        arch, typed = config_from_dict(cfg)
        tensors = {k: torch.tensor(v, dtype=torch.float32) for k, v in w.items()}
        runner = ModelRunner(arch.build_spec(typed), tensors, "float32", max_tokens=n + 64, page_size=page, max_requests=2,
                             max_step_tokens=400)
        for lc in runner.storage.layers:
            lc.k.fill_(float("nan")); lc.v.fill_(float("nan"))
        out = str(tmp_path / f"out{jstar}")
        replay(runner, traces.to_lines(steps), out, report=io.StringIO())
        runner.manager.check()
        got = traces.collect(steps, out, cfg["vocab"])
        close(got["a"], want, 1e-5, f"needle at {jstar}")


# ----------------------------------------------------------------------------- whole models at a sequence's start
def test_first_tokens_of_a_sequence(tmp_path):
    """Sequences of one, two and three tokens beside a longer one in a mixed batch: position 0 reads itself and the sink
    alone, and is not turned."""
    import io
    import traces
    from girolorn_tiny import make_model
    from plain_llama import load_folder
    from xyntetik_runner_amd.engine.runner import ModelRunner
    from xyntetik_runner_amd.trace import replay
    for which in ("G1", "G2", "G4"):
        d = make_model(which, str(tmp_path / which))
        cfg, w = load_folder(d)
        reqs = {f"r{n}": [int(t) for t in np.random.default_rng(n).integers(0, cfg["vocab"], size=n)] for n in (1, 2, 3, 30)}
        steps = traces.mixed(reqs, {k: min(2, len(v)) for k, v in reqs.items()}, max_live=4, seed=1)
        runner = ModelRunner.from_folder(d, dtype="float32", max_tokens=256, page_size=16, max_requests=4)
        out = str(tmp_path / (which + "out"))
        replay(runner, traces.to_lines(steps), out, report=io.StringIO())
        got = traces.collect(steps, out, cfg["vocab"])
        for rid, toks in reqs.items():
            close(got[rid], P.forward(cfg, w, toks), 2e-5, f"{which} {rid}")
