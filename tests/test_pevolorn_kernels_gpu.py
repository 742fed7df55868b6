"""Every mechanism of the Pevolorn parts alone: the kernel against the plain function of ``plain_pevolorn`` (or a few lines
of float64 written here), with rows cut into requests and steps the way an engine cuts them, and with inputs made so that a
fault shows: pages handed out in shuffled order that start as NaN, values of another size than keys, gates that open and
close heads, a state that never decays beside one that forgets at once and sums of decays in the thousands, state rows of
other requests that are garbage, choice scores below zero, identity experts among the chosen, and one token that stands out
hundreds of tokens back at page borders in a layer's own rows and in another layer's."""
import io
import math

import numpy as np
import pytest
import torch

import plain_pevolorn as P
import traces
from test_dinasun_kernels_gpu import close, dev, step_ctx
from test_kegorax_kernels_gpu import fill_pages, run_in_steps
from test_kernels_gpu import FakeCtx, scatter_pages

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DT = {"float32": torch.float32, "bfloat16": torch.bfloat16}


@pytest.fixture(scope="module")
def ops():
    from xyntetik_runner_amd.csrc.ops import load_ops
    return load_ops()


# ----------------------------------------------------------------------------- attention: values of another size, a gate
SHAPES = [  # H, Hk, D, Dv, page
    (6, 2, 64, 48, 64), (4, 4, 64, 32, 16), (6, 1, 48, 32, 32), (2, 1, 16, 32, 16), (4, 2, 32, 16, 64), (8, 1, 80, 64, 64),
    (5, 1, 144, 96, 64), (16, 1, 256, 192, 64), (3, 1, 10, 14, 8), (2, 2, 24, 16, 16), (4, 2, 64, 64, 64), (3, 3, 64, 48, 4)]


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
@pytest.mark.parametrize("cap", [0.0, 1.6])
@pytest.mark.parametrize("shape", SHAPES)
def test_attention_with_values_of_another_size_and_a_gate(ops, dt, cap, shape):
    """A portion from 0, one behind 150 keys, decoded tokens behind 37, 129 and 700 keys, in one batch, into a column range of
    wider rows; gates from closed to open; whatever the work is split into, the gate and the factor come once."""
    H, Hk, D, Dv, ps = shape
    rng = np.random.default_rng(H * 1000 + D + Dv)
    starts, q_lens = [0, 150, 37, 129, 700], [140, 45, 1, 1, 1]
    lens = [s + n for s, n in zip(starts, q_lens)]
    tables, n_pages = scatter_pages(lens, ps, D)
    ctx = FakeCtx(starts, q_lens, tables, ps)
    ks = [torch.tensor(rng.normal(size=(n, Hk, D))).to(DT[dt]) for n in lens]
    vs = [torch.tensor(rng.normal(size=(n, Hk, Dv))).to(DT[dt]) for n in lens]
    qs = [torch.tensor(rng.normal(size=(n, H, D)) * 2).to(DT[dt]) for n in q_lens]
    kc, vc = fill_pages(ks, vs, tables, n_pages, ps, DT[dt])
    T = sum(q_lens)
    gates = rng.normal(size=(T, H + 3)) * 2
    gates[:, 1] = 30.0              # a head that is open
    gates[::3, 2] = -30.0           # and one that is closed for every third token
    out = torch.full((T, H * Dv + 24), 5.0, dtype=DT[dt], device=DEV)
    q = torch.cat(qs).reshape(-1, H * D).contiguous().to(DEV)
    scale = 1.2 / math.sqrt(D)
    back = ops.attention(q, kc, vc, ctx, 0, H, Hk, D, ps, scale, v_head_dim=Dv, softcap=cap, gate=dev(gates)[:, 1:1 + H],
                         out_scale=-1.3, out=out[:, 8:8 + H * Dv])
    assert back.data_ptr() == out[:, 8:].data_ptr()
    want = np.concatenate([P.attend(qs[b].double().numpy(), ks[b].double().numpy(), vs[b].double().numpy(), scale, cap)
                           for b in range(len(starts))])
    gated = -1.3 * want * P.sigmoid(gates[:, 1:1 + H])[:, :, None]
    tol = 2e-5 if dt == "float32" else 2e-2
    close(out[:, 8:8 + H * Dv].float().cpu().numpy(), gated.reshape(T, -1), tol, f"{shape} gated")
    assert (out[:, :8] == 5.0).all() and (out[:, 8 + H * Dv:] == 5.0).all(), "written beside the range"
    bare = ops.attention(q, kc, vc, ctx, 0, H, Hk, D, ps, scale, v_head_dim=Dv, softcap=cap)
    close(bare.float().cpu().numpy(), want.reshape(T, -1), tol, f"{shape} as it is")


@pytest.mark.parametrize("H,Hk,D,Dv,ps", [(6, 3, 64, 48, 64), (16, 1, 256, 192, 64), (2, 2, 64, 32, 32)])
def test_long_portions_with_values_of_another_size(ops, H, Hk, D, Dv, ps):
    """Whole tiles in the middle of an item and masked ones at its edges, items that are split and merged."""
    rng = np.random.default_rng(D + Dv)
    starts, q_lens = [0, 333, 2100], [300, 170, 40]
    lens = [s + n for s, n in zip(starts, q_lens)]
    tables, n_pages = scatter_pages(lens, ps, D)
    ctx = FakeCtx(starts, q_lens, tables, ps)
    ks = [torch.tensor(rng.normal(size=(n, Hk, D))).to(torch.bfloat16) for n in lens]
    vs = [torch.tensor(rng.normal(size=(n, Hk, Dv))).to(torch.bfloat16) for n in lens]
    qs = [torch.tensor(rng.normal(size=(n, H, D)) * 2).to(torch.bfloat16) for n in q_lens]
    kc, vc = fill_pages(ks, vs, tables, n_pages, ps, torch.bfloat16)
    gate = rng.normal(size=(sum(q_lens), H))
    q = torch.cat(qs).reshape(-1, H * D).contiguous().to(DEV)
    got = ops.attention(q, kc, vc, ctx, 0, H, Hk, D, ps, D ** -0.5, v_head_dim=Dv, gate=dev(gate)).float().cpu().numpy()
    want = np.concatenate([P.attend(qs[b].double().numpy(), ks[b].double().numpy(), vs[b].double().numpy(), D ** -0.5) for b in range(3)])
    close(got, (want * P.sigmoid(gate)[:, :, None]).reshape(got.shape), 2e-2, "long portions")


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
@pytest.mark.parametrize("H,D,Dv,ps", [(3, 544, 520, 16), (2, 1024, 1000, 64), (2, 600, 600, 4)])
def test_rows_longer_than_the_matrix_cores_take(ops, dt, H, D, Dv, ps):
    rng = np.random.default_rng(D)
    starts, q_lens = [0, 60], [70, 1]
    lens = [s + n for s, n in zip(starts, q_lens)]
    tables, n_pages = scatter_pages(lens, ps, D)
    ctx = FakeCtx(starts, q_lens, tables, ps)
    ks = [torch.tensor(rng.normal(size=(n, 1, D))).to(DT[dt]) for n in lens]
    vs = [torch.tensor(rng.normal(size=(n, 1, Dv))).to(DT[dt]) for n in lens]
    qs = [torch.tensor(rng.normal(size=(n, H, D)) * 2).to(DT[dt]) for n in q_lens]
    kc, vc = fill_pages(ks, vs, tables, n_pages, ps, DT[dt])
    q = torch.cat(qs).reshape(-1, H * D).contiguous().to(DEV)
    got = ops.attention_pooled(q, kc, vc, None, None, ctx, 0, None, H, 1, D, Dv, ps, D ** -0.5, 1 << 30, 0, matrix_cores=False)
    want = np.concatenate([P.attend(qs[b].double().numpy(), ks[b].double().numpy(), vs[b].double().numpy(), D ** -0.5) for b in range(2)])
    close(got.float().cpu().numpy(), want.reshape(-1, H * Dv), 2e-5 if dt == "float32" else 1e-2, "wide rows")


# ----------------------------------------------------------------------------- rotation, head norms, cache write
def turned_half(x, pos, freq, mult, inter, rot):
    """``x [T, heads, D]``: the rotation with the angle as the 32-bit product of the position and a 32-bit frequency."""
    half = rot // 2
    out = np.array(x)
    a = (np.float32(pos)[:, None] * np.float32(freq)[None, :]).astype(np.float64)
    c, s = np.cos(a)[:, None, :] * mult, np.sin(a)[:, None, :] * mult
    i0 = np.arange(half) * 2 if inter else np.arange(half)
    i1 = i0 + 1 if inter else i0 + half
    out[..., i0] = x[..., i0] * c - x[..., i1] * s
    out[..., i1] = x[..., i1] * c + x[..., i0] * s
    return out


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
@pytest.mark.parametrize("norm", [None, "before", "after"])
@pytest.mark.parametrize("case", [
    # H, Hk, D, Dv, rot, interleaved, page, rows of the requests: (start, length)
    (4, 2, 32, 16, 16, False, 16, [(0, 20), (5, 1), (13, 30)]),
    (3, 1, 10, 14, 6, False, 8, [(0, 1), (7, 9)]),
    (2, 2, 14, 6, 14, True, 4, [(3, 6)]),
    (16, 4, 128, 128, 64, False, 64, [(0, 1), (100, 1), (63, 1), (2047, 1)]),
    (8, 2, 200, 24, 200, False, 64, [(0, 130), (61, 70)]),
    (3, 3, 6, 9, 0, False, 16, [(2, 17)]),
    (2, 1, 256, 256, 128, False, 2, [(1, 11)]),
])
def test_rotation_head_norm_and_cache_write(ops, dt, norm, case):
    """Queries and keys rotated, every head over its own root mean square before or behind the rotation, with weights and
    without, values of their own size to their pages (aligned groups of eight positions and single tokens)."""
    H, Hk, D, Dv, rot, inter, ps, reqs = case
    rng = np.random.default_rng(H * D + rot)
    starts, q_lens = [r[0] for r in reqs], [r[1] for r in reqs]
    lens = [s + n for s, n in zip(starts, q_lens)]
    tables, n_pages = scatter_pages(lens, ps, D)
    ctx = FakeCtx(starts, q_lens, tables, ps)
    T, Q, K, V = sum(q_lens), H * D, Hk * D, Hk * Dv
    proj = rng.normal(size=(T, Q + K + V + 3)) * np.exp(rng.normal(size=(T, 1)))
    freq = 50.0 ** (-2.0 * np.arange(rot // 2) / max(rot, 1))
    pos = np.concatenate([np.arange(s, s + n) for s, n in zip(starts, q_lens)])
    eps, mult = 1e-2, 1.0 if norm == "after" else 1.31
    p = dev(proj)
    tol = 3e-6 if dt == "float32" else 6e-3
    for weighted in (True, False) if norm else (False,):
        wq, wk = (1 + 0.3 * rng.normal(size=D), 1 + 0.3 * rng.normal(size=D)) if weighted else (np.ones(D), np.ones(D))

        def expect(x, w, heads):
            y = x.reshape(T, heads, D)
            if norm == "before":
                y = P.rms_div(y, eps) * w
            y = turned_half(y, pos, freq, mult, inter, rot)
            return P.rms_div(y, eps) * w if norm == "after" else y

        kc = torch.full((n_pages, Hk, ps, D), float("nan"), dtype=DT[dt], device=DEV)
        vc = torch.full((n_pages, Hk, Dv, ps), float("nan"), dtype=DT[dt], device=DEV)
        how = (dev(wq) if weighted else None, dev(wk) if weighted else None, eps, norm)
        args = (ctx, 0, dev(freq) if rot else None)
        q = ops.head_norm_rope_write(p[:, :Q], p[:, Q:Q + K], p[:, Q + K:Q + K + V], *how, kc, vc, *args, H, Hk, D, Dv, rot, inter, mult, ps, DT[dt])
        close(q.float().cpu().numpy(), expect(proj[:, :Q], wq, H).reshape(T, Q), tol, "queries")
        got_k, got_v, t = np.zeros((T, Hk, D)), np.zeros((T, Hk, Dv)), 0
        kh, vh = kc.float().cpu().numpy(), vc.float().cpu().numpy()
        for b, (s, n) in enumerate(reqs):
            for x in range(s, s + n):
                pg = tables[b][x // ps]
                got_k[t], got_v[t] = kh[pg, :, x % ps, :], vh[pg, :, :, x % ps]
                t += 1
        close(got_k, expect(proj[:, Q:Q + K], wk, Hk), tol, "keys")
        close(got_v, proj[:, Q + K:Q + K + V].reshape(T, Hk, Dv), 1e-7 if dt == "float32" else 4e-3, "values")
        assert np.isfinite(kh).sum() == T * K and np.isfinite(vh).sum() == T * V, "something else was written"
        alone = ops.head_norm_rope_write(p[:, :Q], None, None, *how, None, None, *args, H, 0, D, Dv, rot, inter, mult, ps, DT[dt])
        assert torch.equal(alone, q), "queries alone"


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
@pytest.mark.parametrize("H,D,R,C,dims,whole", [(3, 10, 8, 14, 8, False), (2, 16, 16, 48, 16, False), (4, 7, 12, 20, 8, True), (2, 5, 4, 9, 0, False),
                                                 (8, 128, 64, 192, 64, False)])
def test_latent_rows_rotated_in_halves(ops, dt, H, D, R, C, dims, whole):
    """The latent normed and cached with the rotated shared part, queries rotated in pairs (i, i + dims/2), channels behind
    ``dims`` as they are; a layer that stores nothing gets the same queries."""
    rng = np.random.default_rng(C + R)
    starts, q_lens, ps = [5, 0], [1, 19], 8
    lens = [s + n for s, n in zip(starts, q_lens)]
    tables, n_pages = scatter_pages(lens, ps, C)
    ctx = FakeCtx(starts, q_lens, tables, ps)
    T = sum(q_lens)
    pos = np.concatenate([np.arange(s, s + n) for s, n in zip(starts, q_lens)])
    freq = 30.0 ** (-2.0 * np.arange(dims // 2) / max(dims, 1))
    down = rng.normal(size=(T, H * (D + R) + C + R + 5))
    w = 1 + 0.3 * rng.normal(size=C)
    p, Q = dev(down), H * (D + R)
    kc = torch.full((n_pages, 1, ps, C + R), float("nan"), dtype=DT[dt], device=DEV)
    vc = torch.full((n_pages, 1, C + R if whole else C, ps), float("nan"), dtype=DT[dt], device=DEV)
    q_out = torch.zeros((T, H * (C + R)), dtype=DT[dt], device=DEV)
    inv = dev(freq) if dims else None
    qn = ops.latent_prepare(p[:, :Q], p[:, Q:Q + C + R], dev(w), 1e-3, q_out, kc, vc, ctx, 0, inv, H, D, R, C, dims, ps, halves=True)
    q3, kv = down[:, :Q].reshape(T, H, D + R), down[:, Q:Q + C + R]
    row = np.concatenate([P.rms_div(kv[:, :C], 1e-3) * w, turned_half(kv[:, None, C:], pos, freq, 1.0, False, dims)[:, 0]], axis=1)
    tol = 3e-6 if dt == "float32" else 6e-3
    close(qn.float().cpu().numpy(), q3[..., :D].reshape(T, -1), 1e-7 if dt == "float32" else 4e-3, "unrotated")
    close(q_out.float().cpu().numpy().reshape(T, H, C + R)[..., C:], turned_half(q3[..., D:], pos, freq, 1.0, False, dims), tol, "rotated")
    kh, vh, t = kc.float().cpu().numpy(), vc.float().cpu().numpy(), 0
    got_k, got_v = np.zeros((T, C + R)), np.zeros((T, vh.shape[2]))
    for b, (s, n) in enumerate(zip(starts, q_lens)):
        for x in range(s, s + n):
            pg = tables[b][x // ps]
            got_k[t], got_v[t] = kh[pg, 0, x % ps], vh[pg, 0, :, x % ps]
            t += 1
    close(got_k, row, tol, "cached rows")
    close(got_v, row[:, :vh.shape[2]], tol, "and transposed")
    assert np.isfinite(kh).sum() == T * (C + R)
    again = torch.zeros_like(q_out)
    before = kc.clone()
    qn2 = ops.latent_prepare(p[:, :Q], None, None, 1e-3, again, kc, vc, ctx, 0, inv, H, D, R, C, dims, ps, halves=True)
    assert torch.equal(qn2, qn) and torch.equal(again, q_out) and torch.equal(before.nan_to_num(7.0), kc.nan_to_num(7.0))


# ----------------------------------------------------------------------------- the state space
def ssd_case(rng, lens, H, G, N, Dv):
    """(rows [x | B | C | z] of every request, constants [3, H]): head 0 never forgets, head 1 forgets at once (its sums of
    decays go into the thousands), the others lie between."""
    consts = np.stack([np.exp(rng.normal(size=H)), rng.normal(size=H) - 1.0, rng.normal(size=H)])
    consts[0, 0] = 1e-7
    if H > 1:
        consts[0, 1], consts[1, 1] = 400.0, 1.0
    return [rng.normal(size=(L, H * Dv + 2 * G * N + H)) for L in lens], consts


def ssd_want(rows, consts, H, G, N, Dv):
    out = []
    I = H * Dv
    for x in rows:
        dt = P.softplus(x[:, I + 2 * G * N:] + consts[1])
        y = []
        for h in range(H):
            g = h // (H // G)
            xs = x[:, h * Dv:(h + 1) * Dv]
            y.append(P.state_space(xs, x[:, I + g * N:I + (g + 1) * N], x[:, I + (G + g) * N:I + (G + g + 1) * N], dt[:, h], consts[0, h])
                     + consts[2, h] * xs)
        out.append(np.stack(y, axis=1).reshape(x.shape[0], I))
    return out


def ssd_calls(ops, consts, state, H, G, N, Dv):
    I, W = H * Dv, H * Dv + 2 * G * N
    c = dev(consts)
    scalar = lambda ctx, r: ops.linear_recurrence("ssd", r[:, I + G * N:W], r[:, I:I + G * N], r[:, :I], state, ctx, H, G, N, Dv,
                                                  gate=r[:, W:], decay=c)
    chunks = lambda ctx, r: ops.ssd_chunks(r[:, :W].to(torch.bfloat16).contiguous(), r[:, W:], c, state, ctx, H, G, N, Dv)
    return scalar, chunks


SSD_SIZES = [(4, 2, 24, 16), (3, 3, 5, 7), (4, 1, 64, 32), (2, 1, 128, 64), (6, 3, 40, 10)]


@pytest.mark.parametrize("H,G,N,Dv", SSD_SIZES)
def test_state_space_in_portions(ops, H, G, N, Dv):
    from xyntetik_runner_amd.csrc.ops import Ops
    rng = np.random.default_rng(H * 100 + N)
    lens = [70, 31]
    rows, consts = ssd_case(rng, lens, H, G, N, Dv)
    state = torch.full((4,) + Ops.recurrence_state_shape(H, N, Dv), float("nan"), device=DEV)
    state[0] = 0.0
    state[2] = 0.0
    scalar, _ = ssd_calls(ops, consts, state, H, G, N, Dv)
    got = run_in_steps(ops, [(33, 2), (1, 1), (1, 1), (2, 20), (30, 1), (1, 1), (1, 1), (1, 1), (1, 4)], lens, [0, 2], rows, scalar)
    for r, want in enumerate(ssd_want(rows, consts, H, G, N, Dv)):
        close(got[r], want, 5e-6, f"request {r}")
    assert torch.isnan(state[1]).all() and torch.isnan(state[3]).all()


@pytest.mark.parametrize("H,G,N,Dv", [(2, 1, 64, 32), (3, 3, 16, 24)])
def test_state_space_over_long_portions_in_32_bits(ops, H, G, N, Dv):
    """Portions from 1,024 rows on in chunks side by side; a write far back is kept by the head that never forgets."""
    from xyntetik_runner_amd.csrc.ops import Ops
    rng = np.random.default_rng(N)
    lens = [1300, 40, 2100]
    rows, consts = ssd_case(rng, lens, H, G, N, Dv)
    for x in rows:
        x[3, H * Dv:H * Dv + N] *= 30.0
    state = torch.full((5,) + Ops.recurrence_state_shape(H, N, Dv), float("nan"), device=DEV)
    for sl in (4, 0, 2):
        state[sl] = 0.0
    scalar, _ = ssd_calls(ops, consts, state, H, G, N, Dv)
    got = run_in_steps(ops, [(1100, 40, 1024), (200, 0, 1076)], lens, [4, 0, 2], rows, scalar)
    for r, want in enumerate(ssd_want(rows, consts, H, G, N, Dv)):
        close(got[r], want, 3e-5, f"request {r}")


@pytest.mark.parametrize("H,G,N,Dv", [(4, 2, 24, 16), (4, 1, 64, 32), (2, 1, 128, 64), (6, 3, 40, 24), (2, 2, 256, 72), (3, 1, 8, 8), (2, 1, 136, 128)])
def test_state_space_in_chunks_on_the_matrix_cores(ops, H, G, N, Dv):
    """The rows (made of bfloat16 numbers, so that nothing is lost on the way in) in portions that end inside, at and one
    past a chunk's edge, beside single rows, in turn with the kernel that runs token by token: one state for both.  All
    that is 32-bit stays so: the error is that of two bfloat16 parts a number, not of one."""
    from xyntetik_runner_amd.csrc.ops import Ops
    rng = np.random.default_rng(H * 100 + N + Dv)
    lens = [400, 300, 130]
    rows, consts = ssd_case(rng, lens, H, G, N, Dv)
    W = H * Dv + 2 * G * N
    for x in rows:
        x[:, :W] = torch.tensor(x[:, :W]).to(torch.bfloat16).double().numpy()
        x[3, H * Dv:H * Dv + N] = 16.0          # a write that the head which never forgets keeps
    state = torch.full((5,) + Ops.recurrence_state_shape(H, N, Dv), float("nan"), device=DEV)
    slots = [4, 0, 2]
    for sl in slots:
        state[sl] = 0.0
    scalar, chunks = ssd_calls(ops, consts, state, H, G, N, Dv)
    turn = [0]

    def call(ctx, r):
        turn[0] += 1
        return (scalar if turn[0] in (2, 5) else chunks)(ctx, r)

    plan = [(128, 1, 129), (1, 1, 1), (127, 256, 0), (2, 1, 0), (1, 1, 0), (141, 40, 0)]
    got = run_in_steps(ops, plan, lens, slots, rows, call)
    for r, want in enumerate(ssd_want(rows, consts, H, G, N, Dv)):
        close(got[r], want, 2e-5, f"request {r}")
    assert torch.isnan(state[1]).all() and torch.isnan(state[3]).all()


@pytest.mark.parametrize("out", ["float32", "bfloat16"])
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 5])
def test_convolution_with_a_bias(ops, taps, out):
    """Three requests in portions down to one row, one long enough for the kernel that takes eight rows a thread, others of
    one row each; neighbours' carried inputs are garbage."""
    rng = np.random.default_rng(taps)
    C, lens = 300, [150, 20, 90]
    w, b = rng.normal(size=(C, taps)), rng.normal(size=C)
    rows = [rng.normal(size=(L, C)) for L in lens]
    state = torch.full((5, max(1, taps - 1), C), float("nan"), device=DEV)
    slots = [3, 0, 1]
    for sl in slots:
        state[sl] = 0.0
    call = lambda ctx, r: ops.causal_conv(r, dev(w), state if taps > 1 else None, ctx, DT[out], activation="silu", bias=dev(b)).float()
    got = run_in_steps(ops, [(1, 1, 1), (2, 1, 60), (1, 1, 1), (90, 3, 8), (1, 1, 1), (55, 13, 19)], lens, slots, rows, call)
    for r, x in enumerate(rows):
        close(got[r], P.silu(P.causal_conv(x, w, b)), 3e-6 if out == "float32" else 5e-3, f"request {r}")
    if taps > 1:
        assert torch.isnan(state[2]).all() and torch.isnan(state[4]).all()


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
@pytest.mark.parametrize("parts,width", [(1, 30), (2, 48), (1, 192), (3, 200), (8, 512), (1, 1000), (2, 1500), (5, 7)])
def test_gate_before_the_norm_in_parts(ops, dt, parts, width):
    """Parts of different sizes of numbers, so that a norm over the whole row shows; into a column range of wider rows."""
    rng = np.random.default_rng(width)
    T, n = 9, parts * width
    y = rng.normal(size=(T, parts, width)) * np.exp(2 * rng.normal(size=(1, parts, 1)))
    y = y.reshape(T, n)
    z, w = rng.normal(size=(T, n + 4)) * 2, 1 + 0.3 * rng.normal(size=n)
    for lead in (0, 4, 3):
        out = torch.full((T, n + 8), 3.0, dtype=DT[dt], device=DEV)
        ops.gated_rmsnorm(dev(y), dev(z)[:, lead:lead + n], dev(w), parts, width, 1e-3, DT[dt], gate_first=True, out_scale=0.7,
                          out=out[:, lead:lead + n])
        want = 0.7 * P.gated_part_norm(y, z[:, lead:lead + n], parts, w, 1e-3)
        close(out[:, lead:lead + n].float().cpu().numpy(), want, 5e-6 if dt == "float32" else 6e-3, f"offset {lead}")
        assert (out[:, :lead] == 3.0).all() and (out[:, lead + n:] == 3.0).all()
    # the gate behind the norm, as other mixers have it, through the same kernels
    got = ops.gated_rmsnorm(dev(y), dev(z)[:, :n], dev(w), parts, width, 1e-3, DT[dt])
    want = P.rms_div(y.reshape(T, parts, width), 1e-3).reshape(T, n) * w * P.silu(z[:, :n])
    close(got.float().cpu().numpy(), want, 5e-6 if dt == "float32" else 6e-3, "gate behind")


# ----------------------------------------------------------------------------- a stream that is normed behind every sum
@pytest.mark.parametrize("T,E", [(1, 4), (3, 30), (7, 1024), (200, 1024), (2, 4096), (130, 2052), (5, 8192), (3, 9000), (64, 2048)])
def test_norm_of_the_sum(ops, T, E):
    rng = np.random.default_rng(E)
    x0, y, w = rng.normal(size=(T, E)), 3 * rng.normal(size=(T, E)), 1 + 0.3 * rng.normal(size=E)
    want = P.rms_div(2.3 * x0 + y, 1e-4) * w
    for dt, tol in (("float32", 3e-6), ("bfloat16", 5e-3)):
        x = dev(x0)
        h = ops.post_norm(x, dev(y), 2.3, dev(w), 1e-4, DT[dt])
        close(x.cpu().numpy(), want, 3e-6, "stream")
        close(h.float().cpu().numpy(), want, tol, "its copy")


@pytest.mark.parametrize("M", [1, 8, 16, 17, 40, 64, 65, 200, 512, 1100])
@pytest.mark.parametrize("N,K", [(256, 512), (2048, 1024), (100, 64), (30, 24)])
def test_product_and_norm_of_the_sum(ops, M, N, K):
    """Whatever the product is split into: the old rows count alpha times, once."""
    rng = np.random.default_rng(M + N)
    a, w = dev(rng.normal(size=(M, K)), torch.bfloat16), dev(rng.normal(size=(N, K)) / math.sqrt(K), torch.bfloat16)
    x0, nw, b = rng.normal(size=(M, N)), 1 + 0.2 * rng.normal(size=N), rng.normal(size=N)
    x = dev(x0)
    h = ops.linear_post_norm(a, ops.pack_weight(w), x, -1.7, dev(nw), 1e-5, torch.bfloat16, bias=dev(b))
    want = P.rms_div(-1.7 * x0 + a.double().cpu().numpy() @ w.double().cpu().numpy().T + b, 1e-5) * nw
    close(x.cpu().numpy(), want, 1e-5, "stream")
    close(h.float().cpu().numpy(), want, 6e-3, "its copy")
    x = dev(x0)
    h = ops.linear_post_norm(a.float(), w.float(), x, -1.7, dev(nw), 1e-5, torch.float32)
    close(x.cpu().numpy(), P.rms_div(-1.7 * x0 + a.double().cpu().numpy() @ w.double().cpu().numpy().T, 1e-5) * nw, 1e-5, "32 bits")
    assert torch.equal(h, x) and h.data_ptr() != x.data_ptr()


@pytest.mark.parametrize("M", [1, 16, 17, 64, 65, 300, 1100])
@pytest.mark.parametrize("N,K", [(96, 64), (512, 2048), (33, 40), (20, 30)])
def test_relu_squared_in_the_products_epilogue(ops, M, N, K):
    rng = np.random.default_rng(M + N)
    a, w, b = rng.normal(size=(M, K)), rng.normal(size=(N, K)) / math.sqrt(K), rng.normal(size=N)
    for dt, tol in ((torch.float32, 3e-6), (torch.bfloat16, 8e-3)):
        ad, wd = dev(a, dt), dev(w, dt)
        want = P.relu2(ad.double().cpu().numpy() @ wd.double().cpu().numpy().T + b)
        got = ops.linear(ad, ops.pack_weight(wd), bias=dev(b), activation="relu2")
        assert got.dtype == dt
        close(got.float().cpu().numpy(), want, tol, str(dt))


# ----------------------------------------------------------------------------- routing and experts
@pytest.mark.parametrize("n,top,groups,keep", [(16, 4, 4, 3), (8, 2, 4, 2), (6, 2, 3, 3), (4, 2, 4, 3), (8, 3, 2, 1), (5, 5, 1, 1),
                                               (12, 1, 1, 1), (64, 6, 8, 4), (130, 7, 13, 5), (10, 2, 2, 1)])
def test_choice_by_softmax_scores_within_the_groups_of_the_largest(ops, n, top, groups, keep):
    """A group scores its largest choice score alone; corrections make choice scores negative, where a group left out must
    count as minus infinity and not as zero; the weights are the scores without the correction, not their shares."""
    rng = np.random.default_rng(n + top)
    T = 200
    z = rng.normal(size=(T, n + 2)) * 2
    corr = rng.normal(size=n) * 0.3 - (1.5 if n % 2 == 0 else 0.0)
    how = dict(scores="softmax", groups=groups, keep_groups=keep, weight_scale=1.0)
    idx, wts = (t.cpu().numpy() for t in ops.route_logits(dev(z)[:, 1:1 + n], dev(corr), top, group_score="max", **how))
    checked = 0
    for t in range(T):
        if P.route_margin(z[t, 1:1 + n], corr, top, groups, keep) < 1e-5:
            continue                # (decided within the rounding of 32 bits)
        chosen, w = P.route(z[t, 1:1 + n], corr, top, groups, keep)
        assert list(idx[t]) == list(chosen), f"row {t}"
        close(wts[t], w, 3e-6, f"weights of row {t}")
        checked += 1
    assert checked > T * 0.9
    if groups > 1 and keep < groups and n // groups > 1 and n > 8:
        other, _ = ops.route_logits(dev(z)[:, 1:1 + n], dev(corr), top, **how)
        assert (other.cpu().numpy() != idx).any(), "the inputs do not tell the two group scores apart"


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
@pytest.mark.parametrize("T", [1, 5, 9, 40, 700])
@pytest.mark.parametrize("n,ident,top,E,F", [(6, 2, 2, 64, 24), (2, 2, 4, 48, 32), (1, 1, 1, 30, 10), (14, 2, 2, 256, 128), (3, 5, 3, 40, 16)])
def test_experts_of_which_some_are_the_identity(ops, dt, T, n, ident, top, E, F):
    """Tokens that choose only identity experts, none and some; rows beside the sum without a weight; alone, added to rows,
    and with the norm of the whole in the rows' place, by the kernels for few and for many rows."""
    rng = np.random.default_rng(T + n + E)
    h = dev(rng.normal(size=(T, E)), DT[dt])
    up, down = dev(rng.normal(size=(n, F, E)) / math.sqrt(E), DT[dt]), dev(rng.normal(size=(n, E, F)) / math.sqrt(F), DT[dt])
    idx = np.stack([rng.permutation(n + ident)[:top] for _ in range(T)])
    if T > 2 and ident >= top:
        idx[1] = n + np.arange(top)
    wts = rng.uniform(0.1, 1.0, size=(T, top))
    side, x0 = rng.normal(size=(T, E)), rng.normal(size=(T, E))
    hd, ud, dd = (t.double().cpu().numpy() for t in (h, up, down))
    want = np.zeros((T, E))
    for t in range(T):
        for e, a in zip(idx[t], wts[t]):
            want[t] += a * (hd[t] if e >= n else P.relu2(ud[e] @ hd[t]) @ dd[e].T)
    tol, ntol = (1e-5, 1e-5) if dt == "float32" else (1e-2, 1.2e-2)
    args = (h, up, down, dev(idx, torch.int32), dev(wts))
    close(ops.moe_experts(*args, identity=ident).cpu().numpy(), want, tol, "sum")
    close(ops.moe_experts(*args, identity=ident, beside=(dev(side), None)).cpu().numpy(), want + side, tol, "with rows beside")
    x = dev(x0)
    ops.moe_experts(*args, identity=ident, out=x, accumulate=True)
    close(x.cpu().numpy(), want + x0, tol, "added")
    nw, x = 1 + 0.2 * rng.normal(size=E), dev(x0)
    out = ops.moe_experts(*args, identity=ident, out=x, beside=(dev(side), None), norm=(dev(nw), 1e-5, False), post_alpha=1.9)
    normed = P.rms_div(1.9 * x0 + want + side, 1e-5) * nw
    close(x.cpu().numpy(), normed, tol, "the norm in the rows' place")
    close(out.float().cpu().numpy(), normed, ntol, "and its copy")


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
@pytest.mark.parametrize("T", [1, 2])
@pytest.mark.parametrize("n,ident,top,E,F,Fs", [(6, 2, 2, 64, 24, 40), (3, 1, 4, 256, 512, 136), (2, 1, 1, 48, 10, 21), (2, 0, 2, 30, 9, 6), (4, 0, 1, 72, 16, 8)])
def test_a_shared_expert_in_the_chosen_experts_launches(ops, dt, T, n, ident, top, E, F, Fs):
    """A shared expert wider and narrower than the others, from packed matrices and from plain ones."""
    rng = np.random.default_rng(T + E + Fs)
    h = dev(rng.normal(size=(T, E)), DT[dt])
    mats = [dev(rng.normal(size=s) / math.sqrt(s[-1]), DT[dt]) for s in ((n, F, E), (n, E, F), (Fs, E), (E, Fs))]
    idx = np.stack([rng.permutation(n + ident)[:top] for _ in range(T)])
    wts = rng.uniform(0.1, 1.0, size=(T, top))
    hd, ud, dd, su, sd = (t.double().cpu().numpy() for t in [h] + mats)
    want = P.relu2(hd @ su.T) @ sd.T
    for t in range(T):
        for e, a in zip(idx[t], wts[t]):
            want[t] += a * (hd[t] if e >= n else P.relu2(ud[e] @ hd[t]) @ dd[e].T)
    packed = [ops.pack_weight(m) for m in mats[2:]]
    for shared in (mats[2:], packed) if type(packed[0]) is type(packed[1]) else (mats[2:],):
        got = ops.moe_experts(h, mats[0], mats[1], dev(idx, torch.int32), dev(wts), identity=ident, shared=tuple(shared))
        close(got.cpu().numpy(), want, 1e-5 if dt == "float32" else 1e-2, "sum")


# ----------------------------------------------------------------------------- a model with made weights
def needle_model():
    """Three layers without feed-forwards: latent attention, latent attention over the first layer's rows, and the pair whose
    right side counts nothing.  Token 1 (the needle) has a latent, or a key, along every query, with a score far above the
    fillers' (token 0).  Each layer brings the needle's value to a stream channel of its own (3, 4, 5), which the
    embedding's rows 2, 3 and 4 read as logits."""
    E, V, C, R, D, H = 8, 5, 4, 2, 3, 2
    rng = np.random.default_rng(8)
    lat = {"heads": H, "dim": D, "rot_dim": R, "vdim": 2, "kv_rank": C, "scale": 1.0, "rot": {"base": 100.0, "dims": R}}
    both = {"left": {"heads": H, "kv_heads": 1, "dim": 4, "vdim": 3, "scale": 6.0, "softcap": 60.0, "rot": {"base": 1e7, "dims": 2}},
            "right": {"heads": 1, "vdim": 4, "state": 2, "groups": 1, "conv": 2, "norm_groups": 1}, "left_scale": 1.0, "right_scale": 0.0}
    cfg = {"architecture": "Pevolorn", "vocab": V, "width": E, "norm": {"eps": 1e-6}, "postln_alpha": 1.0,
           "layers": [{"type": "latent_attention", "mixer": lat, "mlp": None},
                      {"type": "latent_attention", "mixer": dict(lat, kv_from=0), "mlp": None},
                      {"type": "parallel", "mixer": both, "mlp": None}]}
    small = lambda *s: rng.normal(size=s) * 0.01
    emb = np.zeros((V, E)); emb[0, 1] = emb[1, 0] = emb[2, 3] = emb[3, 4] = emb[4, 5] = 1.0
    w = {"embed": emb, "final.norm": np.zeros(E)}
    dkv = small(C + R, E)
    dkv[0, 0] = dkv[1, 1] = 1.0                     # the needle's latent lies along channel 0, a filler's along channel 1
    w.update({"l0.mix.dkv": dkv, "l0.mix.dkv.norm": np.ones(C)})
    for i in range(2):
        q, uk, uv, o = small(H * (D + R), E), small(H * D, C), small(H * 2, C), small(E, H * 2)
        for h in range(H):
            q[h * (D + R), :2] += 4.0               # every token's query has channel 0
            uk[h * D, 0] = 4.0
            uv[h * 2, 0] = 1.0
        o[3 + i, 0] = o[3 + i, 2] = 2.0
        p = f"l{i}.mix."
        w.update({p + "q": q, p + "uk": uk, p + "uv": uv, p + "o": o, p + "g": small(H, E), f"l{i}.norm1": np.zeros(E)})
    p = "l2.mix.left."
    k, v, bq = small(4, E), small(3, E), np.zeros(H * 4)
    k[3, 0], k[2, 1], v[0, 0] = 1.0, 1.0, 1.0       # (channels behind the rotated ones)
    bq[3] = bq[7] = 1.0
    o = small(E, H * 3)
    o[5, 0] = o[5, 3] = 2.0
    w.update({p + "q": small(H * 4, E), p + "q.b": bq, p + "k": k, p + "k.b": np.zeros(4), p + "v": v, p + "v.b": np.zeros(3),
              p + "g": small(H, E), p + "o": o, p + "o.b": np.zeros(E)})
    p = "l2.mix.right."
    w.update({p + "in": rng.normal(size=(13, E)), p + "conv": rng.normal(size=(8, 2)), p + "conv.b": np.zeros(8), p + "dt_bias": np.zeros(1),
              p + "A_log": np.zeros(1), p + "D": np.ones(1), p + "norm": np.ones(4), p + "o": rng.normal(size=(E, 4)), "l2.norm1": np.zeros(E)})
    return cfg, w


@pytest.mark.parametrize("page", [16, 64])
@pytest.mark.parametrize("decode_from", [None, 40])
@pytest.mark.parametrize("jstar", [0, 15, 16, 63, 64])
def test_a_token_that_stands_out_far_back(tmp_path, page, decode_from, jstar):
    """The needle at a page's first and last place, seen by every later token through 700 fillers, in every layer: in its own
    rows, in another layer's rows, under a soft cap; in a prompt's portions and decoded token by token."""
    from xyntetik_runner_amd.config import config_from_dict
    from xyntetik_runner_amd.engine.runner import ModelRunner
    from xyntetik_runner_amd.trace import replay
    cfg, w = needle_model()
    n = 700 if decode_from is None else 260
    toks = [0] * n
    toks[jstar] = 1
    want, without = P.forward(cfg, w, toks), P.forward(cfg, w, [0] * n)
    assert (want[jstar + 1:, 2:] - without[jstar + 1:, 2:]).min() > 0.4, "the made weights do not show the needle in every layer"
    if decode_from is None:
        steps = traces.portions({"a": toks}, sizes=(17, 2, 40, 3, 400, 64))
    else:
        steps = traces.tail_one_by_one({"a": toks}, tail=n - decode_from)
    arch, typed = config_from_dict(cfg)
    tensors = {k: torch.tensor(v, dtype=torch.float32) for k, v in w.items()}
    runner = ModelRunner(arch.build_spec(typed), tensors, "float32", max_tokens=n + 64, page_size=page, max_requests=2)
    for lc in runner.storage.layers:
        if lc.owns:
            lc.k.fill_(float("nan")); lc.v.fill_(float("nan"))
    out = str(tmp_path / "out")
    replay(runner, traces.to_lines(steps), out, report=io.StringIO())
    close(traces.collect(steps, out, cfg["vocab"])["a"], want, 1e-5, f"needle at {jstar}")


def test_first_tokens_of_a_sequence(tmp_path):
    """Sequences of one, two and three tokens beside a longer one in a mixed batch: position 0 reads itself alone, states and
    carried inputs start at zero."""
    from pevolorn_tiny import make_model
    from plain_llama import load_folder
    from xyntetik_runner_amd.engine.runner import ModelRunner
    from xyntetik_runner_amd.trace import replay
    for which in ("P1", "P2", "P4"):
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
