"""A plain, slow Pevolorn decoder in numpy float64: whole sequences, no cache, no state.

One function per mechanism, each written from its equation; nothing here knows of pages, slots, batches or
kernels, and nothing is shared with the engine.  The tests compare what the engine does, however its work is
cut, with these functions run over the whole sequence.

Notation: ``T`` tokens, ``E`` width; a mixer has ``H`` heads (``G`` key heads or state groups where they are fewer)
with keys of ``D`` and values of ``Dv`` channels.  Weights are ``[out, in]`` and applied as ``W x``.  ``cfg`` is
config.json as a dict, ``w`` a dict name -> float64 array.
"""
from __future__ import annotations

import numpy as np


# ----------------------------------------------------------------------------- small pieces
def rms_div(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps)


def centred_weight_norm(x, w, eps):
    """An RMS norm whose weight is stored as its difference from one."""
    return rms_div(x, eps) * (1.0 + w)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def relu2(z):
    return np.maximum(z, 0.0) ** 2


def softcap(z, cap):
    """``cap tanh(z / cap)``; no cap: ``z``."""
    return cap * np.tanh(z / cap) if cap else z


def rotate_half(x, base, dims, first=0):
    """``x [T, heads, D]`` at positions first..first+T-1: channel i < dims/2 turns with channel i + dims/2 by the angle
    ``p * base^(-2i/dims)``; channels from ``dims`` on pass."""
    half = dims // 2
    f = float(base) ** (-2.0 * np.arange(half) / dims) if dims else np.zeros(0)
    a = (first + np.arange(x.shape[0]))[:, None] * f[None, :]
    c, s = np.cos(a)[:, None, :], np.sin(a)[:, None, :]
    out = np.array(x, dtype=np.float64)
    u, v = x[..., :half], x[..., half:dims]
    out[..., :half] = u * c - v * s
    out[..., half:dims] = v * c + u * s
    return out


# ----------------------------------------------------------------------------- attention
def attend(q, k, v, scale, cap=None):
    """Causal attention ``[T, H, Dv]`` of ``q [T, H, D]`` over ``k [n, G, D]``, ``v [n, G, Dv]`` whose last T positions are
    the queries' own; head h reads key head ``h // (H / G)``; scores ``(q . k) scale`` through the soft cap."""
    T, H, _ = q.shape
    n, G, Dv = v.shape
    out = np.zeros((T, H, Dv))
    pos = np.arange(n - T, n)
    for h in range(H):
        g = h // (H // G)
        s = softcap((q[:, h] @ k[:, g].T) * scale, cap)
        s = np.where(np.arange(n)[None, :] <= pos[:, None], s, -np.inf)
        e = np.exp(s - s.max(axis=-1, keepdims=True))
        out[:, h] = (e / e.sum(axis=-1, keepdims=True)) @ v[:, g]
    return out


def latent_rows(h, w, p, m, eps):
    """What a latent attention keeps of every token: (the normed latent ``[T, kv_rank]``, the rotated key part that the
    heads share ``[T, rot_dim]``)."""
    C = m["kv_rank"]
    y = h @ w[p + "dkv"].T
    return rms_div(y[:, :C], eps) * w[p + "dkv.norm"], rotate_half(y[:, None, C:], m["rot"]["base"], m["rot"]["dims"])[:, 0]


def latent_attention(h, w, p, m, kept):
    """Keys and values made head by head from the latents ``kept`` (this layer's own or an earlier layer's)."""
    H, D, R, Dv, T = m["heads"], m["dim"], m["rot_dim"], m["vdim"], h.shape[0]
    c, shared = kept
    q = (h @ w[p + "q"].T).reshape(T, H, D + R)
    q = np.concatenate([q[..., :D], rotate_half(q[..., D:], m["rot"]["base"], m["rot"]["dims"])], axis=-1)
    k = np.concatenate([(c @ w[p + "uk"].T).reshape(T, H, D), np.broadcast_to(shared[:, None, :], (T, H, R))], axis=-1)
    v = (c @ w[p + "uv"].T).reshape(T, H, Dv)
    o = attend(q, k, v, m["scale"]) * sigmoid(h @ w[p + "g"].T)[:, :, None]
    return o.reshape(T, H * Dv) @ w[p + "o"].T


def capped_attention(h, w, p, m, eps):
    """The left side: biased projections; queries and keys rotated, then over their root mean square head by head;
    a soft cap of the scores; a gate a head."""
    H, G, D, Dv, T = m["heads"], m["kv_heads"], m["dim"], m["vdim"], h.shape[0]
    q = (h @ w[p + "q"].T + w[p + "q.b"]).reshape(T, H, D)
    k = (h @ w[p + "k"].T + w[p + "k.b"]).reshape(T, G, D)
    v = (h @ w[p + "v"].T + w[p + "v.b"]).reshape(T, G, Dv)
    rot = m.get("rot")
    if rot and rot["dims"]:
        q, k = rotate_half(q, rot["base"], rot["dims"]), rotate_half(k, rot["base"], rot["dims"])
    o = attend(rms_div(q, eps), rms_div(k, eps), v, m["scale"], m.get("softcap"))
    o = o * sigmoid(h @ w[p + "g"].T)[:, :, None]
    return o.reshape(T, H * Dv) @ w[p + "o"].T + w[p + "o.b"]


# ----------------------------------------------------------------------------- state space
def causal_conv(x, taps_w, bias):
    """``x [T, C]`` through a convolution over time a channel, ``taps_w [C, taps]`` with the last column the token's own,
    zeros before the start, plus a bias a channel."""
    T, C = x.shape
    taps = taps_w.shape[1]
    y = np.zeros((T, C)) + bias
    for j in range(taps):
        back = taps - 1 - j
        if back < T:
            y[back:] += x[:T - back] * taps_w[:, j]
    return y


def state_space(x, B, C, dt, a):
    """One head: ``S_t = exp(-a dt_t) S_(t-1) + dt_t B_t x_t^T``, ``y_t = S_t^T C_t``; S starts at zero.
    ``x [T, Dv]``, ``B``, ``C`` ``[T, N]``, ``dt [T]``, a number ``a``."""
    S = np.zeros((B.shape[1], x.shape[1]))
    y = np.zeros_like(x)
    for t in range(x.shape[0]):
        S = np.exp(-a * dt[t]) * S + dt[t] * np.outer(B[t], x[t])
        y[t] = S.T @ C[t]
    return y


def gated_part_norm(y, z, parts, w, eps):
    """``y silu(z)``, then every one of ``parts`` equal parts of the row over its own root mean square, times a weight a
    channel."""
    u = y * silu(z)
    T, n = u.shape
    return rms_div(u.reshape(T, parts, n // parts), eps).reshape(T, n) * w


def mamba2(h, w, p, m, eps):
    """The right side."""
    H, Dv, N, G, T = m["heads"], m["vdim"], m["state"], m["groups"], h.shape[0]
    inner = H * Dv
    proj = h @ w[p + "in"].T
    z, xbc, dt = proj[:, :inner], proj[:, inner:2 * inner + 2 * G * N], proj[:, 2 * inner + 2 * G * N:]
    xbc = silu(causal_conv(xbc, w[p + "conv"], w[p + "conv.b"]))
    x = xbc[:, :inner].reshape(T, H, Dv)
    B = xbc[:, inner:inner + G * N].reshape(T, G, N)
    C = xbc[:, inner + G * N:].reshape(T, G, N)
    dt = softplus(dt + w[p + "dt_bias"])
    a = np.exp(w[p + "A_log"])
    y = np.stack([state_space(x[:, i], B[:, i // (H // G)], C[:, i // (H // G)], dt[:, i], a[i]) + w[p + "D"][i] * x[:, i]
                  for i in range(H)], axis=1)
    return gated_part_norm(y.reshape(T, inner), z, m["norm_groups"], w[p + "norm"], eps) @ w[p + "o"].T


def parallel(h, w, p, m, eps):
    return (m["left_scale"] * capped_attention(h, w, p + "left.", m["left"], eps)
            + m["right_scale"] * mamba2(h, w, p + "right.", m["right"], eps))


# ----------------------------------------------------------------------------- feed-forward
def choice_scores(z, correction):
    e = np.exp(z - z.max())
    s = e / e.sum()
    return s, s + correction


def group_scores(c, groups):
    return c.reshape(groups, -1).max(axis=1)


def route(z, correction, top, groups, keep):
    """From router logits ``z [n]`` (experts, then identity experts): (chosen, their weights).  Scores are a softmax over
    all; the choice is by score + correction among the ``keep`` groups (of ``groups`` equal groups of neighbours) whose
    largest choice score is largest; the weights are the scores themselves."""
    s, c = choice_scores(z, correction)
    kept = np.argsort(-group_scores(c, groups), kind="stable")[:keep]
    masked = np.where(np.isin(np.arange(len(z)) // (len(z) // groups), kept), c, -np.inf)
    chosen = np.argsort(-masked, kind="stable")[:top]
    return chosen, s[chosen]


def route_margin(z, correction, top, groups, keep):
    """By how much the choice of ``route`` is decided: the smaller of the lead of the last kept group over the next and
    of the last chosen expert over the next in the kept groups (infinite where there is no next)."""
    _, c = choice_scores(z, correction)
    gs = group_scores(c, groups)
    order = np.argsort(-gs, kind="stable")
    gap = gs[order[keep - 1]] - gs[order[keep]] if keep < groups else np.inf
    allowed = np.sort(c.reshape(groups, -1)[order[:keep]].ravel())[::-1]
    return min(gap, allowed[top - 1] - allowed[top]) if top < len(allowed) else gap


def expert(h, w, p):
    return relu2(h @ w[p + "up"].T) @ w[p + "down"].T


def experts(h, w, mlp, p, choices=None):
    r = mlp["router"]
    groups = r.get("groups") or {"count": 1, "keep": 1}
    z = h @ w[p + "router"].T
    how = (w[p + "correction"], r["top"], groups["count"], groups["keep"])
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        chosen, wts = route(z[t], *how)
        if choices is not None:
            choices.append((z[t], chosen, route_margin(z[t], *how)))
        for e, a in zip(chosen, wts):
            out[t] += a * (expert(h[t], w, f"{p}e{int(e)}.") if e < r["experts"] else h[t])
    if mlp.get("shared"):
        out += expert(h, w, p + "shared.")
    return out


# ----------------------------------------------------------------------------- the model
def forward(cfg, w, tokens, taps=None, choices=None):
    """Logits ``[T, vocab]`` of the whole sequence.  ``taps``: a list that receives the residual stream after every
    layer; ``choices``: one that receives (router logits, chosen experts, ``route_margin``) of every routed token."""
    eps, alpha = cfg["norm"]["eps"], cfg["postln_alpha"]
    x = w["embed"][np.asarray(tokens, dtype=np.int64)].astype(np.float64)
    kept = {}
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}."
        if layer["type"] == "latent_attention":
            j = m.get("kv_from")
            if j is None:
                kept[i] = latent_rows(x, w, p + "mix.", m, eps)
            y = latent_attention(x, w, p + "mix.", m, kept[i if j is None else j])
        elif layer["type"] == "parallel":
            y = parallel(x, w, p + "mix.", m, eps)
        else:
            raise ValueError(layer["type"])
        x = centred_weight_norm(alpha * x + y, w[p + "norm1"], eps)
        if layer.get("mlp") is not None:
            x = centred_weight_norm(alpha * x + experts(x, w, layer["mlp"], p + "mlp.", choices), w[p + "norm2"], eps)
        if taps is not None:
            taps.append(x.copy())
    return centred_weight_norm(x, w["final.norm"], eps) @ w["embed"].T
