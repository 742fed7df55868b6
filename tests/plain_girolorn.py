"""A plain, slow Girolorn decoder in numpy float64: whole sequences, no cache, no state.

One function per mechanism, each written from its equation; nothing here knows of pages, slots, batches or
kernels, and nothing is shared with the engine.  The tests compare what the engine does, however its work is
cut, with these functions run over the whole sequence.

Notation: ``T`` tokens, ``E`` width; a mixer has ``H`` query heads of ``D`` channels and ``G`` key heads whose keys,
as projected, are the values too.  Weights are ``[out, in]`` and applied as ``W x``.  ``cfg`` is config.json as a
dict, ``w`` a dict name -> float64 array.
"""
from __future__ import annotations

import math

import numpy as np


# ----------------------------------------------------------------------------- small pieces
def layer_norm(x, w, eps):
    """(x - mean) / sqrt(mean((x - mean)^2) + eps) * w over the last axis; no bias."""
    d = x - x.mean(axis=-1, keepdims=True)
    return d / np.sqrt((d * d).mean(axis=-1, keepdims=True) + eps) * w


def rms_norm(x, w, eps):
    """x / sqrt(mean(x^2) + eps) * w over the last axis."""
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps) * w


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def softcap(z, cap):
    """``cap tanh(z / cap)``; no cap: ``z``."""
    return cap * np.tanh(z / cap) if cap else z


# ----------------------------------------------------------------------------- rotation
def yarn(dims, base, scaling):
    """(frequencies [dims/2], factor on cosines and sines).  Pair i turns by ``base^(-2i/dims)`` a position; with
    ``scaling`` the pairs that turn ``fast`` times or more in ``original`` positions keep that, those that turn
    ``slow`` times or fewer are slowed by ``factor``, and between the two (by pair number, from the integer below the
    first to the integer above the second) the two frequencies are mixed in a straight line."""
    i = np.arange(dims // 2, dtype=np.float64)
    f = base ** (-2.0 * i / dims)
    if not scaling:
        return f, 1.0
    factor, original = float(scaling["factor"]), float(scaling["original"])

    def pair_of(turns):             # the pair (as a real number) that turns so often in ``original`` positions
        return dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(pair_of(scaling["fast"])), 0)
    hi = min(math.ceil(pair_of(scaling["slow"])), dims - 1)
    slowed = np.clip((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / factor * slowed + f * (1.0 - slowed), 0.1 * math.log(factor) + 1.0


def rotate_neighbours(x, freq, mult, first=0):
    """``x [T, heads, D]`` at positions first..first+T-1: channels 2i and 2i+1, i < len(freq), turn together by the
    angle ``p * freq[i]`` and are multiplied by ``mult``; the channels behind them pass."""
    out = np.array(x, dtype=np.float64)
    n = len(freq)
    for t in range(x.shape[0]):
        a = (first + t) * freq
        c, s = np.cos(a) * mult, np.sin(a) * mult
        u, v = x[t, :, 0:2 * n:2], x[t, :, 1:2 * n:2]
        out[t, :, 0:2 * n:2] = u * c - v * s
        out[t, :, 1:2 * n:2] = v * c + u * s
    return out


# ----------------------------------------------------------------------------- attention
def attend(q, k, v, scale, cap, sink):
    """Causal attention ``[T, H, Dv]`` of ``q [T, H, D]`` over ``k [n, G, D]``, ``v [n, G, Dv]`` whose last T positions are
    the queries' own: scores ``(q . k) scale`` through the soft cap, and a denominator that also holds ``exp(sink_h)``."""
    T, H, _ = q.shape
    n, G, Dv = v.shape
    out = np.zeros((T, H, Dv))
    pos = np.arange(n - T, n)
    for h in range(H):
        g = h // (H // G)
        s = softcap((q[:, h] @ k[:, g].T) * scale, cap)
        s = np.where(np.arange(n)[None, :] <= pos[:, None], s, -np.inf)
        m = s.max(axis=-1, keepdims=True)
        if sink is not None:
            m = np.maximum(m, sink[h])
        e = np.exp(s - m)
        den = e.sum(axis=-1, keepdims=True)
        if sink is not None:
            den = den + np.exp(sink[h] - m)
        out[:, h] = (e / den) @ v[:, g]
    return out


def attention(h, w, m, eps, p):
    """Queries and keys normed over all their heads at once, then rotated; the values are the keys before both."""
    H, G, D = m["heads"], m["kv_heads"], m["dim"]
    T = h.shape[0]
    q, k = h @ w[p + "q"].T, h @ w[p + "k"].T
    v = k.reshape(T, G, m.get("vdim", D))
    q = rms_norm(q, w[p + "q.norm"], eps).reshape(T, H, D)
    k = rms_norm(k, w[p + "k.norm"], eps).reshape(T, G, D)
    rot = m.get("rot")
    if rot and rot.get("dims"):
        freq, mult = yarn(rot["dims"], rot["base"], rot.get("scaling"))
        q, k = rotate_neighbours(q, freq, mult), rotate_neighbours(k, freq, mult)
    o = attend(q, k, v, m["scale"], m.get("softcap"), w[p + "sink"])
    return o.reshape(T, -1) @ w[p + "o"].T


# ----------------------------------------------------------------------------- feed-forward
def clamped_expert(h, w, p, limit):
    """``down(g sigmoid(1.702 g) (u + 1))`` with ``g = min(gate h, limit)``, ``u = clamp(up h, -limit, limit)``."""
    g = np.minimum(h @ w[p + "gate"].T, limit)
    u = np.clip(h @ w[p + "up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w[p + "down"].T


def choose(z, top):
    """(chosen experts, weights) of one token from its logits: the largest (ties: the lower number), and the softmax
    over the chosen logits alone."""
    chosen = np.argsort(-z, kind="stable")[:top]
    e = np.exp(z[chosen] - z[chosen].max())
    return chosen, e / e.sum()


def choice_margin(z, top):
    """By how much the last chosen logit leads the next one (infinite where there is none)."""
    s = np.sort(z)[::-1]
    return s[top - 1] - s[top] if top < len(s) else np.inf


def experts(h, w, mlp, p, choices=None):
    z = h @ w[p + "router"].T + w[p + "router.b"]
    top = mlp["router"]["top"]
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        chosen, wts = choose(z[t], top)
        if choices is not None:
            choices.append((z[t], chosen, choice_margin(z[t], top)))
        for e, a in zip(chosen, wts):
            out[t] += a * clamped_expert(h[t], w, f"{p}e{int(e)}.", mlp["expert"]["limit"])
    shared = mlp.get("shared")
    if shared:
        y = clamped_expert(h, w, p + "shared.", shared["limit"])
        out += sigmoid(h @ w[p + "shared.sg"].T) * y
    return out


# ----------------------------------------------------------------------------- the model
def tensors_of(cfg, i):
    """The layer whose tensors layer i runs with: its own, or those of the layer it names."""
    while cfg["layers"][i].get("weights_of") is not None:
        i = cfg["layers"][i]["weights_of"]
    return i


def forward(cfg, w, tokens, taps=None, choices=None):
    """Logits ``[T, vocab]`` of the whole sequence.  ``taps``: a list that receives the residual stream after every
    layer; ``choices``: one that receives (router logits, chosen experts, ``choice_margin``) of every routed token."""
    eps = cfg["norm"]["eps"]
    x = w["embed"][np.asarray(tokens, dtype=np.int64)].astype(np.float64)
    for i in range(len(cfg["layers"])):
        j = tensors_of(cfg, i)
        layer, p = cfg["layers"][j], f"l{j}."
        x = x + attention(layer_norm(x, w[p + "norm1"], eps), w, layer["mixer"], eps, p + "mix.")
        if layer.get("mlp") is not None:
            x = x + experts(layer_norm(x, w[p + "norm2"], eps), w, layer["mlp"], p + "mlp.", choices)
        if taps is not None:
            taps.append(x.copy())
    return softcap(layer_norm(x, w["final.norm"], eps) @ w["head"].T, cfg.get("logit_softcap"))
