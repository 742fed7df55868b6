"""Small Girolorn configurations for the tests, each with sizes and constants of its own.

Between them they differ in everything config.json gives: width, vocabulary, the number and order of the layers,
which layers run with which others' tensors (neighbours, far ones, chains, one layer alone many times, none),
heads and head sizes (multiples of 16 and of nothing), key/value heads (as many as query heads, fewer, one), scales
and soft caps (absent, wide, one that most scores feel), the rotated part of a head (none, absent, a part, all of it,
multiples of 4 and not), bases, YaRN's numbers (absent, ramps that begin and end inside the rotated pairs, before the
first and behind the last, a factor below one, slow and fast alike), the experts (one, some and all chosen, one
expert in all) and their limits, the shared expert (absent, wider and narrower than the others, another limit), no
feed-forward, the logits' soft cap (absent, wide and narrow) and eps.
"""


def attn(heads, kv_heads, dim, scale, softcap=None, rot=None, scaling=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale}
    if softcap is not None:
        m["softcap"] = softcap
    if rot is not None:
        m["rot"] = {"base": rot[0], "dims": rot[1]}
        if scaling is not None:
            m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return m


def moe(ff, limit, experts, top, shared=None):
    m = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}
    if shared is not None:
        m["shared"] = {"ff": shared[0], "limit": shared[1]}
    return m


def layer(mixer, mlp, weights_of=None):
    out = {"type": "attention", "mixer": mixer, "mlp": mlp}
    if weights_of is not None:
        out["weights_of"] = weights_of
    return out


# two kinds of layer, each run again by a neighbour and the first once more at the end; a ramp inside the rotated pairs;
# a layer without a feed-forward; head sizes the matrix cores take in bfloat16
_A1 = attn(4, 2, 32, 0.3, softcap=6.0, rot=(10000.0, 16), scaling=(8.0, 64, 16.0, 1.0))
_B1 = attn(2, 1, 64, 0.2, softcap=20.0, rot=(500.0, 64))
_M1 = moe(24, 0.8, 8, 2, shared=(40, 0.6))
TINY_G1 = {"architecture": "Girolorn", "vocab": 200, "width": 64, "norm": {"eps": 1e-5}, "logit_softcap": 12.0,
           "layers": [layer(_A1, _M1), layer(_A1, _M1, 0), layer(_B1, None), layer(_B1, None, 2), layer(_A1, _M1, 0)]}

# sizes that are multiples of nothing; one key head; three pairs of a head rotated; no soft cap anywhere; every expert
# chosen; the ramp shorter than a pair (fast and slow alike); no sharing
TINY_G2 = {"architecture": "Girolorn", "vocab": 97, "width": 40, "norm": {"eps": 1e-6},
           "layers": [layer(attn(3, 1, 10, 0.45, rot=(500.0, 6), scaling=(4.0, 100.0, 8.0, 8.0)), moe(12, 1.2, 3, 3, shared=(13, 0.5))),
                      layer(attn(2, 2, 14, 0.4, rot=(50.0, 14)), moe(10, 0.3, 4, 4))]}

# as many key heads as query heads, the whole head rotated; a chain (layer 2 names 1, which names 0); one expert a token,
# none shared
_A3 = attn(4, 4, 64, 0.15, softcap=50.0, rot=(500000.0, 64), scaling=(2.0, 512, 32.0, 2.0))
_M3 = moe(32, 2.0, 6, 1)
TINY_G3 = {"architecture": "Girolorn", "vocab": 256, "width": 96, "norm": {"eps": 1e-5}, "logit_softcap": 30.0,
           "layers": [layer(_A3, _M3), layer(_A3, _M3, 0), layer(_A3, _M3, 1), layer(attn(8, 4, 16, 0.3, softcap=9.0), moe(48, 1.0, 5, 3, shared=(32, 1.5)))]}

# a width no kernel likes (no 16-byte rows, no matrix cores), odd head counts; no rotation; a soft cap that most scores
# feel; a logit cap that most logits feel; limits that most branches meet
TINY_G4 = {"architecture": "Girolorn", "vocab": 61, "width": 30, "norm": {"eps": 1e-5}, "logit_softcap": 1.5,
           "layers": [layer(attn(3, 3, 10, 0.9, softcap=2.5), moe(9, 0.2, 4, 4, shared=(6, 0.15))),
                      layer(attn(3, 1, 8, 0.5, rot=(10.0, 0)), moe(10, 0.1, 2, 1))]}

# YaRN with a factor below one and a ramp that begins before the first pair and ends behind the last; one expert in all;
# a shared expert of the experts' own size
TINY_G5 = {"architecture": "Girolorn", "vocab": 128, "width": 64, "norm": {"eps": 1e-6}, "logit_softcap": 50.0,
           "layers": [layer(attn(8, 2, 16, 0.35, softcap=15.0, rot=(100.0, 16), scaling=(0.5, 4096, 1000.0, 0.01)), moe(64, 1.0, 1, 1, shared=(64, 2.0))),
                      layer(attn(4, 2, 48, 0.14, softcap=30.0, rot=(20000.0, 24), scaling=(16.0, 32, 4.0, 0.5)), moe(16, 0.7, 8, 3, shared=(24, 0.4)))]}

# a single layer run four times, each run with pages of its own
_A6 = attn(16, 4, 16, 0.3, softcap=10.0, rot=(1000.0, 8), scaling=(3.0, 40, 6.0, 1.5))
_M6 = moe(32, 0.9, 3, 3, shared=(16, 0.7))
TINY_G6 = {"architecture": "Girolorn", "vocab": 64, "width": 48, "norm": {"eps": 1e-5}, "logit_softcap": 8.0,
           "layers": [layer(_A6, _M6)] + [layer(_A6, _M6, 0) for _ in range(3)]}

# sizes nearer a real model's: heads of 128 and 96, every expert chosen (no choice that a rounding could change: every row
# is compared in bfloat16), the first two layers run again in turn
_A7 = attn(4, 1, 128, 0.1, softcap=25.0, rot=(250000.0, 128), scaling=(4.0, 256, 32.0, 1.0))
_B7 = attn(2, 2, 96, 0.12, softcap=40.0, rot=(10000.0, 32))
_M7 = moe(64, 1.0, 2, 2, shared=(192, 0.8))
TINY_G7 = {"architecture": "Girolorn", "vocab": 512, "width": 320, "norm": {"eps": 1e-5}, "logit_softcap": 40.0,
           "layers": [layer(_A7, _M7), layer(_B7, _M7), layer(_A7, _M7, 0), layer(_B7, _M7, 1)]}

# (configuration, seed, deviation of the matrices)
CONFIGS = {"G1": (TINY_G1, 51, 0.2), "G2": (TINY_G2, 52, 0.2), "G3": (TINY_G3, 53, 0.12), "G4": (TINY_G4, 54, 0.2),
           "G5": (TINY_G5, 55, 0.15), "G6": (TINY_G6, 56, 0.2), "G7": (TINY_G7, 57, 0.06)}


def make_model(which: str, folder: str, std: float = 0.0) -> str:
    from xyntetik_runner_amd.weights import write_random_model
    config, seed, own = CONFIGS[which]
    std = std or own
    return write_random_model(config, folder, seed=seed, std=std, norm_jitter=0.1, dtype="bfloat16")
