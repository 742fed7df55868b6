"""Small Pevolorn configurations for the tests, each with sizes and constants of its own.

Between them they differ in everything config.json gives: width, vocabulary, the number, kind and order of the layers, the
stream's factor (below, at and above one), which layers read which others' rows (the one before, one far back, several the
same one, none), heads, key and value sizes (multiples of 16, of 8 and of nothing, values longer and shorter than keys),
cached rows (whose latent is a multiple of 16, is not, and rows longer than the matrix cores take), key/value heads (as many
as query heads, fewer, one), scales, soft caps (absent, wide, one that most scores feel), the rotated part of a head (none,
absent, a part, all of it), bases, the state space's heads, groups (one, some, as many as heads), states, taps (one to
five), parts of its norm (one, several), the sides' factors (one of them zero or negative), the experts (one, some and all
chosen), identity experts (none, one, as many as others), groups (one, some, one expert each), the shared expert (absent,
narrower and wider than the others), no feed-forward, and eps.
"""


def latent(heads, dim, rot_dim, vdim, kv_rank, scale, base=10000.0, kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale,
         "rot": {"base": base, "dims": rot_dim}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return m


def pair(left, right, left_scale, right_scale):
    heads, kv_heads, dim, vdim, scale, cap, rot = left
    lf = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if cap is not None:
        lf["softcap"] = cap
    if rot is not None:
        lf["rot"] = {"base": rot[0], "dims": rot[1]}
    names = ("heads", "vdim", "state", "groups", "conv", "norm_groups")
    return {"left": lf, "right": dict(zip(names, right)), "left_scale": left_scale, "right_scale": right_scale}


def moe(ff, experts, top, identity=0, groups=None, shared=None):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if identity:
        m["router"]["identity"] = identity
    if groups is not None:
        m["router"]["groups"] = {"count": groups[0], "keep": groups[1]}
    if shared is not None:
        m["shared"] = {"ff": shared}
    return m


def layer(mixer, mlp):
    return {"type": "parallel" if "left" in mixer else "latent_attention", "mixer": mixer, "mlp": mlp}


def model(vocab, width, alpha, layers, eps=1e-5):
    return {"architecture": "Pevolorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "postln_alpha": alpha, "layers": layers}


# sizes the matrix cores take in bfloat16; a reader two layers behind its owner, a second owner of other sizes; a layer
# without a feed-forward; experts in groups with identity experts
_M1 = moe(24, 6, 2, identity=2, groups=(4, 2), shared=40)
_A1 = moe(32, 2, 4, identity=2, groups=(2, 2), shared=24)       # (every expert chosen: bfloat16 rows up to the last layer compare)
TINY_P1 = model(200, 64, 1.7, [
    layer(latent(4, 16, 16, 24, 32, 0.3), _A1),
    layer(pair((4, 2, 32, 16, 0.25, 9.0, (10000.0, 16)), (4, 16, 24, 2, 3, 2), 0.8, 0.5), _A1),
    layer(latent(2, 24, 16, 16, 32, 0.2, kv_from=0), None),
    layer(latent(8, 8, 16, 8, 16, 0.25, base=300.0), _A1),
    layer(pair((2, 1, 16, 32, 0.4, None, None), (8, 8, 16, 8, 2, 4), 1.2, -0.7), _M1)])

# sizes that are multiples of nothing; one tap (no state of the convolution); a state smaller than a lane group; every
# expert chosen, the identity among them; eps of another size
TINY_P2 = model(97, 40, 1.0, [
    layer(pair((3, 1, 10, 14, 0.3, 2.0, (500.0, 6)), (3, 10, 5, 1, 1, 5), 0.6, 0.9), moe(12, 3, 4, identity=1)),
    layer(latent(3, 10, 6, 7, 14, 0.35, base=50.0), moe(10, 2, 3, identity=1, groups=(3, 3), shared=9)),
    layer(latent(2, 5, 6, 9, 14, 0.3, base=50.0, kv_from=1), moe(13, 3, 3, shared=17))], eps=1e-4)

# as many key heads as query heads, the whole head rotated, values half as long; prompts that end beside a page's edge; one
# expert a token, none shared, no identity
TINY_P3 = model(256, 96, 2.2, [
    layer(latent(4, 32, 16, 32, 64, 0.15), moe(32, 6, 1, groups=(3, 1))),
    layer(latent(6, 16, 16, 16, 64, 0.2, kv_from=0), moe(24, 6, 1)),
    layer(pair((4, 4, 64, 32, 0.12, 30.0, (30000.0, 64)), (8, 32, 64, 4, 4, 4), 0.5, 0.5), moe(48, 5, 3, identity=3, shared=32)),
    layer(latent(4, 16, 16, 48, 64, 0.2, kv_from=0), moe(32, 4, 2, shared=64))])

# a width no kernel likes, odd head counts; a factor below one; a soft cap that most scores feel; five taps
TINY_P4 = model(61, 30, 0.6, [
    layer(pair((3, 3, 10, 6, 0.9, 1.5, (10.0, 0)), (3, 7, 9, 3, 5, 3), 1.0, 1.0), moe(9, 2, 3, identity=1, shared=6)),
    layer(latent(3, 8, 2, 5, 11, 0.5, base=10.0), None),
    layer(latent(5, 3, 2, 4, 11, 0.5, base=10.0, kv_from=1), moe(7, 2, 2))])

# a latent that is no multiple of 16 in a row that is (the values hold whole rows); two readers of it; a left side without
# a rotation; 8 choices in 4 groups in the last layer
_M5 = moe(64, 5, 3, identity=3, groups=(4, 2), shared=16)
_A5 = moe(40, 3, 4, identity=1, groups=(2, 2), shared=16)       # (every expert chosen: bfloat16 rows up to the last layer compare)
TINY_P5 = model(128, 64, 1.3, [
    layer(latent(8, 8, 12, 16, 20, 0.3), _A5), layer(latent(4, 16, 12, 8, 20, 0.3, kv_from=0), _A5),
    layer(pair((8, 2, 16, 16, 0.3, 15.0, None), (2, 32, 16, 1, 4, 1), 0.0, 1.5), moe(16, 4, 4)),
    layer(latent(4, 8, 12, 24, 20, 0.25, kv_from=0), None),
    layer(pair((4, 2, 48, 48, 0.14, 20.0, (20000.0, 24)), (4, 24, 8, 2, 4, 1), 1.1, 0.4), _M5)], eps=1e-6)

# one owner and three readers; as many identity experts as others, every one chosen
_M6 = moe(32, 2, 4, identity=2, shared=48)
TINY_P6 = model(64, 48, 2.0, [layer(latent(4, 16, 16, 16, 32, 0.3), _M6)]
                + [layer(latent(4, 16, 16, 16, 32, 0.3, kv_from=0), _M6) for _ in range(3)])

# sizes nearer a real model's; every expert chosen (every row is compared in bfloat16)
_M7 = moe(64, 2, 3, identity=1, groups=(3, 3), shared=160)
_P7 = pair((4, 1, 128, 128, 0.09, 25.0, (250000.0, 64)), (8, 64, 128, 2, 4, 2), 0.7, 0.8)
TINY_P7 = model(512, 256, 2.4, [layer(latent(4, 64, 64, 64, 192, 0.09), _M7), layer(_P7, _M7),
                                layer(latent(2, 128, 64, 64, 192, 0.07, kv_from=0), _M7), layer(_P7, _M7)])

# cached rows longer than the matrix cores take, and longer than 512
TINY_P8 = model(80, 48, 1.5, [layer(latent(2, 16, 24, 16, 520, 0.1), moe(16, 2, 2)),
                              layer(latent(3, 8, 32, 8, 272, 0.15), None),
                              layer(latent(2, 8, 24, 24, 520, 0.15, kv_from=0), moe(16, 1, 2, identity=1))])

# (configuration, seed, deviation of the matrices)
CONFIGS = {"P1": (TINY_P1, 61, 0.2), "P2": (TINY_P2, 62, 0.2), "P3": (TINY_P3, 63, 0.12), "P4": (TINY_P4, 64, 0.2),
           "P5": (TINY_P5, 65, 0.15), "P6": (TINY_P6, 66, 0.2), "P7": (TINY_P7, 67, 0.06), "P8": (TINY_P8, 68, 0.12)}


def make_model(which: str, folder: str, std: float = 0.0) -> str:
    from xyntetik_runner_amd.weights import write_random_model
    config, seed, own = CONFIGS[which]
    return write_random_model(config, folder, seed=seed, std=std or own, norm_jitter=0.1, dtype="bfloat16")
