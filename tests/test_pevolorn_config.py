"""Pevolorn without a GPU: the config's refusals by key, the spec it builds, the caches and states of its layers, layers that
read other layers' rows, the random-weights writer, and the plain mechanisms against closed forms."""
import json

import numpy as np
import pytest
import torch

import plain_pevolorn as P
from pevolorn_tiny import CONFIGS, TINY_P1, TINY_P2, TINY_P4, TINY_P5, make_model


def parse(raw):
    from xyntetik_runner_amd.config import config_from_dict
    return config_from_dict(raw)


def test_config_reads_every_size_and_constant():
    arch, cfg = parse(TINY_P1)
    assert arch.name == "Pevolorn" and (cfg.vocab, cfg.width, cfg.eps, cfg.alpha) == (200, 64, 1e-5, 1.7)
    a, b = cfg.layers[0].mixer.latent, cfg.layers[2].mixer.latent
    assert (a.heads, a.dim, a.rot_dim, a.vdim, a.kv_rank, a.scale, a.rot_base, a.rot_dims, a.kv_from) == (4, 16, 16, 24, 32, 0.3, 10000.0, 16, None)
    assert (b.heads, b.dim, b.vdim, b.kv_from) == (2, 24, 16, 0) and cfg.layers[2].mlp is None
    m = cfg.layers[1].mixer
    assert (m.kind, m.left_scale, m.right_scale) == ("parallel", 0.8, 0.5)
    l, r = m.left, m.right
    assert (l.heads, l.kv_heads, l.dim, l.vdim, l.scale, l.softcap, l.rot_base, l.rot_dims) == (4, 2, 32, 16, 0.25, 9.0, 10000.0, 16)
    assert (r.heads, r.vdim, r.state, r.groups, r.conv, r.norm_groups) == (4, 16, 24, 2, 3, 2)
    e = cfg.layers[4].mlp
    assert (e.ff, e.experts, e.identity, e.top, e.groups, e.keep_groups, e.shared_ff) == (24, 6, 2, 2, 4, 2, 40)
    assert (cfg.layers[4].mixer.left.softcap, cfg.layers[4].mixer.left.rot_dims, cfg.layers[4].mixer.right_scale) == (0.0, 0, -0.7)
    _, c2 = parse(TINY_P2)
    e = c2.layers[0].mlp
    assert (e.identity, e.groups, e.keep_groups, e.shared_ff) == (1, 1, 1, 0)
    _, c4 = parse(TINY_P4)          # a "rot" that turns no channel
    assert c4.layers[0].mixer.left.rot_dims == 0 and c4.alpha == 0.6
    nulls = json.loads(json.dumps(TINY_P1))
    nulls["layers"][1]["mixer"]["left"]["softcap"] = nulls["layers"][0]["mixer"]["kv_from"] = nulls["layers"][4]["mlp"]["shared"] = None
    nulls["layers"][4]["mlp"]["router"]["groups"] = nulls["layers"][4]["mlp"]["router"]["identity"] = None
    _, cn = parse(nulls)
    e = cn.layers[4].mlp
    assert cn.layers[1].mixer.left.softcap == 0.0 and (e.identity, e.groups, e.shared_ff) == (0, 1, 0)


def put(raw, path, value):
    raw = json.loads(json.dumps(raw))
    node = raw
    for key in path[:-1]:
        node = node[key]
    if value is KeyError:
        del node[path[-1]]
    else:
        node[path[-1]] = value
    return raw


LEFT, RIGHT, LATENT, MLP = ("layers", 1, "mixer", "left"), ("layers", 1, "mixer", "right"), ("layers", 0, "mixer"), ("layers", 4, "mlp")


@pytest.mark.parametrize("path,value,word", [
    (("vocab",), 0, "vocab"), (("norm",), None, "norm"), (("norm", "eps"), -1.0, "eps"), (("postln_alpha",), KeyError, "postln_alpha"),
    (("layers", 0, "type"), "attention", "type"), (LATENT, None, "mixer"), (LATENT + ("kv_rank",), 0, "kv_rank"),
    (LATENT + ("scale",), KeyError, "scale"), (LATENT + ("rot", "dims"), 18, "dims"), (LATENT + ("rot", "dims"), 7, "dims"),
    (LATENT + ("rot", "base"), 0.0, "base"), (LATENT + ("kv_from",), 0, "kv_from"), (("layers", 2, "mixer", "kv_from"), 1, "kv_from"),
    (("layers", 2, "mixer", "kv_from"), 3, "kv_from"), (("layers", 3, "mixer", "kv_from"), 2, "kv_from"),
    (("layers", 2, "mixer", "kv_rank"), 48, "kv_rank"), (("layers", 2, "mixer", "rot", "base"), 99.0, "rotation"),
    (("layers", 2, "mixer", "rot", "dims"), 8, "rotation"), (LEFT, None, "left"), (RIGHT, None, "right"), (LEFT + ("kv_heads",), 3, "kv_heads"),
    (LEFT + ("scale",), KeyError, "scale"), (LEFT + ("softcap",), -1.0, "softcap"), (LEFT + ("rot", "dims"), 34, "dims"),
    (RIGHT + ("groups",), 3, "groups"), (RIGHT + ("norm_groups",), 7, "norm_groups"), (RIGHT + ("conv",), 0, "conv"), (RIGHT + ("state",), KeyError, "state"),
    (MLP + ("kind",), "dense", "kind"), (MLP + ("expert",), None, "expert"), (MLP + ("router",), None, "router"), (MLP + ("router", "top"), 9, "top"),
    (MLP + ("router", "groups", "count"), 3, "groups"), (MLP + ("router", "groups", "keep"), 5, "keep"), (MLP + ("router", "top"), 5, "choices"),
    (MLP + ("router", "identity"), -1, "identity"), (MLP + ("shared", "ff"), KeyError, "ff"),
])
def test_config_refuses_by_key(path, value, word):
    from xyntetik_runner_amd.config import ConfigError
    with pytest.raises(ConfigError) as e:
        parse(put(TINY_P1, path, value))
    assert word in str(e.value)


def test_spec_caches_states_and_tensors():
    from xyntetik_runner_amd.cache import cache_groups
    from xyntetik_runner_amd.engine.model import Model
    arch, cfg = parse(TINY_P1)
    spec = arch.build_spec(cfg)
    assert [(s.layer, s.cache_of) for s in spec.order] == [(0, None), (1, None), (2, 0), (3, None), (4, None)]
    model = Model(spec)
    kv, st, of = model.cache_needs()
    assert of == [None, None, 0, None, None]
    assert [(k.num_kv_heads, k.head_dim, k.value_dim, k.window) for k in kv] == [
        (1, 48, 32, None), (2, 32, 16, None), (1, 48, 32, None), (1, 32, 16, None), (1, 16, 32, None)]
    specs, owners = cache_groups(kv, of)
    assert owners == [1, 1, 1, 1]
    assert st[0] is None and sorted(st[1]) == ["mixer.right.S", "mixer.right.conv"] and st[1]["mixer.right.conv"].shape == (2, 64 + 96)
    assert all(s.dtype == torch.float32 for s in st[1].values())
    shapes = {"embed": (200, 64), "final.norm": (64,), "l0.norm1": (64,), "l0.norm2": (64,), "l0.mix.q": (128, 64), "l0.mix.dkv": (48, 64),
              "l0.mix.dkv.norm": (32,), "l0.mix.uk": (64, 32), "l0.mix.uv": (96, 32), "l0.mix.g": (4, 64), "l0.mix.o": (64, 96),
              "l4.mlp.router": (8, 64), "l4.mlp.correction": (8,), "l4.mlp.e5.up": (24, 64), "l4.mlp.e5.down": (64, 24), "l4.mlp.shared.up": (40, 64),
              "l4.mlp.shared.down": (64, 40), "l1.mix.left.q": (128, 64), "l1.mix.left.q.b": (128,), "l1.mix.left.k.b": (64,), "l1.mix.left.v": (32, 64),
              "l1.mix.left.g": (4, 64), "l1.mix.left.o": (64, 64), "l1.mix.left.o.b": (64,), "l1.mix.right.in": (64 + 160 + 4, 64),
              "l1.mix.right.conv": (160, 3), "l1.mix.right.conv.b": (160,), "l1.mix.right.A_log": (4,), "l1.mix.right.dt_bias": (4,),
              "l1.mix.right.D": (4,), "l1.mix.right.norm": (64,), "l1.mix.right.o": (64, 64), "l2.mix.q": (80, 64), "l2.norm2": (64,)}
    names = model.expected()
    for name, shape in shapes.items():
        assert names[name].shape == shape, name
    assert not any(n in names for n in ("head", "l2.mix.dkv", "l2.mix.dkv.norm", "l4.mlp.e6.up", "l4.mlp.shared.gate", "l1.mix.left.q.norm", "l2.mlp.router"))
    assert names["l2.norm2"].optional and not names["l0.norm2"].optional
    assert model.capturable()


def test_pages_are_held_for_owners_only():
    from xyntetik_runner_amd.cache import CacheStorage
    from xyntetik_runner_amd.engine.model import Model
    arch, cfg = parse(TINY_P5)
    kv, st, of = Model(arch.build_spec(cfg)).cache_needs()
    store = CacheStorage(kv, st, of, 16, 5, 2, torch.float32, torch.device("cpu"))
    assert [lc.owns for lc in store.layers] == [True, False, True, False, True]
    assert store.layers[1].k is store.layers[0].k and store.layers[3].v is store.layers[0].v
    assert store.layers[0].v.shape[2] == 20 and store.layers[0].k.shape[3] == 32


def test_parts_refuse_what_they_do_not_build():
    from xyntetik_runner_amd.config import PartSpec
    from xyntetik_runner_amd.parts import make_part
    from xyntetik_runner_amd.parts.base import make_block
    for kind, params, word in [
            ("latent_attention", dict(hidden_size=8, num_heads=1, head_dim=4, rot_dim=4, v_head_dim=4, q_rank=4, kv_rank=4, scale=1.0, eps=0.0, kv_shared=True), "query latent"),
            ("latent_attention", dict(hidden_size=8, num_heads=1, head_dim=4, rot_dim=4, v_head_dim=4, q_rank=None, kv_rank=1030, scale=1.0, eps=0.0), "1030"),
            ("state_space", dict(hidden_size=8, num_heads=2, v_head_dim=4, state_size=300, groups=1, conv_taps=4, eps=0.0), "300"),
            ("state_space", dict(hidden_size=8, num_heads=2, v_head_dim=4, state_size=8, groups=1, conv_taps=4, eps=0.0, norm_groups=3), "equal parts")]:
        with pytest.raises(ValueError) as e:
            make_part("mixer", PartSpec(kind, params))
        assert word in str(e.value)
    base = dict(hidden_size=8, intermediate_size=4, num_experts=4, top=2)
    for more, word in ((dict(identity=-1), "identity"), (dict(identity=2, groups=4, keep_groups=2), "groups"), (dict(group_score="mean"), "mean"),
                       (dict(identity=1, routing="table", vocab_size=9), "router")):
        with pytest.raises(ValueError) as e:
            make_part("feed_forward", PartSpec("routed_experts", dict(base, **more)))
        assert word in str(e.value)
    late = PartSpec("head_rmsnorm", {"head_dim": 8, "eps": 0.0, "after_rotation": True, "temp_every": 4, "temp_coef": 0.1})
    with pytest.raises(ValueError) as e:
        make_part("mixer", PartSpec("paged_attention", dict(hidden_size=8, num_heads=1, num_kv_heads=1, head_dim=8, qk_transform=late)))
    assert "behind the rotation" in str(e.value)
    with pytest.raises(ValueError) as e:
        make_block("postnorm", object(), None, {n: make_part("norm", PartSpec("layernorm", {"size": 8, "eps": 0.0})) for n in ("mixer_norm", "feed_forward_norm")})
    assert "RMS norm" in str(e.value)


@pytest.mark.parametrize("which", sorted(CONFIGS))
def test_random_weights_load(which, tmp_path):
    from plain_llama import load_folder
    d = make_model(which, str(tmp_path))
    cfg, w = load_folder(d)
    out = P.forward(cfg, w, [1, 2, 3])
    assert out.shape == (3, cfg["vocab"]) and np.isfinite(out).all()
    assert abs(w["final.norm"].mean()) < 0.1            # stored around zero


# ----------------------------------------------------------------------------- the plain mechanisms
def test_plain_rotation_and_norms():
    x = np.zeros((3, 1, 6)); x[:, 0, 0] = 1.0; x[:, 0, 5] = 7.0
    y = P.rotate_half(x, 100.0, 4, first=2)
    for t in range(3):
        a = 2.0 + t
        assert np.allclose(y[t, 0], [np.cos(a), 0, np.sin(a), 0, 0, 7.0])
    assert np.allclose(P.centred_weight_norm(np.array([[3.0, 4.0]]), np.array([0.0, 1.0]), 0.0), np.array([[3.0, 8.0]]) / np.sqrt(12.5))
    assert np.allclose(P.gated_part_norm(np.array([[2.0, 0.0, 0.0, 9.0]]), np.full((1, 4), 50.0), 2, np.ones(4), 0.0), np.sqrt(2) * np.array([1, 0, 0, 1]))


def test_plain_state_space():
    """Without a decay the state sums what was written; with one the first write is scaled by every step behind it."""
    x, one = np.array([[1.0], [2.0], [3.0]]), np.ones((3, 1))
    dt = np.array([0.5, 1.0, 2.0])
    assert np.allclose(P.state_space(x, one, one, dt, 0.0)[:, 0], [0.5, 2.5, 8.5])
    assert np.allclose(P.state_space(x, one, one, dt, np.log(2.0))[:, 0], [0.5, 0.25 + 2.0, (0.25 + 2.0) / 4 + 6.0])
    assert np.allclose(P.causal_conv(np.array([[1.0], [10.0], [100.0]]), np.array([[3.0, 1.0]]), np.array([0.5]))[:, 0], [1.5, 13.5, 130.5])


def test_plain_choice_in_groups():
    """Four groups of two: the largest score of a group decides, and experts of the others are out even where all choice
    scores are negative."""
    z, corr = np.log(np.array([4.0, 1.0, 3.0, 3.0, 1.0, 1.0, 1.0, 2.0])), np.full(8, -2.0)
    chosen, w = P.route(z, corr, 2, 4, 1)
    assert list(chosen) == [0, 1] and np.allclose(w, [4 / 16, 1 / 16])
    chosen, w = P.route(z, corr, 3, 4, 2)
    assert list(chosen) == [0, 2, 3]
    corr[7] = 0.0
    assert list(P.route(z, corr, 2, 4, 1)[0]) == [7, 6]
    assert P.route_margin(z, np.zeros(8), 8, 1, 1) == np.inf


def test_plain_layers_that_read_another_layers_rows(tmp_path):
    """A reader's logits change with its owner's down projection and not with one of its own."""
    from plain_llama import load_folder
    cfg, w = load_folder(make_model("P1", str(tmp_path)))
    toks = [3, 7, 11, 2]
    base = P.forward(cfg, w, toks)
    w["l2.mix.dkv"] = np.ones_like(w["l0.mix.dkv"])
    assert np.array_equal(P.forward(cfg, w, toks), base)
    own = json.loads(json.dumps(cfg))
    del own["layers"][2]["mixer"]["kv_from"]
    w["l2.mix.dkv.norm"] = w["l0.mix.dkv.norm"]
    assert np.abs(P.forward(own, w, toks) - base).max() > 1e-3
