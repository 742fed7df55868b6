"""Girolorn without a GPU: the config's refusals by key, the spec it builds, the caches of its layer runs, layers that run
with other layers' tensors, YaRN's table, the random-weights writer, and the plain mechanisms against closed forms."""
import json
import math

import numpy as np
import pytest
import torch

import plain_girolorn as P
from girolorn_tiny import CONFIGS, TINY_G1, TINY_G2, TINY_G3, TINY_G4, TINY_G6, make_model


def parse(raw):
    from xyntetik_runner_amd.config import config_from_dict
    return config_from_dict(raw)


def test_config_reads_every_size_and_constant():
    arch, cfg = parse(TINY_G1)
    assert arch.name == "Girolorn" and cfg.vocab == 200 and cfg.width == 64 and cfg.eps == 1e-5 and cfg.logit_softcap == 12.0
    a, b = cfg.layers[0].mixer, cfg.layers[2].mixer
    assert (a.kind, a.heads, a.kv_heads, a.dim, a.scale, a.softcap, a.rot_base, a.rot_dims) == ("attention", 4, 2, 32, 0.3, 6.0, 10000.0, 16)
    s = a.rot_scaling
    assert (s.factor, s.original, s.fast, s.slow) == (8.0, 64.0, 16.0, 1.0)
    assert (b.kv_heads, b.rot_dims, b.rot_scaling) == (1, 64, None)
    m = cfg.layers[0].mlp
    assert (m.kind, m.ff, m.limit, m.experts, m.top, m.shared_ff, m.shared_limit) == ("moe", 24, 0.8, 8, 2, 40, 0.6)
    assert cfg.layers[2].mlp is None and [l.weights_of for l in cfg.layers] == [None, 0, None, 2, 0]
    assert [cfg.tensors_of(i) for i in range(5)] == [0, 0, 2, 2, 0]
    _, c2 = parse(TINY_G2)
    assert c2.logit_softcap == 0.0 and c2.layers[0].mixer.softcap == 0.0 and c2.layers[1].mlp.shared_ff == 0
    _, c3 = parse(TINY_G3)
    assert [c3.tensors_of(i) for i in range(4)] == [0, 0, 0, 3]
    _, c4 = parse(TINY_G4)          # no "rot", and a "rot" that turns no channel
    assert [l.mixer.rot_dims for l in c4.layers] == [0, 0]
    nulls = json.loads(json.dumps(TINY_G1))
    nulls["logit_softcap"] = nulls["layers"][2]["mixer"]["softcap"] = nulls["layers"][3]["mixer"]["softcap"] = None
    nulls["layers"][2]["mixer"]["rot"]["scaling"] = nulls["layers"][3]["mixer"]["rot"]["scaling"] = None
    _, cn = parse(nulls)
    assert cn.logit_softcap == 0.0 and cn.layers[2].mixer.softcap == 0.0 and cn.layers[2].mixer.rot_scaling is None


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


@pytest.mark.parametrize("path,value,word", [
    (("vocab",), 0, "vocab"), (("norm",), None, "norm"), (("norm", "eps"), -1.0, "eps"), (("logit_softcap",), -3.0, "logit_softcap"),
    (("layers", 0, "type"), "wkv", "type"), (("layers", 2, "mixer"), None, "mixer"), (("layers", 2, "mixer", "kv_heads"), 3, "kv_heads"),
    (("layers", 2, "mixer", "scale"), KeyError, "scale"), (("layers", 2, "mixer", "scale"), 0.0, "scale"),
    (("layers", 2, "mixer", "softcap"), -1.0, "softcap"), (("layers", 2, "mixer", "vdim"), 32, "vdim"),
    (("layers", 2, "mixer", "rot", "dims"), 7, "dims"), (("layers", 2, "mixer", "rot", "dims"), 66, "dims"),
    (("layers", 0, "mixer", "rot", "scaling", "factor"), 0.0, "factor"), (("layers", 0, "mixer", "rot", "scaling", "original"), KeyError, "original"),
    (("layers", 0, "mixer", "rot", "scaling", "slow"), 0, "slow"), (("layers", 0, "mixer", "rot", "base"), 1.0, "base"),
    (("layers", 0, "mlp", "kind"), "dense", "kind"), (("layers", 0, "mlp", "expert"), None, "expert"), (("layers", 0, "mlp", "router", "top"), 9, "top"),
    (("layers", 0, "mlp", "expert", "limit"), KeyError, "limit"), (("layers", 0, "mlp", "shared", "ff"), KeyError, "ff"),
    (("layers", 1, "weights_of"), 5, "weights_of"), (("layers", 1, "weights_of"), 1, "weights_of"), (("layers", 1, "weights_of"), 2, "weights_of"),
    (("layers", 0, "weights_of"), 4, "weights_of"), (("layers", 4, "mlp", "expert", "limit"), 0.9, "weights_of"),
    (("layers", 3, "mixer", "scale"), 0.21, "weights_of"),
])
def test_config_refuses_by_key(path, value, word):
    from xyntetik_runner_amd.config import ConfigError
    with pytest.raises(ConfigError) as e:
        parse(put(TINY_G1, path, value))
    assert word in str(e.value)


def test_spec_caches_and_tensors_of_every_run():
    from xyntetik_runner_amd.engine.model import Model
    arch, cfg = parse(TINY_G1)
    spec = arch.build_spec(cfg)
    assert [(s.layer, s.cache_of) for s in spec.order] == [(0, None), (0, None), (1, None), (1, None), (0, None)] and len(spec.layers) == 2
    model = Model(spec)
    kv, st, of = model.cache_needs()
    assert all(o is None for o in of) and all(s is None for s in st)        # every run owns what it keeps
    assert [(k.num_kv_heads, k.head_dim, k.value_dim, k.window) for k in kv] == [(2, 32, 32, None)] * 2 + [(1, 64, 64, None)] * 2 + [(2, 32, 32, None)]
    names = model.expected()
    shapes = {"embed": (200, 64), "head": (200, 64), "final.norm": (64,), "l0.norm1": (64,), "l0.norm2": (64,), "l0.mix.q": (128, 64),
              "l0.mix.k": (64, 64), "l0.mix.o": (64, 128), "l0.mix.q.norm": (128,), "l0.mix.k.norm": (64,), "l0.mix.sink": (4,),
              "l0.mlp.router": (8, 64), "l0.mlp.router.b": (8,), "l0.mlp.e7.gate": (24, 64), "l0.mlp.e7.down": (64, 24),
              "l0.mlp.shared.up": (40, 64), "l0.mlp.shared.sg": (1, 64), "l2.mix.k": (64, 64), "l2.mix.sink": (2,)}
    for name, shape in shapes.items():
        assert tuple(names[name].shape) == shape, name
    assert not any(n.startswith(("l1.", "l3.", "l4.")) or n.startswith("l2.mlp") or ".v" in n for n in names)
    assert names["l2.norm2"].optional and not names["l0.norm2"].optional
    arch2, cfg2 = parse(TINY_G2)
    assert "l1.mlp.shared.sg" not in Model(arch2.build_spec(cfg2)).expected()
    # a feed-forward of one layer, six entries of its order, one set of tensors
    arch6, cfg6 = parse(TINY_G6)
    m6 = Model(arch6.build_spec(cfg6))
    assert len(m6.blocks) == 1 and [s.layer for s in m6.spec.order] == [0] * 4


@pytest.mark.parametrize("dims,base,scaling", [
    (16, 10000.0, (8.0, 64, 16.0, 1.0)), (6, 500.0, (4.0, 100.0, 8.0, 8.0)), (128, 1e6, (4.0, 4096, 32.0, 1.0)),
    (64, 500000.0, (2.0, 512, 32.0, 2.0)), (16, 100.0, (0.5, 4096, 1000.0, 0.01)), (24, 20000.0, (16.0, 32, 4.0, 0.5)),
    (8, 10.0, (3.0, 7, 6.0, 1.5)), (2, 50.0, (4.0, 64, 32.0, 1.0)), (32, 10000.0, (1.0, 2048, 32.0, 1.0)), (32, 5.0, None),
])
def test_yarn_table_of_the_rotation(dims, base, scaling):
    from xyntetik_runner_amd.parts import rotary_inv_freq, yarn_mscale
    own = dict(zip(("factor", "original", "fast", "slow"), scaling)) if scaling else None
    want, mult = P.yarn(dims, base, own)
    named = ({"rope_type": "yarn", "factor": scaling[0], "original_max_position_embeddings": scaling[1], "beta_fast": scaling[2],
              "beta_slow": scaling[3]} if scaling else None)
    assert np.allclose(rotary_inv_freq(dims, base, named).numpy(), want, rtol=1e-12, atol=0)
    assert mult == (yarn_mscale(scaling[0]) if scaling else 1.0)


def test_yarn_by_hand():
    # 8 channels, base 16, 2 pi 64 positions: pair number t turns 64 / 16^(t/4) times; 64 turns at pair 0, 16 at pair 2, 4 at 4
    f, mult = P.yarn(8, 16.0, {"factor": 2.0, "original": 2 * math.pi * 64, "fast": 40.0, "slow": 10.0})
    # 40 turns lie at pair 0.68 (floor 0), 10 at pair 2.68 (ceiling 3): the ramp is 0, 1/3, 2/3, 1
    g = 16.0 ** (-np.arange(4) / 4)
    assert np.allclose(f, g * np.array([1.0, 5 / 6, 4 / 6, 0.5])) and mult == 1.0 + 0.1 * math.log(2.0)


def test_parts_refuse_what_they_cannot_do():
    from xyntetik_runner_amd.parts import LinearHead, PagedAttention, RoutedExperts
    with pytest.raises(ValueError, match="soft cap"):
        PagedAttention(64, 4, 2, 16, softcap=-1.0)
    with pytest.raises(ValueError, match="soft cap"):
        LinearHead(10, 8, softcap=-1.0)
    with pytest.raises(ValueError, match="groups"):
        RoutedExperts(64, 32, 8, 2, scores="logits", groups=2, keep_groups=1)
    with pytest.raises(ValueError, match="shared"):
        RoutedExperts(64, 32, 8, 2, scores="logits", shared_gate_name="sg")


@pytest.mark.parametrize("which", sorted(CONFIGS))
def test_random_model_round_trip(tmp_path, which):
    from plain_llama import load_folder
    d = make_model(which, str(tmp_path))
    cfg, w = load_folder(d)
    logits = P.forward(cfg, w, [1, 2, 3, 4, 5])
    assert cfg["architecture"] == "Girolorn" and logits.shape == (5, cfg["vocab"]) and np.isfinite(logits).all()
    cap = cfg.get("logit_softcap")
    assert not cap or np.abs(logits).max() < cap


def test_values_that_are_the_keys_stand_once_in_the_input_matrix():
    """Where the kernel behind the product takes values from the keys' columns; an attention whose transform is another
    keeps the rows twice."""
    from xyntetik_runner_amd.config import PartSpec
    from xyntetik_runner_amd.parts import PagedAttention, Runtime

    class Packs:
        def pack_weight(self, w, gated=False):
            return w
    rows = {}
    for kind, params in (("row_rmsnorm", {"q_size": 32, "k_size": 16}), ("head_rmsnorm", {"head_dim": 8})):
        a = PagedAttention(24, 4, 2, 8, values="keys", qk_transform=PartSpec(kind, dict(params, eps=1e-5)))
        tensors = {n: torch.zeros(s.shape) for n, s in a.param_specs().items()}
        a.bind(tensors, Runtime(torch.device("cpu"), torch.float32, Packs()))
        rows[kind] = a.w_in.shape[0]
    assert rows == {"row_rmsnorm": 48, "head_rmsnorm": 64}


def test_plain_mechanisms_against_closed_forms():
    rng = np.random.default_rng(0)
    # a sink: one key of score s and a sink of score s share the weight; the cap bends the key's score and not the sink
    q, k, v = np.ones((1, 1, 2)), np.ones((1, 1, 2)), np.full((1, 1, 3), 4.0)
    assert np.allclose(P.attend(q, k, v, 0.5, None, np.array([1.0])), 2.0)
    assert np.allclose(P.attend(q, k, v, 0.5, 0.25, np.array([0.25 * np.tanh(4.0)])), 2.0)
    assert np.allclose(P.softcap(np.array([1e-3, 1e6, -1e6]), 3.0), [1e-3, 3.0, -3.0], atol=1e-9)
    # the layer norm takes off the mean, the row norm does not
    x = np.array([[1.0, 3.0]])
    assert np.allclose(P.layer_norm(x, np.array([1.0, 2.0]), 0.0), [[-1.0, 2.0]])
    assert np.allclose(P.rms_norm(x, np.ones(2), 4.0), x / 3.0)
    # rotation: neighbours turn together, position 0 is multiplied only, the rest passes
    x = rng.normal(size=(3, 1, 6))
    f = np.array([1.0, 0.1])
    y = P.rotate_neighbours(x, f, 1.5)
    assert np.allclose(y[0, 0, :4], 1.5 * x[0, 0, :4]) and np.allclose(y[..., 4:], x[..., 4:])
    assert np.allclose(y[2, 0, 2], 1.5 * (x[2, 0, 2] * np.cos(0.2) - x[2, 0, 3] * np.sin(0.2)))
    assert np.allclose(y[2, 0, 3], 1.5 * (x[2, 0, 3] * np.cos(0.2) + x[2, 0, 2] * np.sin(0.2)))
    assert np.allclose(P.rotate_neighbours(x[2:], f, 1.5, first=2), y[2:])
    # the choice: ties go to the lower number, the weights add up to one over the chosen alone
    chosen, wts = P.choose(np.array([0.0, 2.0, 2.0, 1.0]), 2)
    assert list(chosen) == [1, 2] and np.allclose(wts, 0.5) and P.choice_margin(np.array([0.0, 2.0, 2.0, 1.0]), 2) == 1.0
    # an expert: the gate is cut from above only, the other branch on both sides
    w = {"gate": np.eye(3), "up": np.array([[5.0, 0, 0], [0, -5.0, 0], [0, 0, 0.1]]), "down": np.eye(3)}
    out = P.clamped_expert(np.array([2.0, -2.0, 0.5]), w, "", 1.0)
    sw = lambda g: g / (1.0 + np.exp(-1.702 * g))
    assert np.allclose(out, [sw(1.0) * 2.0, sw(-2.0) * 2.0, sw(0.5) * 1.05])
