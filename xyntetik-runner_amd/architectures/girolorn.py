"""``Girolorn``: a decoder of soft-capped attention and routed experts whose layers may share their tensors, put together
from parts.

Every layer is pre-norm with layer norms (a weight, no bias): ``x += mixer(norm1(x)); x += feed_forward(norm2(x))``, the
feed-forward optional.  The mixer is attention whose values are its keys as projected; queries and keys are normed over
all their heads at once (RMS, a weight a channel of the whole projection), then rotated in neighbouring pairs by
frequencies that YaRN scales; scores pass a soft cap, and the softmax's denominator holds a learned sink a head.  The
feed-forward is a set of experts with both branches clamped, chosen by the largest router logits (with the router's bias)
and weighted by the softmax over the chosen ones, plus a shared expert of the same form that a sigmoid a token scales.
A layer with ``weights_of`` runs with another layer's tensors and a cache of its own: an entry of the run order, no layer.
The head has a table of its own; its logits pass a soft cap.
Tensors: ``embed``, ``l<i>.norm1``/``norm2``, ``l<i>.mix.*``, ``l<i>.mlp.*``, ``final.norm``, ``head``.
"""
from __future__ import annotations

from ..config import ExecStep, LayerSpec, ModelSpec, PartSpec, register_architecture
from ..config.girolorn import GirolornConfig
from ..parts.rotary import yarn_mscale


def _mixer_spec(cfg: GirolornConfig, i: int, prefix: str) -> PartSpec:
    m = cfg.layers[i].mixer
    position = None
    if m.rot_dims:
        s = m.rot_scaling
        scaling = ({"rope_type": "yarn", "factor": s.factor, "original_max_position_embeddings": s.original,
                    "beta_fast": s.fast, "beta_slow": s.slow} if s is not None else None)
        position = PartSpec("rotary", {"head_dim": m.dim, "theta": m.rot_base, "rotary_dim": m.rot_dims, "scaling": scaling,
                                       "interleaved": True, "mscale": yarn_mscale(s.factor) if s is not None else 1.0})
    return PartSpec("paged_attention", {
        "hidden_size": cfg.width, "num_heads": m.heads, "num_kv_heads": m.kv_heads, "head_dim": m.dim, "scale": m.scale,
        "bias": False, "values": "keys", "position": position, "softcap": m.softcap, "sink": "learned", "sink_name": "sink",
        "q_name": "q", "k_name": "k", "o_name": "o", "weight_suffix": "",
        "qk_transform": PartSpec("row_rmsnorm", {"q_size": m.heads * m.dim, "k_size": m.kv_heads * m.dim, "eps": cfg.eps,
                                                 "q_name": "q.norm", "k_name": "k.norm"})}, prefix=prefix)


def _mlp_spec(cfg: GirolornConfig, i: int, prefix: str):
    mlp = cfg.layers[i].mlp
    if mlp is None:
        return None
    return PartSpec("routed_experts", {
        "hidden_size": cfg.width, "intermediate_size": mlp.ff, "num_experts": mlp.experts, "top": mlp.top,
        "activation": "clamped_swish", "activation_param": mlp.limit, "scores": "logits", "correction_name": "router.b",
        "shared_size": mlp.shared_ff, "shared_activation": "clamped_swish", "shared_param": mlp.shared_limit,
        "shared_gate_name": "shared.sg" if mlp.shared_ff else None}, prefix=prefix)


def build_girolorn_spec(cfg: GirolornConfig) -> ModelSpec:
    E = cfg.width
    layers, at = [], {}
    for i, layer in enumerate(cfg.layers):
        if layer.weights_of is not None:
            continue
        p = f"l{i}."
        has_ff = layer.mlp is not None

        def norm(name, optional=False):
            return PartSpec("layernorm", {"size": E, "eps": cfg.eps, "weight_name": name, "optional": optional}, prefix=p)

        at[i] = len(layers)
        # a layer without a feed-forward has no use for its second norm; a file may still bring it
        layers.append(LayerSpec(
            mixer=_mixer_spec(cfg, i, p + "mix."), feed_forward=_mlp_spec(cfg, i, p + "mlp."),
            norms={"mixer_norm": norm("norm1"), "feed_forward_norm": norm("norm2", optional=not has_ff)},
            block="prenorm_optional"))
    order = [ExecStep(at[cfg.tensors_of(i)]) for i in range(len(cfg.layers))]
    return ModelSpec(
        architecture=cfg.architecture, hidden_size=E, vocab_size=cfg.vocab, max_position=cfg.max_position,
        embedding=PartSpec("token_embedding", {"vocab_size": cfg.vocab, "hidden_size": E, "weight_name": "embed"}),
        layers=layers, order=order,
        final_norm=PartSpec("layernorm", {"size": E, "eps": cfg.eps, "weight_name": "norm"}, prefix="final."),
        head=PartSpec("linear", {"vocab_size": cfg.vocab, "hidden_size": E, "tied": False, "weight_name": "head",
                                 "softcap": cfg.logit_softcap}))


register_architecture("Girolorn", GirolornConfig.from_dict, build_girolorn_spec)
