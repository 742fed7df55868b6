"""``Pevolorn``: a decoder whose residual stream is normed behind every sum, put together from parts.

Every layer: ``x <- norm1(alpha x + mixer(x)); x <- norm2(alpha x + feed_forward(x))``, the feed-forward optional; mixer and
feed-forward take the stream as it is, with no norm in front.  Norm weights are stored around zero (RMS norms).  Mixers by ``type``:

* "latent_attention": keys and values from one cached latent a token, with queries straight from the input, one rotated key
  part that the heads share (rotate-half layout) and a sigmoid gate a head; a layer with ``kv_from`` has no latent of its
  own and reads an earlier layer's cached rows.
* "parallel": attention with biased projections, a rotation of a part of every head, queries and keys over their root mean
  square head by head behind it, soft-capped scores and a sigmoid gate a head, beside a selective state space; the result is
  a weighted sum of the two, made as one product over both sides' rows.

The feed-forward is a set of experts ``down(relu(up h)^2)`` chosen by softmax scores with a correction, limited to the best
groups (a group scores its largest), weighted by the scores themselves; the last choices are identity experts, whose output
is the input; a shared expert of the same form is added.  The head is the embedding table.
Tensors: ``embed``, ``l<i>.norm1``/``norm2``, ``l<i>.mix.*``, ``l<i>.mlp.*``, ``final.norm``.
"""
from __future__ import annotations

from ..config import ExecStep, LayerSpec, ModelSpec, PartSpec, register_architecture
from ..config.pevolorn import PevolornConfig

NORM_WEIGHT_OFFSET = 1.0    # a norm's stored weight is its difference from one
EXPERT_WEIGHT_SCALE = 1.0   # the chosen scores are the weights, as they are


def _mixer_spec(cfg: PevolornConfig, i: int, prefix: str) -> PartSpec:
    m, E = cfg.layers[i].mixer, cfg.width
    if m.kind == "latent_attention":
        a = m.latent
        return PartSpec("latent_attention", {
            "hidden_size": E, "num_heads": a.heads, "head_dim": a.dim, "rot_dim": a.rot_dim, "v_head_dim": a.vdim, "q_rank": None,
            "kv_rank": a.kv_rank, "scale": a.scale, "eps": cfg.eps, "rot_dims": a.rot_dims, "rot_base": a.rot_base,
            "pairs": "halves", "gate_name": "g", "kv_shared": a.kv_from is not None}, prefix=prefix)
    a, r = m.left, m.right
    left = PartSpec("paged_attention", {
        "hidden_size": E, "num_heads": a.heads, "num_kv_heads": a.kv_heads, "head_dim": a.dim, "v_head_dim": a.vdim,
        "scale": a.scale, "softcap": a.softcap, "bias": True, "out_bias": True, "gate_name": "g",
        "position": PartSpec("rotary", {"head_dim": a.dim, "theta": a.rot_base, "rotary_dim": a.rot_dims}) if a.rot_dims else None,
        "qk_transform": PartSpec("head_rmsnorm", {"head_dim": a.dim, "eps": cfg.eps, "weighted": False, "after_rotation": True}),
        "q_name": "q", "k_name": "k", "v_name": "v", "o_name": "o", "weight_suffix": "", "bias_suffix": ".b"})
    right = PartSpec("state_space", {
        "hidden_size": E, "num_heads": r.heads, "v_head_dim": r.vdim, "state_size": r.state, "groups": r.groups,
        "conv_taps": r.conv, "norm_groups": r.norm_groups, "eps": cfg.eps})
    return PartSpec("parallel_mixers", {"hidden_size": E, "left": left, "right": right, "left_scale": m.left_scale,
                                        "right_scale": m.right_scale, "joint": True}, prefix=prefix)


def _mlp_spec(cfg: PevolornConfig, i: int, prefix: str):
    mlp = cfg.layers[i].mlp
    if mlp is None:
        return None
    return PartSpec("routed_experts", {
        "hidden_size": cfg.width, "intermediate_size": mlp.ff, "num_experts": mlp.experts, "identity": mlp.identity,
        "top": mlp.top, "activation": "relu2", "scores": "softmax", "groups": mlp.groups, "keep_groups": mlp.keep_groups,
        "group_score": "max", "weight_scale": EXPERT_WEIGHT_SCALE, "shared_size": mlp.shared_ff, "shared_activation": "relu2"},
        prefix=prefix)


def build_pevolorn_spec(cfg: PevolornConfig) -> ModelSpec:
    E = cfg.width

    def norm(prefix, name, optional=False):
        return PartSpec("rmsnorm", {"size": E, "eps": cfg.eps, "weight_name": name, "optional": optional,
                                    "weight_offset": NORM_WEIGHT_OFFSET}, prefix=prefix)

    layers, order = [], []
    for i, layer in enumerate(cfg.layers):
        p = f"l{i}."
        has_ff = layer.mlp is not None
        # a layer without a feed-forward has no use for its second norm; a file may still bring it
        layers.append(LayerSpec(
            mixer=_mixer_spec(cfg, i, p + "mix."), feed_forward=_mlp_spec(cfg, i, p + "mlp."),
            norms={"mixer_norm": norm(p, "norm1"), "feed_forward_norm": norm(p, "norm2", optional=not has_ff)},
            block="postnorm", block_params={"alpha": cfg.alpha}))
        order.append(ExecStep(i, cache_of=layer.mixer.latent.kv_from if layer.mixer.latent is not None else None))
    return ModelSpec(
        architecture=cfg.architecture, hidden_size=E, vocab_size=cfg.vocab, max_position=cfg.max_position,
        embedding=PartSpec("token_embedding", {"vocab_size": cfg.vocab, "hidden_size": E, "weight_name": "embed"}),
        layers=layers, order=order, final_norm=norm("final.", "norm"),
        head=PartSpec("linear", {"vocab_size": cfg.vocab, "hidden_size": E, "tied": True}))


register_architecture("Pevolorn", PevolornConfig.from_dict, build_pevolorn_spec)
