"""``GirolornConfig``: the hyper-parameters of a Girolorn decoder, typed.

config.json of this design is nested: ``vocab``, ``width``, ``norm.eps``, ``logit_softcap`` (absent: the logits stay
as they are) and a list ``layers`` whose entries name their mixer (``type``), the mixer's sizes (``mixer``), the
feed-forward (``mlp``, or null for a layer without one) and, where a layer runs with another layer's tensors,
that layer (``weights_of``; the rest of the entry is then that layer's).  Every size and constant that can differ
between models is read here and nowhere else; what the design fixes lives in the parts and in the builder.

====================  =====================================================================
type                  keys of ``mixer``
====================  =====================================================================
attention             heads, kv_heads, dim, vdim (the values are the keys: equal to dim), scale, softcap (absent: none),
                      rot.base, rot.dims (absent or 0: no rotation), rot.scaling (absent: none; factor, original,
                      fast, slow)
====================  =====================================================================

``mlp``: ``kind`` "moe" with ``expert.ff``, ``expert.limit``, ``router.experts``, ``router.top`` and ``shared.ff``,
``shared.limit`` (absent: no shared expert).
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, List, Mapping, Optional, Tuple

from .base import ConfigError, Fields

MIXERS = ("attention",)
MLPS = ("moe",)


@dataclass(frozen=True)
class GirolornScaling:
    factor: float
    original: float
    fast: float
    slow: float


@dataclass(frozen=True)
class GirolornMixer:
    kind: str
    heads: int
    kv_heads: int
    dim: int
    scale: float
    softcap: float = 0.0                # 0: none
    rot_base: float = 0.0
    rot_dims: int = 0                   # 0: no rotation
    rot_scaling: Optional[GirolornScaling] = None


@dataclass(frozen=True)
class GirolornMLP:
    kind: str
    ff: int
    limit: float
    experts: int
    top: int
    shared_ff: int = 0                  # 0: no shared expert
    shared_limit: float = 0.0


@dataclass(frozen=True)
class GirolornLayer:
    mixer: GirolornMixer
    mlp: Optional[GirolornMLP]
    weights_of: Optional[int] = None    # the layer whose tensors this one runs with (None: its own)


@dataclass(frozen=True)
class GirolornConfig:
    architecture: str
    vocab: int
    width: int
    eps: float
    layers: Tuple[GirolornLayer, ...]
    logit_softcap: float                # 0: none
    max_position: int

    def tensors_of(self, i: int) -> int:
        """The layer whose tensors layer ``i`` runs with."""
        while self.layers[i].weights_of is not None:
            i = self.layers[i].weights_of
        return i

    @staticmethod
    def from_dict(raw: Mapping[str, Any]) -> "GirolornConfig":
        f = Fields(raw)
        norm = f.mapping("norm")
        if norm is None:
            raise ConfigError("config.json: 'norm' is a required object")
        fields = f.mappings("layers")
        layers: List[GirolornLayer] = []
        for lf in fields:
            kind = lf.string("type", choices=MIXERS)
            mf = lf.mapping("mixer")
            if mf is None:
                raise ConfigError(f"{lf.where}: 'mixer' is required")
            layers.append(GirolornLayer(_mixer(kind, mf), _mlp(lf),
                                        weights_of=lf.integer("weights_of", default=None, lo=0, hi=len(fields) - 1)))
        _check_sharing(fields, layers)
        return GirolornConfig(
            architecture="Girolorn", vocab=f.integer("vocab"), width=f.integer("width"), eps=norm.number("eps", lo=0.0),
            layers=tuple(layers), logit_softcap=f.number("logit_softcap", default=0.0, lo=0.0),
            max_position=f.integer("max_position", default=1 << 20, hi=1 << 30))


def _check_sharing(fields, layers) -> None:
    """Every chain of ``weights_of`` ends in a layer with tensors of its own, and a layer that runs with another's
    tensors has its sizes and constants."""
    for i, (lf, layer) in enumerate(zip(fields, layers)):
        seen, j = {i}, i
        while layers[j].weights_of is not None:
            j = layers[j].weights_of
            if j in seen:
                raise ConfigError(f"{lf.where}: 'weights_of' leads back to layer {j}: no layer of the chain has tensors of its own")
            seen.add(j)
        if (layers[j].mixer, layers[j].mlp) != (layer.mixer, layer.mlp):
            raise ConfigError(f"{lf.where}: 'weights_of' names layer {j}, whose mixer or feed-forward differs from this entry's")


def _mlp(lf: Fields) -> Optional[GirolornMLP]:
    mlp = lf.mapping("mlp")
    if mlp is None:
        return None
    kind = mlp.string("kind", choices=MLPS)
    ef, rf = mlp.mapping("expert"), mlp.mapping("router")
    if ef is None or rf is None:
        raise ConfigError(f"{mlp.where}: 'expert' and 'router' are required objects")
    experts = rf.integer("experts", hi=1 << 10)
    sf = mlp.mapping("shared")
    return GirolornMLP(kind, ef.integer("ff"), ef.number("limit", lo=0.0), experts=experts, top=rf.integer("top", hi=experts),
                       shared_ff=sf.integer("ff") if sf is not None else 0,
                       shared_limit=sf.number("limit", lo=0.0) if sf is not None else 0.0)


def _mixer(kind: str, mf: Fields) -> GirolornMixer:
    heads = mf.integer("heads")
    kv_heads = mf.integer("kv_heads", default=heads, hi=heads)
    if heads % kv_heads:
        raise ConfigError(f"{mf.where}: {heads} heads are not a multiple of kv_heads = {kv_heads}")
    dim = mf.integer("dim")
    vdim = mf.integer("vdim", default=dim)
    if vdim != dim:
        raise ConfigError(f"{mf.where}: the values are the keys, so vdim = {vdim} must equal dim = {dim}")
    rot = mf.mapping("rot")
    dims = rot.integer("dims", default=0, lo=0, hi=dim) if rot is not None else 0
    if dims % 2:
        raise ConfigError(f"{mf.where}: rot.dims = {dims} must be even")
    scaling = None
    sf = rot.mapping("scaling") if dims else None
    if sf is not None:
        scaling = GirolornScaling(sf.number("factor", lo=0.0, lo_open=True), sf.number("original", lo=0.0, lo_open=True),
                                  sf.number("fast", lo=0.0, lo_open=True), sf.number("slow", lo=0.0, lo_open=True))
    base = rot.number("base", lo=0.0, lo_open=True) if dims else 0.0
    if scaling is not None and base == 1.0:
        raise ConfigError(f"{mf.where}: rot.base = 1 turns every pair alike, which rot.scaling cannot tell apart")
    return GirolornMixer(kind, heads, kv_heads, dim, mf.number("scale", lo=0.0, lo_open=True),
                         softcap=mf.number("softcap", default=0.0, lo=0.0), rot_base=base, rot_dims=dims, rot_scaling=scaling)
