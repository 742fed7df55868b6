"""``PevolornConfig``: the hyper-parameters of a Pevolorn decoder, typed.

config.json of this design is nested: ``vocab``, ``width``, ``norm.eps``, ``postln_alpha`` (what the residual stream counts
in every sum that is normed) and a list ``layers`` whose entries name their mixer (``type``), the mixer's sizes (``mixer``)
and the feed-forward (``mlp``, or null for a layer without one).  Every size and constant that can differ between models is
read here and nowhere else; what the design fixes lives in the parts and in the builder.

====================  =====================================================================
type                  keys of ``mixer``
====================  =====================================================================
latent_attention      heads, dim, rot_dim, vdim, kv_rank, scale, rot.base, rot.dims (absent: rot_dim), kv_from (an
                      earlier layer whose cached rows this one reads; absent: rows of its own)
parallel              left: heads, kv_heads, dim, vdim, scale, softcap (absent: none), rot.base, rot.dims (absent or 0:
                      no rotation); right: heads, vdim, state, groups, conv (taps), norm_groups; left_scale, right_scale
====================  =====================================================================

``mlp``: ``kind`` "moe" with ``expert.ff``, ``router.experts``, ``router.identity`` (absent: none), ``router.top``,
``router.groups.count`` and ``router.groups.keep`` (absent: one group), ``shared.ff`` (absent: no shared expert).
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping, Optional, Tuple

from .base import ConfigError, Fields

MIXERS = ("latent_attention", "parallel")
MLPS = ("moe",)


@dataclass(frozen=True)
class PevolornLatent:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    rot_base: float
    rot_dims: int
    kv_from: Optional[int] = None


@dataclass(frozen=True)
class PevolornAttention:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    softcap: float = 0.0            # 0: none
    rot_base: float = 0.0
    rot_dims: int = 0               # 0: no rotation


@dataclass(frozen=True)
class PevolornState:
    heads: int
    vdim: int
    state: int
    groups: int
    conv: int
    norm_groups: int


@dataclass(frozen=True)
class PevolornMixer:
    kind: str
    latent: Optional[PevolornLatent] = None
    left: Optional[PevolornAttention] = None
    right: Optional[PevolornState] = None
    left_scale: float = 1.0
    right_scale: float = 1.0


@dataclass(frozen=True)
class PevolornMLP:
    ff: int
    experts: int
    identity: int
    top: int
    groups: int = 1
    keep_groups: int = 1
    shared_ff: int = 0              # 0: no shared expert


@dataclass(frozen=True)
class PevolornLayer:
    mixer: PevolornMixer
    mlp: Optional[PevolornMLP]


@dataclass(frozen=True)
class PevolornConfig:
    architecture: str
    vocab: int
    width: int
    eps: float
    alpha: float
    layers: Tuple[PevolornLayer, ...]
    max_position: int

    @staticmethod
    def from_dict(raw: Mapping[str, Any]) -> "PevolornConfig":
        f = Fields(raw)
        norm = f.mapping("norm")
        if norm is None:
            raise ConfigError("config.json: 'norm' is a required object")
        layers = []
        for lf in f.mappings("layers"):
            kind = lf.string("type", choices=MIXERS)
            mf = lf.mapping("mixer")
            if mf is None:
                raise ConfigError(f"{lf.where}: 'mixer' is required")
            layers.append(PevolornLayer(_latent(mf, layers) if kind == "latent_attention" else _parallel(mf), _mlp(lf)))
        return PevolornConfig(
            architecture="Pevolorn", vocab=f.integer("vocab"), width=f.integer("width"), eps=norm.number("eps", lo=0.0),
            alpha=f.number("postln_alpha"), layers=tuple(layers), max_position=f.integer("max_position", default=1 << 20, hi=1 << 30))


def _rotation(mf: Fields, room: int, default: int) -> Tuple[float, int]:
    """(base, rotated channels) of at most ``room``."""
    rot = mf.mapping("rot")
    dims = rot.integer("dims", default=default, lo=0, hi=room) if rot is not None else 0
    if dims % 2:
        raise ConfigError(f"{mf.where}: rot.dims = {dims} must be even")
    return (rot.number("base", lo=0.0, lo_open=True) if dims else 1.0), dims


def _latent(mf: Fields, before) -> PevolornMixer:
    rot_dim, kv_rank = mf.integer("rot_dim", lo=0), mf.integer("kv_rank")
    base, dims = _rotation(mf, rot_dim, rot_dim)
    kv_from = mf.integer("kv_from", default=None, lo=0)
    if kv_from is not None:
        owner = before[kv_from].mixer.latent if kv_from < len(before) else None
        if owner is None or owner.kv_from is not None:
            raise ConfigError(f"{mf.where}: 'kv_from' = {kv_from} names no earlier layer with cached rows of its own")
        if (owner.kv_rank, owner.rot_dim, owner.rot_dims, owner.rot_base) != (kv_rank, rot_dim, dims, base):
            raise ConfigError(f"{mf.where}: kv_rank, rot_dim and rotation differ from those of layer {kv_from}, whose rows it reads")
    return PevolornMixer("latent_attention", latent=PevolornLatent(
        mf.integer("heads"), mf.integer("dim"), rot_dim, mf.integer("vdim"), kv_rank, mf.number("scale"), base, dims, kv_from))


def _parallel(mf: Fields) -> PevolornMixer:
    lf, rf = mf.mapping("left"), mf.mapping("right")
    if lf is None or rf is None:
        raise ConfigError(f"{mf.where}: 'left' and 'right' are required objects")
    heads = lf.integer("heads")
    kv_heads = lf.integer("kv_heads", default=heads, hi=heads)
    if heads % kv_heads:
        raise ConfigError(f"{lf.where}: {heads} heads are not a multiple of kv_heads = {kv_heads}")
    dim = lf.integer("dim")
    base, dims = _rotation(lf, dim, 0)
    left = PevolornAttention(heads, kv_heads, dim, lf.integer("vdim", default=dim), lf.number("scale"),
                             softcap=lf.number("softcap", default=0.0, lo=0.0), rot_base=base, rot_dims=dims)
    heads, vdim, groups = rf.integer("heads"), rf.integer("vdim"), rf.integer("groups", default=1)
    norm_groups = rf.integer("norm_groups", default=1)
    if heads % groups:
        raise ConfigError(f"{rf.where}: {heads} heads are not a multiple of groups = {groups}")
    if (heads * vdim) % norm_groups:
        raise ConfigError(f"{rf.where}: {heads} x {vdim} channels do not form norm_groups = {norm_groups} equal parts")
    right = PevolornState(heads, vdim, rf.integer("state"), groups, rf.integer("conv", lo=1, hi=16), norm_groups)
    return PevolornMixer("parallel", left=left, right=right, left_scale=mf.number("left_scale", default=1.0),
                         right_scale=mf.number("right_scale", default=1.0))


def _mlp(lf: Fields) -> Optional[PevolornMLP]:
    mlp = lf.mapping("mlp")
    if mlp is None:
        return None
    mlp.string("kind", choices=MLPS)
    ef, rf, sf = mlp.mapping("expert"), mlp.mapping("router"), mlp.mapping("shared")
    if ef is None or rf is None:
        raise ConfigError(f"{mlp.where}: 'expert' and 'router' are required objects")
    experts = rf.integer("experts", hi=1 << 10)
    identity = rf.integer("identity", default=0, lo=0, hi=1 << 10)
    n = experts + identity
    top = rf.integer("top", hi=n)
    gf = rf.mapping("groups")
    groups = gf.integer("count", hi=n) if gf is not None else 1
    keep = gf.integer("keep", hi=groups) if gf is not None else 1
    if n % groups:
        raise ConfigError(f"{rf.where}: {n} experts do not form {groups} equal groups")
    if top > keep * (n // groups):
        raise ConfigError(f"{rf.where}: {keep} groups of {n // groups} experts cannot give {top} choices")
    return PevolornMLP(ef.integer("ff"), experts, identity, top, groups, keep, sf.integer("ff") if sf is not None else 0)
