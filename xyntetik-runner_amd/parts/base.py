"""Interfaces of the parts a model is put together from.

A part is built from a ``PartSpec`` (its sizes and constants), names the tensors
it needs, is given them by ``bind`` and is then called by the step function.  No
part knows which architecture it is in; an architecture's builder chooses parts
layer by layer.

Families and what each must offer:

* ``Norm``: ``forward(ctx, x, rows=None) -> h``.  ``x`` is the 32-bit residual
  stream ``[T, E]``; ``h`` is in the compute dtype.  ``rows`` (device int32)
  selects rows of ``x``.  ``fold()`` may return ``(weight, eps)`` if the norm is an
  RMSNorm that the product before it may compute (see below), ``fold_row()`` the same for a
  layer norm too, for kernels that hold whole rows.
* ``PositionEncoding``: ``rotary()`` returns the parameters of a rotation that
  the attention kernels apply themselves, or ``None``; then ``apply(ctx, q, k)``
  is called on the 32-bit queries and keys before they are cached.
* ``QKTransform``: ``apply(ctx, q, k)`` on an attention mixer's 32-bit queries and keys, between
  their projection and the position encoding, in place.
* ``Mixer``: ``kv_spec()`` and ``state_spec()`` say what the cache manager must
  keep for it; ``forward(ctx, cache, h) -> y`` returns ``[T, E]`` in the compute
  dtype; ``forward_add(ctx, cache, h, residual)`` adds it into the 32-bit
  residual stream (the default calls ``forward``; a part with a fused epilogue
  overrides it).
* ``FeedForward``: ``forward(ctx, h) -> y`` and ``forward_add(ctx, h, residual)``.
* ``SequenceFilter``: ``forward(ctx, state, h) -> h'``: what a sublayer reads passes through it on
  its way from the norm; ``state_spec()`` says what it carries from token to token.
* ``Connection``: how a sublayer meets several copies of the residual stream: the weights that make its
  input of them and spread its result over them.
* ``Injection``: ``forward(ctx, x, x0) -> x'``: remakes the 32-bit residual stream from itself and the
  embedding's rows before the run-order entries that are entered through it.
* ``Block``: the arrangement; it names its norms (``norm_names``), may do without a mixer or a
  feed-forward, and ``forward(ctx, cache, x)`` updates ``x`` in place.

``forward_post(..., x, alpha, norm)`` of a mixer or feed-forward is for an arrangement whose residual stream is normed
behind every sum: ``x <- norm(alpha x + result)`` in place, the new rows in the compute dtype come back.

Optional, for fewer kernels when a few tokens are decoded: a mixer or feed-forward
may override ``forward_add_norm(..., residual, norm, defer)``, which adds into the
residual stream and returns ``norm`` of the result, so that its last product can do
both (``Ops.linear_add_rmsnorm``).  With ``defer`` the result may be an
``UnscaledRows`` (the rows still lack the division by their root mean square, which
the next product applies to its own result); a caller sets ``defer`` only if the part
that reads the result has ``takes_unscaled_rows`` set, which says that it hands ``h``
to ``Ops.linear`` or ``Ops.linear_gated`` and reads nothing else of it than its
``shape``, ``dtype`` and ``device``.  A block with ``chained`` set takes the result of
its first norm from the block before it and makes the next block's
(``entry_norm()``); every default does the plain thing.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Callable, Dict, Optional, Tuple

import torch


@dataclass(frozen=True)
class ParamSpec:
    """One tensor a part reads from the checkpoint.

    ``role``: "matrix" tensors are kept in the engine's compute dtype; "vector"
    tensors keep 32 bits if the file stores them so (bfloat16 otherwise, in a
    bfloat16 engine); "int" tensors become int32.
    ``init`` tells the random-weights mode what to write: "normal" (the model's deviation),
    "normal:<s>" (deviation s), "ones", "ones_jitter" (1 + N(0, jitter)), "zeros", or for an integer
    table "choice:<n>" (every row distinct numbers below n).
    An axis of ``shape`` may be -1: a size that no configuration names and the stored tensor decides
    (the part reads it in ``bind``); ``random_shape`` then says what the random-weights mode writes.
    """
    shape: Tuple[int, ...]
    role: str = "matrix"
    init: str = "normal"
    optional: bool = False
    random_shape: Optional[Tuple[int, ...]] = None

    def fits(self, stored: Tuple[int, ...]) -> bool:
        return len(stored) == len(self.shape) and all(a == -1 or a == b for a, b in zip(self.shape, stored))


@dataclass(frozen=True)
class KVSpec:
    """What a mixer with keys and values asks of the cache manager.

    Layers whose specs are equal share a group: one pool of pages and one block
    table per request.  ``window`` = None keeps every key; a number keeps only
    the pages that the last ``window`` positions touch.  ``v_head_dim``: the size of a
    value where it differs from a key's.  ``pooled`` = P: beside its keys and values the
    layer keeps one mean key and one mean value for every block of P positions, in a
    cache of their own whose group has ``stride`` P (one entry for every ``stride``
    positions a request has filled, never given back while the request lives).
    ``keep_first``: with a window, the pages of the first so many positions are kept as well for as
    long as the request lives.
    """
    num_kv_heads: int
    head_dim: int
    window: Optional[int] = None
    v_head_dim: Optional[int] = None
    pooled: Optional[int] = None
    stride: int = 1
    keep_first: int = 0

    @property
    def value_dim(self) -> int:
        return self.v_head_dim if self.v_head_dim is not None else self.head_dim

    def pooled_spec(self) -> Optional["KVSpec"]:
        """The group that holds this spec's block means."""
        if not self.pooled:
            return None
        return KVSpec(self.num_kv_heads, self.head_dim, None, self.v_head_dim, None, int(self.pooled))


@dataclass(frozen=True)
class StateSpec:
    """Fixed-size state per request (one slot per live request).  ``dtype`` None: the engine's
    compute dtype."""
    shape: Tuple[int, ...]
    dtype: Optional[torch.dtype] = torch.float32


class Part:
    """Common base: parameters by relative name."""

    #: False if ``forward`` reads device data on the host (which kernels it launches then
    #: depends on the data): steps of a model with such a part are never recorded as HIP graphs.
    capturable = True

    def param_specs(self) -> Dict[str, ParamSpec]:
        return {}

    def bind(self, tensors: Dict[str, torch.Tensor], rt: "Runtime") -> None:
        """Take the loaded tensors (already on the device, in the dtype their role asks for)."""
        self.rt = rt
        for k, v in tensors.items():
            setattr(self, "w_" + k.replace(".", "_"), v)


class Norm(Part):
    def forward(self, ctx, x: torch.Tensor, rows: Optional[torch.Tensor] = None) -> torch.Tensor:
        raise NotImplementedError

    def fold(self) -> Optional[Tuple[torch.Tensor, float]]:
        """``(weight, eps)`` if this is ``x / sqrt(mean(x^2) + eps) * weight``, which the product
        that writes ``x`` may compute in its own kernel; None for any other norm."""
        return None

    def fold_row(self) -> Optional[Tuple[torch.Tensor, float, bool]]:
        """``(weight, eps, centred)`` of a norm that a kernel which holds whole rows of ``x`` may compute: the one of
        ``fold()``, or with ``centred`` the layer norm ``(x - mean) / sqrt(var + eps) * weight`` with a 32-bit weight and a
        result in the compute dtype; None for any other norm."""
        f = self.fold()
        return (f[0], f[1], False) if f is not None else None


@dataclass(frozen=True)
class RotaryParams:
    """A rotation the attention kernels apply to queries and keys themselves."""
    inv_freq: torch.Tensor      # [rotary_dim / 2] float32, on the device
    rotary_dim: int
    interleaved: bool           # False: pairs (j, j + rotary_dim/2); True: pairs (2j, 2j+1)
    mscale: float = 1.0
    table_key: Any = None       # equal keys promise equal tables (layers then share a step's cosines and sines)


class PositionEncoding(Part):
    def rotary(self) -> Optional[RotaryParams]:
        return None

    def apply(self, ctx, q: torch.Tensor, k: Optional[torch.Tensor]) -> None:
        """Transform 32-bit ``q [T, H, D]`` and ``k [T, Hk, D]`` in place (default: nothing)."""
        return None


class QKTransform(Part):
    """Something an attention mixer does to its 32-bit queries and keys between their projection and
    the position encoding (a norm over every head's channels, say: the reference's optional
    ``attn_q_norm`` / ``attn_k_norm``, src/model.c:2838-2852, src/model.h:229-235).  Its tensors are named
    relative to the mixer's prefix."""

    def apply(self, ctx, q: torch.Tensor, k: Optional[torch.Tensor]) -> None:
        """Transform ``q [T, H, D]`` and ``k [T, Hk, D]`` (None in a layer that computes no keys) in
        place; channels are in the checkpoint's order."""
        raise NotImplementedError


class Mixer(Part):
    def kv_spec(self) -> Optional[KVSpec]:
        return None

    def state_spec(self) -> Optional[StateSpec]:
        """Fixed-size state per request: ``cache.state [slots + 1, *shape]``, request ``b`` of a step
        owning row ``ctx.slots[b]`` (on the device; zero when the request first uses it).  A mixer
        that finds its rows through ``ctx.slots`` can be recorded into a HIP graph, where the rows
        that pad a batch use the last state row, which is nobody's; one that reads the slots on
        the host (``ctx.slots_host``, absent in a recorded step) sets ``capturable = False``.
        A mixer with several tensors of state returns a mapping name -> ``StateSpec`` and finds them
        in ``cache.states`` under ``"mixer." + name``."""
        return None

    def forward(self, ctx, cache, h: torch.Tensor) -> torch.Tensor:
        raise NotImplementedError

    #: True if ``h`` may be an ``UnscaledRows`` (it only goes into ``Ops.linear``)
    takes_unscaled_rows = False

    def forward_add(self, ctx, cache, h: torch.Tensor, residual: torch.Tensor) -> None:
        ctx.ops.add_(residual, self.forward(ctx, cache, h))

    def forward_f32(self, ctx, cache, h: torch.Tensor) -> torch.Tensor:
        """``forward`` as 32-bit rows, for an arrangement that does more with a sublayer's result than add
        it to one residual stream.  A part whose last product can leave 32 bits overrides this; the
        default widens what ``forward`` rounded."""
        return ctx.ops.convert(self.forward(ctx, cache, h).contiguous(), torch.float32)

    def forward_add_norm(self, ctx, cache, h, residual: torch.Tensor, norm: Norm, defer: bool = False):
        """``forward_add``, then ``norm`` of the updated residual stream."""
        self.forward_add(ctx, cache, h, residual)
        return norm.forward(ctx, residual)

    def forward_post(self, ctx, cache, h, x: torch.Tensor, alpha: float, norm: Norm) -> torch.Tensor:
        """``x <- norm(alpha x + forward(h))``; a part whose last kernel can do that overrides it."""
        return post_sum(ctx, self.rt.dtype, x, self.forward_f32(ctx, cache, h), alpha, norm)


def post_sum(ctx, dtype, x: torch.Tensor, y: torch.Tensor, alpha: float, norm: Norm) -> torch.Tensor:
    """``x <- norm(alpha x + y)`` by a kernel of its own; the new rows in ``dtype``."""
    w, eps = norm.fold()
    if w.dtype != torch.float32:                # (a weight kept in bfloat16; once, the norm keeps the copy)
        kept = getattr(norm, "_f32_weight", None)
        if kept is None or kept[0] is not w:
            kept = norm._f32_weight = (w, w.float().contiguous())
        w = kept[1]
    return ctx.ops.post_norm(x, y.contiguous(), alpha, w, eps, dtype)


class SequenceFilter(Part):
    """What a sublayer's input passes through on its way from the norm, with the inputs it carries
    from token to token as state (a short convolution over time, say).  A block arrangement names
    its filters as it names its norms; ``forward(ctx, state, h) -> h'`` in the compute dtype."""

    def state_spec(self) -> Optional[StateSpec]:
        return None

    def forward(self, ctx, state: Optional[torch.Tensor], h: torch.Tensor) -> torch.Tensor:
        raise NotImplementedError


class Connection(Part):
    """How one sublayer meets ``streams`` copies of the residual stream.  A block arrangement names its
    connections as it names its norms."""
    streams = 1


class Injection(Part):
    """What remakes the residual stream from itself and the embedding's rows at the start of a pass over a
    span of layers: ``forward(ctx, x, x0, pass_index) -> x'`` with ``x`` and the result 32-bit ``[T, E]``; ``x0`` is
    what ``prepare(ctx, embedded)`` made of the embedding's rows when the step began; ``pass_index`` counts the
    passes from 0."""

    def prepare(self, ctx, embedded: torch.Tensor):
        return embedded

    def forward(self, ctx, x: torch.Tensor, x0, pass_index: int = 0) -> torch.Tensor:
        raise NotImplementedError


class FeedForward(Part):
    def forward(self, ctx, h: torch.Tensor) -> torch.Tensor:
        raise NotImplementedError

    #: True if ``h`` may be an ``UnscaledRows`` (it only goes into ``Ops.linear`` or ``Ops.linear_gated``)
    takes_unscaled_rows = False

    def forward_add(self, ctx, h: torch.Tensor, residual: torch.Tensor) -> None:
        ctx.ops.add_(residual, self.forward(ctx, h))

    def forward_f32(self, ctx, h: torch.Tensor) -> torch.Tensor:
        """``forward`` as 32-bit rows (see ``Mixer.forward_f32``)."""
        return ctx.ops.convert(self.forward(ctx, h).contiguous(), torch.float32)

    def forward_add_norm(self, ctx, h, residual: torch.Tensor, norm: Norm, defer: bool = False):
        """``forward_add``, then ``norm`` of the updated residual stream."""
        self.forward_add(ctx, h, residual)
        return norm.forward(ctx, residual)

    def forward_post(self, ctx, h, x: torch.Tensor, alpha: float, norm: Norm) -> torch.Tensor:
        """As ``Mixer.forward_post``."""
        return post_sum(ctx, self.rt.dtype, x, self.forward_f32(ctx, h), alpha, norm)


class Block:
    """An arrangement of a layer's parts around the residual stream: a mixer, a feed-forward
    (an arrangement may do without either) and the norms it names in ``norm_names``."""

    #: the norms this arrangement has, by the names a ``LayerSpec`` gives them
    norm_names: Tuple[str, ...] = ()
    #: the sequence filters it has, likewise
    filter_names: Tuple[str, ...] = ()
    #: the connections to several residual streams it has, likewise
    connection_names: Tuple[str, ...] = ()
    needs_mixer = True
    #: True, False, or None for an arrangement that runs with or without a feed-forward
    needs_feed_forward: Optional[bool] = True

    def __init__(self, mixer: Optional[Mixer], feed_forward: Optional[FeedForward], norms: Dict[str, Norm],
                 filters: Optional[Dict[str, "SequenceFilter"]] = None,
                 connections: Optional[Dict[str, "Connection"]] = None):
        kind = type(self).__name__
        if (mixer is None) == self.needs_mixer or (self.needs_feed_forward is not None
                                                   and (feed_forward is None) == self.needs_feed_forward):
            raise ValueError(f"{kind}: this arrangement has {'a' if self.needs_mixer else 'no'} mixer and "
                             f"{'a' if self.needs_feed_forward else 'no'} feed-forward")
        if set(norms) != set(self.norm_names):
            raise ValueError(f"{kind}: this arrangement has the norms {sorted(self.norm_names)}, "
                             f"the layer names {sorted(norms)}")
        filters = dict(filters or {})
        if set(filters) != set(self.filter_names):
            raise ValueError(f"{kind}: this arrangement has the filters {sorted(self.filter_names)}, "
                             f"the layer names {sorted(filters)}")
        connections = dict(connections or {})
        if set(connections) != set(self.connection_names):
            raise ValueError(f"{kind}: this arrangement has the connections {sorted(self.connection_names)}, "
                             f"the layer names {sorted(connections)}")
        self.mixer, self.feed_forward, self.norms, self.filters = mixer, feed_forward, dict(norms), filters
        self.connections = connections

    def parts(self):
        """Every part of the layer by name."""
        out = dict(self.norms)
        out.update(self.filters)
        out.update(self.connections)
        if self.mixer is not None:
            out["mixer"] = self.mixer
        if self.feed_forward is not None:
            out["feed_forward"] = self.feed_forward
        return out

    def state_specs(self) -> Dict[str, StateSpec]:
        """Every tensor of per-request state the layer keeps, by the name it is found under in
        ``cache.states``: the mixer's as "mixer" (or "mixer.<name>" if it has several), a filter's
        under the filter's name."""
        out: Dict[str, StateSpec] = {}
        st = self.mixer.state_spec() if self.mixer is not None else None
        if isinstance(st, StateSpec):
            out["mixer"] = st
        elif st:
            out.update({"mixer." + k: v for k, v in st.items()})
        for name, f in self.filters.items():
            fs = f.state_spec()
            if fs is not None:
                out[name] = fs
        return out

    #: True if ``forward`` also takes ``h`` (the result of this block's first norm, made by the
    #: block before) and ``after`` (the next block's ``entry_norm()``), and returns the next
    #: block's ``h`` or None
    chained = False

    def entry_norm(self) -> Optional[Tuple[Norm, bool]]:
        """(the norm this block applies to the residual stream first, whether what reads its
        result takes ``UnscaledRows``), if the block before may compute it; else None."""
        return None

    def forward(self, ctx, cache, x: torch.Tensor) -> None:
        raise NotImplementedError


@dataclass
class Runtime:
    """What every part needs at run time: the device, the dtypes, and the kernels."""
    device: torch.device
    dtype: torch.dtype              # compute dtype: torch.float32 or torch.bfloat16
    ops: Any                        # xyntetik_runner_amd.csrc.ops.Ops

    @property
    def is_fp32(self) -> bool:
        return self.dtype == torch.float32


# --------------------------------------------------------------------------- registries

_REGISTRIES: Dict[str, Dict[str, Callable[..., Any]]] = {
    "norm": {}, "position": {}, "qk_transform": {}, "mixer": {}, "feed_forward": {}, "block": {}, "embedding": {},
    "head": {}, "filter": {}, "connection": {}, "injection": {},
}


def _register(family: str, kind: str, factory: Callable[..., Any], replace: bool = False) -> None:
    reg = _REGISTRIES[family]
    if kind in reg and not replace:
        raise ValueError(f"{family} part {kind!r} is already registered")
    reg[kind] = factory


def register_norm(kind, factory, replace=False):
    _register("norm", kind, factory, replace)


def register_position(kind, factory, replace=False):
    _register("position", kind, factory, replace)


def register_qk_transform(kind, factory, replace=False):
    _register("qk_transform", kind, factory, replace)


def register_mixer(kind, factory, replace=False):
    _register("mixer", kind, factory, replace)


def register_filter(kind, factory, replace=False):
    _register("filter", kind, factory, replace)


def register_connection(kind, factory, replace=False):
    _register("connection", kind, factory, replace)


def register_injection(kind, factory, replace=False):
    _register("injection", kind, factory, replace)


def register_feed_forward(kind, factory, replace=False):
    _register("feed_forward", kind, factory, replace)


def register_block(kind, factory, replace=False):
    _register("block", kind, factory, replace)


def register_embedding(kind, factory, replace=False):
    _register("embedding", kind, factory, replace)


def register_head(kind, factory, replace=False):
    _register("head", kind, factory, replace)


def unregister(family: str, kind: str) -> None:
    _REGISTRIES[family].pop(kind, None)


def make_part(family: str, spec) -> Any:
    """Build the part a ``PartSpec`` describes."""
    reg = _REGISTRIES[family]
    if spec.kind not in reg:
        raise ValueError(f"no {family} part of kind {spec.kind!r}; registered: {sorted(reg)}")
    return reg[spec.kind](**spec.params)


def make_block(kind: str, mixer, feed_forward, norms, filters=None, connections=None, params=None) -> Block:
    """The arrangement ``kind`` around the given parts (``norms``: name -> norm; ``filters``: name ->
    sequence filter, ``connections``: name -> connection, for an arrangement that has any; ``params``: the
    arrangement's own constants, as keyword arguments)."""
    reg = _REGISTRIES["block"]
    if kind not in reg:
        raise ValueError(f"no block arrangement {kind!r}; registered: {sorted(reg)}")
    if params:
        return reg[kind](mixer, feed_forward, norms, filters or {}, connections or {}, **dict(params))
    if connections:
        return reg[kind](mixer, feed_forward, norms, filters or {}, connections)
    if filters:
        return reg[kind](mixer, feed_forward, norms, filters)
    return reg[kind](mixer, feed_forward, norms)
