"""Two mixers side by side: both read the same input, and their results meet in one sum.

``ParallelMixers``: ``y = a_left f(left(h)) + a_right f(right(h))`` with two numbers and ``f`` either the identity
or, with ``out_norm``, an RMS norm over the model's width with a weight of its own a side (the plain weight, eps
inside the root).  The two sides are mixers of any registered kind, built from their own ``PartSpec``; their
tensors lie under the prefixes ``left.`` and ``right.``.  At most one side keeps paged keys and values (it gets
the layer's pages); the sides' per-request state is kept under the side's name, and each side sees a view of the
layer's cache that holds what is its own (``SideCache``).  The results are 32-bit rows and the sum is made in 32 bits, straight
into the residual stream where the arrangement adds it there.

``joint``: both sides offer their input rows and output columns (``joint_inputs``, ``joint_outputs``) and work from and to
rows they are given (``joint_read_out``).  The pair is then two products: one with the rows of all the projections that read
the input, and one over both sides' rows side by side, each side's times its number before it is rounded, with the output
projections side by side: ``[a_l u_l | a_r u_r] [W_l | W_r]^T = a_l W_l u_l + a_r W_r u_r``.
"""
from __future__ import annotations

from typing import Dict, Optional

import torch

from dataclasses import dataclass, field

from .base import Mixer, ParamSpec, StateSpec, make_part, register_mixer


@dataclass
class SideCache:
    """What one side sees of the layer's cache: the fields of the layer's own record that a mixer reads."""
    group: int
    page_size: int
    owns: bool
    k: Optional[torch.Tensor]
    v: Optional[torch.Tensor]
    state: Optional[torch.Tensor] = None
    states: Dict[str, torch.Tensor] = field(default_factory=dict)

SIDES = ("left", "right")


class ParallelMixers(Mixer):
    def __init__(self, hidden_size: int, left, right, left_scale: float = 1.0, right_scale: float = 1.0,
                 out_norm: bool = False, eps: float = 0.0, left_norm_name: str = "left.out", right_norm_name: str = "right.out",
                 joint: bool = False):
        self.hidden_size = int(hidden_size)
        self.sides = {"left": make_part("mixer", left), "right": make_part("mixer", right)}
        self.scales = {"left": float(left_scale), "right": float(right_scale)}
        self.out_norm, self.eps = bool(out_norm), float(eps)
        self.norm_names = {"left": left_norm_name, "right": right_norm_name}
        self.norm_w: Dict[str, Optional[torch.Tensor]] = {"left": None, "right": None}
        if sum(1 for m in self.sides.values() if m.kv_spec() is not None) > 1:
            raise ValueError("parallel mixers: only one side can keep paged keys and values")
        self.joint = bool(joint)
        if self.joint and (self.out_norm or not all(getattr(m, "joint", False) for m in self.sides.values())):
            raise ValueError("parallel mixers: a joint pair needs two sides that work from rows they are given, and no norm of a side's result")

    @property
    def capturable(self) -> bool:
        return all(m.capturable for m in self.sides.values())

    def kv_spec(self):
        for m in self.sides.values():
            if m.kv_spec() is not None:
                return m.kv_spec()
        return None

    def state_spec(self):
        out: Dict[str, StateSpec] = {}
        for side, m in self.sides.items():
            st = m.state_spec()
            if isinstance(st, StateSpec):
                out[side] = st
            elif st:
                out.update({f"{side}.{name}": spec for name, spec in st.items()})
        return out or None

    def param_specs(self) -> Dict[str, ParamSpec]:
        specs = {}
        for side, m in self.sides.items():
            specs.update({f"{side}.{name}": ps for name, ps in m.param_specs().items()})
            if self.out_norm:
                specs[self.norm_names[side]] = ParamSpec((self.hidden_size,), role="vector", init="ones_jitter")
        return specs

    def bind(self, tensors, rt) -> None:
        self.rt = rt
        if self.joint:
            mine = {side: {name: tensors[f"{side}.{name}"] for name in m.param_specs() if f"{side}.{name}" in tensors}
                    for side, m in self.sides.items()}
            w_in, b_in, w_out, b_out = [], [], [], None
            for side, m in self.sides.items():
                m.joint_bind(mine[side], rt)
                w, b = m.joint_inputs(mine[side])
                w_in.append(w)
                b_in.append(b)
                w, b = m.joint_outputs(mine[side])
                w_out.append(w)
                if b is not None:
                    b_out = self.scales[side] * b + (b_out if b_out is not None else 0.0)
            self.in_rows, self.out_cols = [w.shape[0] for w in w_in], [w.shape[1] for w in w_out]
            self.b_in = None
            if any(b is not None for b in b_in):
                self.b_in = torch.cat([b if b is not None else torch.zeros((w.shape[0],), dtype=torch.float32, device=w.device)
                                       for w, b in zip(w_in, b_in)]).contiguous()
            self.w_in = rt.ops.pack_weight(torch.cat(w_in, dim=0).contiguous())
            self.w_out = rt.ops.pack_weight(torch.cat(w_out, dim=1).contiguous())
            self.b_out = b_out.contiguous() if b_out is not None else None
            return
        for side, m in self.sides.items():
            m.bind({name: tensors[f"{side}.{name}"] for name in m.param_specs() if f"{side}.{name}" in tensors}, rt)
            if self.out_norm:
                self.norm_w[side] = tensors[self.norm_names[side]].float().contiguous()

    def _view(self, cache, side: str):
        """What ``side`` sees of the layer's cache: the pages if it keeps any, and its own state tensors under the
        names it gave them."""
        m = self.sides[side]
        pages = m.kv_spec() is not None
        own, single = {}, cache.states.get(f"mixer.{side}")
        if single is not None:
            own["mixer"] = single
        lead = f"mixer.{side}."
        own.update({"mixer." + name[len(lead):]: t for name, t in cache.states.items() if name.startswith(lead)})
        return SideCache(cache.group if pages else -1, cache.page_size, cache.owns, cache.k if pages else None,
                         cache.v if pages else None, single, own)

    def _joint_rows(self, ctx, cache, h):
        """Both sides' rows side by side, as the joint output product reads them."""
        proj = self.rt.ops.linear(h, self.w_in, bias=self.b_in, out_dtype=torch.float32)
        out = torch.empty((h.shape[0], sum(self.out_cols)), dtype=self.rt.dtype, device=h.device)
        row = col = 0
        for side, n, k in zip(SIDES, self.in_rows, self.out_cols):
            self.sides[side].joint_read_out(ctx, self._view(cache, side), proj[:, row:row + n], out[:, col:col + k], self.scales[side])
            row, col = row + n, col + k
        return out

    def _results(self, ctx, cache, h):
        return [self.sides[side].forward_f32(ctx, self._view(cache, side), h) for side in SIDES]

    def forward_add(self, ctx, cache, h, residual) -> None:
        if self.joint:
            self.rt.ops.linear(self._joint_rows(ctx, cache, h), self.w_out, bias=self.b_out, out=residual, accumulate=True)
            return
        yl, yr = self._results(ctx, cache, h)
        self.rt.ops.pair_combine_(residual, yl.contiguous(), yr.contiguous(), self.scales["left"], self.scales["right"],
                                  self.norm_w["left"], self.norm_w["right"], self.eps)

    def forward_add_norm(self, ctx, cache, h, residual, norm, defer=False):
        """The sides' sum into the residual stream and ``norm`` of the updated rows in the same kernel, where
        ``norm`` is an RMS norm with a weight."""
        fold = norm.fold()
        if fold is None or fold[0] is None:
            return super().forward_add_norm(ctx, cache, h, residual, norm, defer)
        if self.joint:
            return self.rt.ops.linear_add_rmsnorm(self._joint_rows(ctx, cache, h), self.w_out, residual, fold[0], fold[1],
                                                  self.rt.dtype, bias=self.b_out, defer=defer)
        kept = getattr(norm, "_f32_weight", None)
        if kept is None or kept[0] is not fold[0]:
            kept = norm._f32_weight = (fold[0], fold[0].float().contiguous())
        yl, yr = self._results(ctx, cache, h)
        return self.rt.ops.pair_combine_(residual, yl.contiguous(), yr.contiguous(), self.scales["left"], self.scales["right"],
                                         self.norm_w["left"], self.norm_w["right"], self.eps,
                                         then_norm=(kept[1], fold[1]), out_dtype=self.rt.dtype)

    def forward_post(self, ctx, cache, h, x, alpha, norm):
        w, eps = norm.fold()
        if not self.joint or w.dtype != torch.float32:
            return super().forward_post(ctx, cache, h, x, alpha, norm)
        return self.rt.ops.linear_post_norm(self._joint_rows(ctx, cache, h), self.w_out, x, alpha, w, eps, self.rt.dtype, bias=self.b_out)

    def forward_f32(self, ctx, cache, h):
        if self.joint:
            return self.rt.ops.linear(self._joint_rows(ctx, cache, h), self.w_out, bias=self.b_out, out_dtype=torch.float32)
        yl, yr = self._results(ctx, cache, h)
        out = torch.empty_like(yl)
        self.rt.ops.fill_rows_(out.view(1, -1), None, 1, 0)
        self.rt.ops.pair_combine_(out, yl.contiguous(), yr.contiguous(), self.scales["left"], self.scales["right"],
                                  self.norm_w["left"], self.norm_w["right"], self.eps)
        return out

    def forward(self, ctx, cache, h):
        return self.rt.ops.convert(self.forward_f32(ctx, cache, h), self.rt.dtype)


register_mixer("parallel_mixers", ParallelMixers)
