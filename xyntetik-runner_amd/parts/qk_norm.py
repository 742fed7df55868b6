"""Transforms of an attention's 32-bit queries and keys between their projection and the cache.

``HeadRMSNorm``: every query head and every key head is divided by its root mean square (eps inside
the root) and multiplied by a weight over the head's channels that all heads share (one for the
queries, one for the keys; the plain weight, not one plus it).  With ``temp_every`` the queries of the
token at position p are also multiplied by ``1 + temp_coef ln(floor((p + 1) / temp_every) + 1)``, which
sharpens the attention of tokens far into a sequence.  ``weighted=False``: no weights (and no tensors);
``after_rotation``: the norm comes behind the position encoding.

``RowRMSNorm``: the queries of all heads together are divided by their one root mean square and multiplied by
a weight over the whole projection, and so are the keys.
"""
from __future__ import annotations

from typing import Dict, Optional

import torch

from .base import ParamSpec, QKTransform, register_qk_transform


class HeadRMSNorm(QKTransform):
    def __init__(self, head_dim: int, eps: float, q_name: Optional[str] = "q_norm", k_name: Optional[str] = "k_norm",
                 temp_coef: float = 0.0, temp_every: int = 0, weighted: bool = True, after_rotation: bool = False):
        if temp_every < 0:
            raise ValueError(f"head norm: a query temperature every {temp_every} positions")
        self.head_dim, self.eps = int(head_dim), float(eps)
        self.q_name, self.k_name = q_name, k_name                   # None: that side is not normed
        self.temp_coef, self.temp_every = float(temp_coef), int(temp_every)
        self.weighted, self.after_rotation = bool(weighted), bool(after_rotation)
        if not self.weighted and (q_name is None or k_name is None):
            raise ValueError("head norm: without weights both queries and keys are normed")
        self.w_q = self.w_k = None

    def param_specs(self) -> Dict[str, ParamSpec]:
        out = {}
        for name in (self.q_name, self.k_name):
            if name is not None and self.weighted:
                out[name] = ParamSpec((self.head_dim,), role="vector", init="ones_jitter")
        return out

    def bind(self, tensors, rt) -> None:
        self.rt = rt
        if not self.weighted:
            self.w_q = self.w_k = torch.ones((self.head_dim,), dtype=torch.float32, device=rt.device)
            return
        self.w_q = tensors[self.q_name].float().contiguous() if self.q_name is not None else None
        self.w_k = tensors[self.k_name].float().contiguous() if self.k_name is not None else None

    @property
    def can_head_norm(self) -> bool:
        return self.q_name is not None and self.k_name is not None and not self.temp_every

    def head_norm(self):
        """(query weight, key weight, eps, "before" or "after" the rotation) for the kernel that also rotates and caches the
        heads (``Ops.head_norm_rope_write``), which serves where both sides are normed and queries have no temperature."""
        w = (self.w_q, self.w_k) if self.weighted else (None, None)
        return w + (self.eps, "after" if self.after_rotation else "before")

    def apply(self, ctx, q, k) -> None:
        self.rt.ops.head_rmsnorm_(q, k, self.w_q, self.w_k if k is not None else None, self.eps, ctx.positions,
                                  self.temp_coef, self.temp_every)


class RowRMSNorm(QKTransform):
    def __init__(self, q_size: int, k_size: int, eps: float, q_name: str = "q_norm", k_name: str = "k_norm"):
        self.q_size, self.k_size, self.eps = int(q_size), int(k_size), float(eps)
        self.q_name, self.k_name = q_name, k_name
        self.w_q = self.w_k = None

    def param_specs(self) -> Dict[str, ParamSpec]:
        return {self.q_name: ParamSpec((self.q_size,), role="vector", init="ones_jitter"),
                self.k_name: ParamSpec((self.k_size,), role="vector", init="ones_jitter")}

    def bind(self, tensors, rt) -> None:
        self.rt = rt
        self.w_q = tensors[self.q_name].float().contiguous()
        self.w_k = tensors[self.k_name].float().contiguous()

    def row_norm(self):
        """(query weight, key weight, eps) for the kernel that also rotates and caches the row (``Ops.row_norm_rope_write``)."""
        return self.w_q, self.w_k, self.eps

    def apply(self, ctx, q, k) -> None:
        # a row is one head of its whole width
        ops = self.rt.ops
        ops.head_rmsnorm_(q.flatten(1).unsqueeze(1), None, self.w_q, None, self.eps)
        if k is not None:
            ops.head_rmsnorm_(k.flatten(1).unsqueeze(1), None, self.w_k, None, self.eps)


register_qk_transform("head_rmsnorm", HeadRMSNorm)
register_qk_transform("row_rmsnorm", RowRMSNorm)
