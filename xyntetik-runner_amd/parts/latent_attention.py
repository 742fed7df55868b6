"""Attention whose keys and values are made from one small latent a token.

Per token: ``c_q = rmsnorm(W_dq h)``, ``q = W_uq c_q`` (H heads, each ``D`` unrotated channels followed
by ``R`` rotated ones); ``W_dkv h`` has ``C + R`` rows: the first ``C``, RMS-normed, are the latent ``c``, the
last ``R`` are one key part that all heads share.  The rotation turns the first ``rot_dims`` of the ``R``
channels (of every query head and of the shared key part) in pairs ``(2i, 2i + 1)`` by
``position x base^(-2i / rot_dims)``.  A head's key is ``[W_uk c | shared part]``, its value ``W_uv c``; the
score is ``(q . k) * scale``; a token sees itself and the ``window - 1`` before it (all, without a
window); softmax in 32-bit; ``W_o`` on the concatenated heads.

Options: ``q_rank`` None: the queries are one projection of the input (``q_name``), without a latent of their own;
``pairs`` "halves": the rotation turns channel i with channel ``i + rot_dims / 2`` (else "neighbours"); ``gate_name``: a
projection ``[H, E]`` of the mixer's input whose sigmoid multiplies every head's output; ``kv_shared``: the layer has no
``W_dkv`` and reads another layer's cached rows with its own queries, ``W_uk`` and ``W_uv``.  Without a query latent
everything that reads the mixer's input is one product.

Only ``[c | shared part]`` is cached, one row a token, as the one key/value head of a paged cache
that all query heads share.  The queries are brought into the latent's space instead of the keys
out of it: ``q_abs = W_uk_h^T q_unrotated`` gives ``q_abs . c = q_unrotated . (W_uk_h c)``; attention then
runs over the cached rows with value ``c``, and ``W_uv_h`` is applied to its output
(``W_uv_h sum_j p_j c_j = sum_j p_j W_uv_h c_j``).  The value pages hold the row transposed, as
every attention cache here does; where the matrix-core attention serves (bfloat16, a row length
that is a multiple of 16 up to 256) and ``C`` is no multiple of 16 they hold all ``C + R`` channels, and the
output's last ``R`` channels are not read.
"""
from __future__ import annotations

from typing import Dict, Optional

import torch

from .base import KVSpec, Mixer, ParamSpec, register_mixer
from .rotary import rotary_inv_freq

MAX_ROW = 1024      # the 32-bit attention kernel keeps a cached row in registers up to this size (the matrix-core kernels: 256)


class LatentAttention(Mixer):
    def __init__(self, hidden_size: int, num_heads: int, head_dim: int, rot_dim: int, v_head_dim: int, q_rank: Optional[int],
                 kv_rank: int, scale: float, eps: float, rot_dims: Optional[int] = None, rot_base: float = 10000.0,
                 window: Optional[int] = None, dq_name: str = "dq", dq_norm_name: str = "dq.norm", uq_name: str = "uq",
                 dkv_name: str = "dkv", dkv_norm_name: str = "dkv.norm", uk_name: str = "uk", uv_name: str = "uv",
                 o_name: str = "o", q_name: str = "q", pairs: str = "neighbours", gate_name: Optional[str] = None,
                 kv_shared: bool = False):
        if pairs not in ("neighbours", "halves"):
            raise ValueError(f"latent attention: the rotation pairs {pairs!r} (neighbours or halves)")
        self.halves, self.gate_name, self.kv_shared = pairs == "halves", gate_name, bool(kv_shared)
        self.hidden_size, self.num_heads = int(hidden_size), int(num_heads)
        self.head_dim, self.rot_dim, self.v_head_dim = int(head_dim), int(rot_dim), int(v_head_dim)
        self.q_rank, self.kv_rank = int(q_rank) if q_rank is not None else None, int(kv_rank)
        if self.kv_shared and self.q_rank is not None:
            raise ValueError("latent attention: a layer that reads another layer's rows is built without a query latent")
        self.row = self.kv_rank + self.rot_dim          # what is cached a token
        if not (1 <= self.row <= MAX_ROW):
            raise ValueError(f"latent attention: a cached row of {self.kv_rank} + {self.rot_dim} channels is outside what the "
                             f"attention kernels take (1 to {MAX_ROW})")
        self.rot_dims = self.rot_dim if rot_dims is None else int(rot_dims)
        if self.rot_dims % 2 or not (0 <= self.rot_dims <= self.rot_dim):
            raise ValueError(f"latent attention: {self.rot_dims} rotated channels must be even and at most {self.rot_dim}")
        if window is not None and window < 1:
            raise ValueError(f"attention window {window} must be at least 1")
        self.rot_base, self.scale, self.eps = float(rot_base), float(scale), float(eps)
        self.window = int(window) if window is not None else None
        self.names = dict(dq=dq_name, dq_norm=dq_norm_name, uq=uq_name, dkv=dkv_name, dkv_norm=dkv_norm_name, uk=uk_name,
                          uv=uv_name, o=o_name, q=q_name, g=gate_name)
        self.rt = None

    def _matrix_cores(self) -> bool:
        """Whether the matrix-core attention kernels take this layer's cached rows."""
        return self.rt is not None and self.rt.ops.attention_on_matrix_cores(self.rt.dtype, self.row, self._value_rows(True))

    def _value_rows(self, matrix_cores: bool) -> int:
        """Channels of a row that the value pages hold."""
        return self.row if matrix_cores and self.kv_rank % 16 else self.kv_rank

    def kv_spec(self) -> Optional[KVSpec]:
        values = self._value_rows(self._matrix_cores())
        return KVSpec(1, self.row, self.window, values if values != self.row else None)

    def param_specs(self) -> Dict[str, ParamSpec]:
        E, H, D, R, Dv, n = self.hidden_size, self.num_heads, self.head_dim, self.rot_dim, self.v_head_dim, self.names
        specs = {n["uk"]: ParamSpec((H * D, self.kv_rank)), n["uv"]: ParamSpec((H * Dv, self.kv_rank)),
                 n["o"]: ParamSpec((E, H * Dv))}
        if self.q_rank is None:
            specs[n["q"]] = ParamSpec((H * (D + R), E))
        else:
            specs.update({n["dq"]: ParamSpec((self.q_rank, E)), n["uq"]: ParamSpec((H * (D + R), self.q_rank)),
                          n["dq_norm"]: ParamSpec((self.q_rank,), role="vector", init="ones_jitter")})
        if not self.kv_shared:
            specs.update({n["dkv"]: ParamSpec((self.row, E)),
                          n["dkv_norm"]: ParamSpec((self.kv_rank,), role="vector", init="ones_jitter")})
        if self.gate_name is not None:
            specs[n["g"]] = ParamSpec((H, E), init="normal:0.1")
        return specs

    def bind(self, tensors, rt) -> None:
        self.rt = rt
        ops, n = rt.ops, self.names
        H, D, R, Dv, C = self.num_heads, self.head_dim, self.rot_dim, self.v_head_dim, self.kv_rank
        # everything that reads the input in one product: queries (or their latent), the cached row, the gate
        inputs = [n["q"] if self.q_rank is None else n["dq"]] + ([] if self.kv_shared else [n["dkv"]]) + ([n["g"]] if self.gate_name else [])
        self.w_down = ops.pack_weight(torch.cat([tensors[name] for name in inputs], dim=0).contiguous())
        if self.q_rank is not None:
            self.w_dq_norm = tensors[n["dq_norm"]]
            self.w_uq = ops.pack_weight(tensors[n["uq"]])
        self.w_c_norm = tensors[n["dkv_norm"]].float().contiguous() if not self.kv_shared else None
        # Per head: W_uk_h^T [C, D] takes the unrotated query channels into the latent's space,
        # W_uv_h [Dv, C] the attention's output out of it; each is one launch over all heads.
        self.w_absorb = tensors[n["uk"]].view(H, D, C).transpose(1, 2).contiguous()      # [H, C, D]
        self.w_expand = tensors[n["uv"]].view(H, Dv, C).contiguous()                     # [H, Dv, C]
        self.w_out = ops.pack_weight(tensors[n["o"]])
        self.inv_freq = (rotary_inv_freq(self.rot_dims, self.rot_base).to(torch.float32).to(rt.device)
                         if self.rot_dims else None)

    def _attend(self, ctx, cache, h):
        ops, rt = self.rt.ops, self.rt
        H, D, R, Dv, C, DK = self.num_heads, self.head_dim, self.rot_dim, self.v_head_dim, self.kv_rank, self.row
        T = h.shape[0]
        if cache.owns == self.kv_shared:
            raise ValueError("latent attention: a layer stores its own latents, or has no projection of them and reads another's")
        down = ops.linear(h, self.w_down, out_dtype=torch.float32)         # [T, (q_rank or H * (D + R)) + (C + R) + gate]
        at = self.q_rank if self.q_rank is not None else H * (D + R)
        if self.q_rank is not None:
            cq = ops.rmsnorm(down[:, :at], self.w_dq_norm, self.eps, rt.dtype)
            q_in = ops.linear(cq, self.w_uq, out_dtype=torch.float32)                    # [T, H * (D + R)]
        else:
            q_in = down[:, :at]
        kv_in = down[:, at:at + DK] if not self.kv_shared else None
        gate = down[:, down.shape[1] - H:] if self.gate_name is not None else None
        q = torch.empty((T, H * DK), dtype=rt.dtype, device=h.device)
        qn = ops.latent_prepare(q_in, kv_in, self.w_c_norm, self.eps, q, cache.k, cache.v, ctx, cache.group,
                                self.inv_freq, H, D, R, C, self.rot_dims, cache.page_size, halves=self.halves)
        ops.heads_linear(qn, self.w_absorb, q, H, D, DK)
        Dvc = cache.v.shape[2]
        # (a gate multiplies a whole head: on the attention's output or, as here, on what W_uv makes it of)
        if self._matrix_cores():
            o = ops.attention(q, cache.k, cache.v, ctx, cache.group, H, 1, DK, cache.page_size, self.scale, self.window,
                              v_head_dim=Dvc, gate=gate)
        else:
            o = ops.attention_pooled(q, cache.k, cache.v, None, None, ctx, cache.group, None, H, 1, DK, Dvc,
                                     cache.page_size, self.scale, self.window or (1 << 30), 0, matrix_cores=False)
            if gate is not None:
                ops.head_gate_(o, gate, H, Dvc)
        ov = torch.empty((T, H * Dv), dtype=rt.dtype, device=h.device)
        ops.heads_linear(o, self.w_expand, ov, H, Dvc, Dv)
        return ov

    def forward(self, ctx, cache, h):
        return self.rt.ops.linear(self._attend(ctx, cache, h), self.w_out)

    def forward_f32(self, ctx, cache, h):
        return self.rt.ops.linear(self._attend(ctx, cache, h), self.w_out, out_dtype=torch.float32)

    def forward_add(self, ctx, cache, h, residual) -> None:
        self.rt.ops.linear(self._attend(ctx, cache, h), self.w_out, out=residual, accumulate=True)


    def forward_post(self, ctx, cache, h, x, alpha, norm):
        w, eps = norm.fold()
        if w.dtype != torch.float32:
            return super().forward_post(ctx, cache, h, x, alpha, norm)
        return self.rt.ops.linear_post_norm(self._attend(ctx, cache, h), self.w_out, x, alpha, w, eps, self.rt.dtype)


register_mixer("latent_attention", LatentAttention)
