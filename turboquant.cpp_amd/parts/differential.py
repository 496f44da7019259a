"""Differential attention over the paged cache: every head attends twice, and what one map takes off the other is left.

A head's q has two maps of ``head_dim`` numbers, and so has a key head's k; both maps look at the same values (``value_dim``
numbers).  q and k are RMS-normed per head and map over head_dim (one weight vector for all query heads and maps, one for
the keys); there is no rotation.  A query at position p is multiplied by ``1 + coef ln(floor((p + 1) / every) + 1)``
(``temperature``: (coef, every), or None).  With a1 and a2 the outputs of the two ordinary softmax attentions (scores times
``scale``, causal) and

    lambda = exp(lq1 . lk1) - exp(lq2 . lk2) + diff              (one number for the layer, of learned vectors [head_dim])

a head's output is ``o = a1 - lambda a2``, divided by its root mean square over value_dim (``eps``, no weight), times
``1 - diff``; the heads side by side are multiplied by sigmoid(W_g x) element by element and go through the output product.
``shares_kv``: the mixer has no key and value matrices and reads the cache of an earlier schedule entry.

Layout: a key head's two maps lie side by side in one row of the cache, each ``D / 2`` wide, D being twice the larger of
head_dim and half the value width rounded up to 16; the value row is D wide.  So both maps' scores come from one pass over one
row of keys, and no value is kept twice.  On the bfloat16 library, for rows of up to 256, the difference, its norm and the gate
are made where the attention normalises its output.  Added rows and columns of the matrices are zeros.  Float32 on both libraries: norms,
temperature, scores, softmax, lambda, the difference's norm and the gate.
"""
from __future__ import annotations

import math

import torch

from ..csrc import ops
from .base import CacheNeed, ParamSpec, Part, register_part


@register_part("mixer", "differential_attention")
class DifferentialAttention(Part):
    graph_safe = True

    def __init__(self, hidden_size: int, num_heads: int, num_kv_heads: int, head_dim: int, value_dim: int, eps: float, diff: float,
                 scale: float | None = None, temperature: tuple[float, float] | None = None, shares_kv: bool = False):
        if num_heads % num_kv_heads:
            raise ValueError(f"num_heads {num_heads} is not a multiple of num_kv_heads {num_kv_heads}")
        if temperature is not None and not temperature[1] > 0:
            raise ValueError(f"the temperature's step must be positive, got {temperature[1]}")
        self.hidden_size, self.num_heads, self.num_kv_heads = hidden_size, num_heads, num_kv_heads
        self.key_dim, self.value_dim, self.eps, self.diff = head_dim, value_dim, eps, float(diff)
        self.half = -(-max(head_dim, -(-value_dim // 2)) // 16) * 16
        self.head_dim = 2 * self.half            # the kernels' width of a row of keys and of a row of values
        self.scale = scale if scale is not None else 1.0 / math.sqrt(head_dim)
        self.temperature, self.shares_kv = temperature, shares_kv
        for name in self.param_specs():
            setattr(self, name, None)
        if shares_kv:
            self.k_weight = self.v_weight = self.k_norm = None
        self.in_weight, self.lam = None, 0.0     # made by prepare()

    def param_specs(self):
        H, G, K, V, W = self.num_heads, self.num_kv_heads, self.key_dim, self.value_dim, self.hidden_size
        specs = {"q_weight": ParamSpec((H * 2 * K, W)), "g_weight": ParamSpec((H * V, W)), "out_weight": ParamSpec((W, H * V)),
                 "q_norm": ParamSpec((K,), role="scale"),
                 **{n: ParamSpec((K,), role="scale") for n in ("lq1", "lk1", "lq2", "lk2")}}
        if not self.shares_kv:
            specs.update({"k_weight": ParamSpec((G * 2 * K, W)), "v_weight": ParamSpec((G * V, W)),
                          "k_norm": ParamSpec((K,), role="scale")})
        return specs

    def cache_need(self) -> CacheNeed:
        return CacheNeed(self.num_kv_heads, self.head_dim)

    def state_need(self):
        return None

    def prepare(self, device, act):
        if self.in_weight is not None:
            return
        H, G, K, V, D, W = self.num_heads, self.num_kv_heads, self.key_dim, self.value_dim, self.head_dim, self.hidden_size

        def laid_out(t, units, width, to):
            """[units * width, ...] -> [units * to, ...], zeros behind each unit's rows."""
            if width == to:
                return t
            out = t.new_zeros((units, to, *t.shape[1:]))
            out[:, :width] = t.view(units, width, *t.shape[1:])
            return out.view(units * to, *t.shape[1:])

        rows = [laid_out(self.q_weight, 2 * H, K, self.half)]
        self.q_norm = laid_out(self.q_norm, 1, K, self.half).contiguous()
        if not self.shares_kv:
            rows += [laid_out(self.k_weight, 2 * G, K, self.half), laid_out(self.v_weight, G, V, D)]
            self.k_norm = laid_out(self.k_norm, 1, K, self.half).contiguous()
        rows.append(laid_out(self.g_weight, H, V, D))
        self.in_weight = torch.cat(rows).contiguous()
        if V != D:
            out = self.out_weight.new_zeros((W, H, D))
            out[:, :, :V] = self.out_weight.view(W, H, V)
            self.out_weight = out.view(W, H * D).contiguous()
        lq1, lk1, lq2, lk2 = (getattr(self, n).double() for n in ("lq1", "lk1", "lq2", "lk2"))
        self.lam = float(torch.exp((lq1 * lk1).sum()) - torch.exp((lq2 * lk2).sum())) + self.diff
        self.q_weight = self.k_weight = self.v_weight = self.g_weight = None

    def forward(self, normed, ctx, entry):
        b, kv = ctx.batch, ctx.kv(entry)
        if kv.owns == self.shares_kv:
            raise ValueError("an attention keeps a cache of its own exactly if it has keys and values of its own")
        H, G, D = self.num_heads, self.num_kv_heads, self.head_dim
        proj = ops.gemm(normed, self.in_weight, ctx.act)                   # float32 [T, q | k | v | gate], or [T, q | gate]
        width = (H + (0 if self.shares_kv else 2 * G)) * D
        # queries: both maps of a head side by side where one pass over the keys serves both, else each map with zeros beside it
        expand = b.is_decode or not ops.diff_attention_fused(ctx.act, D, kv.page_size, kv.page_stride, self.scale)
        q = ops.diff_prep_kv_write(proj[:, :width], b.positions, b.slot_of_token, kv.table, kv.k_pages if kv.owns else None,
                                   kv.v_pages if kv.owns else None, kv.layer_offset, kv.page_size, kv.page_stride, H, G, D, ctx.act,
                                   self.q_norm, self.k_norm, self.eps, self.key_dim, self.temperature, expand=expand,
                                   runs=b.runs())
        o = ops.diff_attention(q, kv.k_pages, kv.v_pages, kv.layer_offset, b.positions, b.slot_of_token, kv.table, kv.page_size,
                               kv.page_stride, H, G, D, self.scale, self.lam, self.eps, self.value_dim, 1.0 - self.diff,
                               proj[:, width:], ctx.act, b.runs())
        return ops.gemm(o, self.out_weight, ctx.act, partial_sums=True)
