"""A matrix memory with exponential gates (the mLSTM cell).

q = W_q x / sqrt(dim) and k = W_k x ([heads, dim]), v = W_v x ([heads, vdim]).  Per head, the logarithms of two gates,
``i = cap tanh((W_i x + b_i) / cap)`` and ``f = logsigmoid(cap tanh((W_f x + b_f) / cap))``, a state S [dim, vdim], a normaliser
n [dim] and a running maximum m, all zero when a sequence starts and carried from token to token:

    m' = max(f + m, i);  S <- e^(f + m - m') S + e^(i - m') k v^T;  n <- e^(f + m - m') n + e^(i - m') k
    o = S^T q / (max(|n . q|, e^(-m')) + 1e-6)

Each head's o is divided by its root mean square over vdim (``eps``), multiplied by a weight per channel of all heads and by
sigmoid(W_g x), and the heads go through the output product.

The sequence's state is one row of float32 per slot (``StateNeed``): S, n and m.  Gates, recurrence, norm and gate are
float32 on both libraries (sums of gate logarithms in double); the two products are the activation type's, the first one
leaving its result in float32.  Three launches a decode step: the product of all projections (one matrix), ``mm_decode``, the
output product.  A prompt step takes ``mm_chunked`` (from ``chunked_from`` tokens of its longest run on: chunks of 64 tokens on
the matrix cores in float32) or ``mm_scan`` (token by token), and ``mm_out`` behind either.
"""
from __future__ import annotations

import torch

from ..csrc import ops
from .base import ParamSpec, Part, StateNeed, register_part


@register_part("mixer", "matrix_memory")
class MatrixMemory(Part):
    graph_safe = True       # what changes from step to step is read from the batch's device arrays only
    chunked_from = 32       # a step whose longest run has this many tokens takes the chunked form

    def __init__(self, hidden_size: int, num_heads: int, head_dim: int, value_dim: int, gate_cap: float, eps: float):
        if not gate_cap > 0:
            raise ValueError(f"gate_cap must be positive, got {gate_cap}")
        if not 1 <= head_dim <= 1024:
            raise ValueError(f"a key width of {head_dim} is beyond the 1,024 that the recurrence's kernel takes")
        self.hidden_size, self.eps = hidden_size, eps
        self.dims = ops.MemoryDims(num_heads, head_dim, value_dim, float(gate_cap))
        for name in self.param_specs():
            setattr(self, name, None)
        self.in_weight = self.gate_bias = None     # made by prepare()

    def param_specs(self):
        d, W = self.dims, self.hidden_size
        qk, v = d.heads * d.dim, d.heads * d.vdim
        return {"q_weight": ParamSpec((qk, W)), "k_weight": ParamSpec((qk, W)), "v_weight": ParamSpec((v, W)),
                "g_weight": ParamSpec((v, W)), "i_weight": ParamSpec((d.heads, W)), "f_weight": ParamSpec((d.heads, W)),
                "i_bias": ParamSpec((d.heads,), role="bias"), "f_bias": ParamSpec((d.heads,), role="bias"),
                "out_norm": ParamSpec((v,), role="scale"), "out_weight": ParamSpec((W, v))}

    def cache_need(self):
        return None

    def state_need(self) -> StateNeed:
        return StateNeed((self.dims.state_floats,), torch.float32)

    def prepare(self, device, act):
        if self.in_weight is not None:
            return
        rows = [self.q_weight, self.k_weight, self.v_weight, self.g_weight, self.i_weight, self.f_weight]
        fill = -self.dims.projections % 8      # rows of whole 16-byte pieces, whatever the number of heads
        if fill:
            rows.append(self.q_weight.new_zeros((fill, self.hidden_size)))
        self.in_weight = torch.cat(rows).contiguous()
        self.gate_bias = torch.cat([self.i_bias.float(), self.f_bias.float()]).contiguous()     # it enters float arithmetic only
        for name in ("q_weight", "k_weight", "v_weight", "g_weight", "i_weight", "f_weight", "i_bias", "f_bias"):
            setattr(self, name, None)

    # the product of the layer's input, for an arrangement that makes it together with another mixer's (parts/parallel.py)
    def input_weight(self) -> torch.Tensor:
        return self.in_weight

    def take_input_weight(self, weight: torch.Tensor) -> None:
        self.in_weight = weight

    def output_weight(self) -> torch.Tensor:
        return self.out_weight

    def writes_into(self, act: str) -> bool:
        return True

    def scale_output(self, factor: float) -> None:
        """Multiplies what the mixer puts out: a factor on the weights of its last norm, in float32."""
        self.out_norm = (self.out_norm.float() * factor).contiguous()

    def takes_kv_write(self, proj, ctx) -> bool:
        """Whether this step's ``read_out`` can lay out another mixer's keys and values in its launch."""
        return ctx.batch.is_decode and ops.mm_decode_fits(proj, self.dims)

    def read_out(self, proj, ctx, entry, out=None, kv_write=None):
        """What follows the product of the layer's input, up to the output product: activation rows [T, heads * vdim]."""
        d, b, state = self.dims, ctx.batch, ctx.state(entry)
        runs = b.runs()
        if runs["decode"] and ops.mm_decode_fits(proj, d):
            return ops.mm_decode(proj, self.gate_bias, runs, state, self.out_norm, self.eps, d, ctx.act, out=out, kv_write=kv_write)
        at = 2 * d.heads * d.dim + d.heads * d.vdim
        gate = proj[:, at:at + d.heads * d.vdim]
        if runs["max_new"] >= self.chunked_from and d.dim <= 256:
            num, den = ops.mm_chunked(proj, self.gate_bias, runs, state, d, ctx.act)
            return ops.mm_out(num, den, gate, self.out_norm, self.eps, d, ctx.act, out=out)
        num, den, mrow = ops.mm_scan(proj, self.gate_bias, runs, state, d, ctx.act)
        return ops.mm_out(num, den, gate, self.out_norm, self.eps, d, ctx.act, mrow=mrow, slot_of_token=b.slot_of_token,
                          state=state, out=out)

    def forward(self, normed, ctx, entry):
        out = self.read_out(ops.gemm(normed, self.in_weight, ctx.act), ctx, entry)
        return ops.gemm(out, self.out_weight, ctx.act, partial_sums=True)
