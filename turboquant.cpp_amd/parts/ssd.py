"""Selective state spaces in their dual form (the Mamba-2 mixer).

One product of the layer's input gives z [heads * vdim], x [heads * vdim], B and C [groups, state] and dt [heads].  x, B and C
pass a causal convolution over time (one filter of ``conv_taps`` taps and a bias per channel, zeros before the start, the last
tap is the current token's) and silu; dt <- softplus(dt + dt_bias).  Per head h, which reads group h // (heads / groups), a
state S [state, vdim] that starts at zero and is carried from token to token of a sequence:

    S <- exp(-exp(A_log_h) dt) S + dt B x^T;   y = S^T C + D_h x

The heads side by side are multiplied by silu(z), divided by their root mean square in ``norm_parts`` equal parts (``eps``),
multiplied by a weight per channel, and go through the output product.

The sequence's state is one row of float32 per slot (``StateNeed``): S as [heads, state, vdim], then the convolution's last
taps - 1 inputs of every channel.  Convolution, step sizes, decays, recurrence, gate and norm are float32 on both libraries;
the two products are the activation type's, the first one leaving its result in float32.  Four launches a decode step: the
product, ``ssd_decode``, ``ssd_out`` (which also moves the convolution's state on), the output product.  A prompt step takes
``ssd_prep`` and then ``ssd_chunked`` (from ``chunked_from`` tokens of its longest run on: chunks of 64 tokens on the matrix
cores in float32) or ``ssd_scan`` (token by token) in ``ssd_decode``'s place.
"""
from __future__ import annotations

import torch

from ..csrc import ops
from .base import ParamSpec, Part, StateNeed, register_part


@register_part("mixer", "ssd")
class StateSpaceDual(Part):
    graph_safe = True       # what changes from step to step is read from the batch's device arrays only
    chunked_from = 32       # a step whose longest run has this many tokens takes the chunked form

    def __init__(self, hidden_size: int, num_heads: int, value_dim: int, state_dim: int, groups: int, conv_taps: int,
                 norm_parts: int, eps: float):
        if groups < 1 or num_heads % groups:
            raise ValueError(f"num_heads {num_heads} is not a multiple of groups {groups}")
        if norm_parts < 1 or (num_heads * value_dim) % norm_parts:
            raise ValueError(f"{num_heads} heads of {value_dim} do not fall into {norm_parts} equal parts")
        if not 1 <= state_dim <= 1024:
            raise ValueError(f"a state of {state_dim} channels is beyond the 1,024 that the recurrence's kernel takes")
        if not 1 <= conv_taps <= 64:
            raise ValueError(f"{conv_taps} taps are beyond the 64 that the convolution's kernel takes")
        self.hidden_size, self.eps, self.norm_parts = hidden_size, eps, norm_parts
        self.dims = ops.SsdDims(num_heads, value_dim, state_dim, groups, conv_taps)
        for name in self.param_specs():
            setattr(self, name, None)
        self._prepared = False

    def param_specs(self):
        d, W = self.dims, self.hidden_size
        return {"in_weight": ParamSpec((d.projections, W)),
                "conv": ParamSpec((d.channels, d.taps), role="scale"), "conv_bias": ParamSpec((d.channels,), role="bias"),
                "dt_bias": ParamSpec((d.heads,), role="bias"), "a_log": ParamSpec((d.heads,), role="scale"),
                "skip": ParamSpec((d.heads,), role="scale"), "out_norm": ParamSpec((d.inner,), role="scale"),
                "out_weight": ParamSpec((W, d.inner))}

    def cache_need(self):
        return None

    def state_need(self) -> StateNeed:
        return StateNeed((self.dims.state_floats,), torch.float32)

    def prepare(self, device, act):
        if self._prepared:
            return
        self._prepared = True
        fill = -self.dims.projections % 8      # rows of whole 16-byte pieces, whatever the sizes
        if fill:
            self.in_weight = torch.cat([self.in_weight, self.in_weight.new_zeros((fill, self.hidden_size))]).contiguous()
        for name in ("conv", "conv_bias", "dt_bias", "a_log", "skip"):      # they enter float arithmetic only
            setattr(self, name, getattr(self, name).float().contiguous())

    def forward(self, normed, ctx, entry):
        d, b, state = self.dims, ctx.batch, ctx.state(entry)
        runs = b.runs()
        proj = ops.gemm(normed, self.in_weight, ctx.act)                            # float32 [T, z | x | B | C | dt]
        if runs["decode"]:
            y = ops.ssd_decode(proj, runs, state, self.conv, self.conv_bias, self.dt_bias, self.a_log, self.skip, d, ctx.act)
        else:
            xbc, dt = ops.ssd_prep(proj, b.slot_of_token, state, self.conv, self.conv_bias, self.dt_bias, d, ctx.act)
            form = ops.ssd_chunked if runs["max_new"] >= self.chunked_from and d.state <= 256 else ops.ssd_scan
            y = form(xbc, dt, self.a_log, self.skip, runs, state, d, ctx.act)
        out = ops.ssd_out(y, proj, self.out_norm, self.eps, self.norm_parts, runs, state, d, ctx.act)
        return ops.gemm(out, self.out_weight, ctx.act, partial_sums=True)
