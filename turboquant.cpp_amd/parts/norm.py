"""Norms fused with the sum into the residual stream: the RMS norm, and the layer norm at the end of this file.

``out = (v * (1 / sqrt(mean(v^2) + eps))) * weight`` with ``v = x + pending``, everything in float32
(/root/reference/src/engine/tq_ops.c:1373-1410; a plain weight, no ``+1``).

``offset`` c and ``mult`` m, for designs that store their norm weights around zero or scale what a norm lets into the
stream: the norm multiplies by ``m (c + weight)``.  The product is formed once, in float32, when the weights are placed,
so every kernel that takes a norm's weights takes these as they are.
"""
from __future__ import annotations

from ..csrc import ops
from .base import ParamSpec, Part, register_part


@register_part("norm", "rmsnorm")
class RMSNorm(Part):
    graph_safe = True
    def __init__(self, size: int, eps: float, offset: float = 0.0, mult: float = 1.0):
        self.size, self.eps, self.offset, self.mult = size, eps, float(offset), float(mult)
        self.weight = None
        self._folded = False

    def prepare(self, device, act):
        if not self._folded and (self.offset != 0.0 or self.mult != 1.0):
            self.weight = ((self.weight.float() + self.offset) * self.mult).contiguous()
        self._folded = True

    def param_specs(self):
        return {"weight": ParamSpec((self.size,), role="scale")}

    def native(self):
        from ..csrc import host_api
        return host_api.NormDesc(host_api.weight(self.weight), self.eps)

    def over(self, inner) -> ops.NormedDelta:
        """What a part left for the stream, to pass this norm as it is added."""
        return ops.NormedDelta(inner, self.weight, self.eps)

    def forward(self, x, delta, ctx, rows=None, want_act=True, want_f32=False):
        return ops.add_rmsnorm(x, delta, self.weight, self.eps, ctx.act, rows=rows, want_act=want_act,
                               want_f32=want_f32)


@register_part("norm", "layernorm")
class LayerNorm(Part):
    """``out = (v - mean(v)) * (1 / sqrt(mean((v - mean(v))^2) + eps)) * weight + bias`` with ``v = x + pending``, in float32;
    the weights and the bias enter float32 arithmetic only and are kept in it."""
    graph_safe = True

    def __init__(self, size: int, eps: float):
        self.size, self.eps = size, eps
        self.weight = self.bias = None

    def param_specs(self):
        return {"weight": ParamSpec((self.size,), role="scale"), "bias": ParamSpec((self.size,), role="scale")}

    def prepare(self, device, act):
        self.weight, self.bias = self.weight.float().contiguous(), self.bias.float().contiguous()

    def over(self, inner) -> ops.NormedDelta:
        return ops.NormedDelta(inner, self.weight, self.eps, bias=self.bias)

    def forward(self, x, delta, ctx, rows=None, want_act=True, want_f32=False):
        return ops.add_rmsnorm(x, delta, self.weight, self.eps, ctx.act, rows=rows, want_act=want_act, want_f32=want_f32,
                               bias=self.bias)
