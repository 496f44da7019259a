"""What a layer adds to the stream beside its mixer and its feed-forward.

``token_side``: the layer's own small vector of every token of the vocabulary joins the stream, gated by the stream:

    e = columns of the model's second table with a row per token;   y = W_proj (f(W_gate x) * e)
    x <- x + y / sqrt(mean(y^2) + eps) * weight

f one of the activations of ``ops.GATES``.  Float32 on both libraries: the activation, its product with e, the norm.  Three
launches (two for up to 16 tokens): the product, ``token_gate``, the second product, whose partial sums the next norm adds up, norms and adds.
"""
from __future__ import annotations

from ..csrc import ops
from .base import ParamSpec, Part, register_part


@register_part("side", "token_side")
class TokenSide(Part):
    graph_safe = True

    def __init__(self, hidden_size: int, dim: int, first_column: int, eps: float, activation: str = "gelu_tanh"):
        if activation not in ops.GATES:
            raise ValueError(f"unknown activation {activation!r}; known: {', '.join(sorted(ops.GATES))}")
        self.hidden_size, self.dim, self.eps, self.activation = hidden_size, dim, eps, activation
        self.token_columns = (first_column, first_column + dim)      # of the model's table with a row per token
        self.token_rows = None                                       # these columns, set by the model
        self.gate = self.proj = self.norm = None

    def param_specs(self):
        return {"gate": ParamSpec((self.dim, self.hidden_size)), "proj": ParamSpec((self.hidden_size, self.dim)),
                "norm": ParamSpec((self.hidden_size,), role="scale")}

    def prepare(self, device, act):
        self.norm = self.norm.float().contiguous()      # it enters float arithmetic only

    def forward(self, h, ctx) -> ops.NormedDelta:
        g = ops.token_gate_product(h, self.gate, ctx.batch.tokens, self.token_rows, self.activation, ctx.act)
        return ops.NormedDelta(ops.gemm(g, self.proj, ctx.act, partial_sums=True), self.norm, self.eps)
