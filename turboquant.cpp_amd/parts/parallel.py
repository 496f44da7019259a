"""Two mixers side by side: ``left_scale * left(h) + right_scale * right(h)``, both reading the same h.

Either may keep keys and values and either a state of fixed size, but each kind of storage one of them at most: the schedule
entry has one cache and one state.  What the two return stays unsummed (``ops.Terms``): the next norm adds both into the stream
with their scales in float32.  Where both make one product of their input first, the two matrices lie one behind the other and
one product makes both (``input_weight`` / ``take_input_weight`` / ``forward_projected``; ``projects_alone`` says for which steps
a mixer would rather make its own, as an attention does that stores its keys and values in the product's launch).
"""
from __future__ import annotations

import torch

from ..config.plan import PartSpec
from ..csrc import ops
from .base import Part, build_part, register_part


@register_part("mixer", "parallel")
class ParallelMixer(Part):
    graph_safe = True

    def __init__(self, left, right, left_scale: float = 1.0, right_scale: float = 1.0):
        self.left, self.right = (build_part("mixer", p) if isinstance(p, PartSpec) else p for p in (left, right))
        if self.left.cache_need() is not None and self.right.cache_need() is not None:
            raise ValueError("one of two mixers side by side may keep keys and values, not both")
        if self.left.state_need() is not None and self.right.state_need() is not None:
            raise ValueError("one of two mixers side by side may keep a state per sequence, not both")
        self.left_scale, self.right_scale = float(left_scale), float(right_scale)
        self.in_weight = None       # made by prepare(): both mixers' input matrices, if both have one
        self.left_rows = 0

    def children(self):
        return {"left": self.left, "right": self.right}

    def cache_need(self):
        own = self.left.cache_need()
        return own if own is not None else self.right.cache_need()

    def state_need(self):
        own = self.left.state_need()
        return own if own is not None else self.right.state_need()

    def prepare(self, device, act):
        if self.in_weight is not None:
            return
        for part in (self.left, self.right):
            part.prepare(device, act)
        ws = [part.input_weight() if hasattr(part, "input_weight") else None for part in (self.left, self.right)]
        if any(w is None for w in ws) or ws[0].dtype != ws[1].dtype:
            return
        self.in_weight, self.left_rows = torch.cat(ws).contiguous(), ws[0].shape[0]
        self.left.take_input_weight(self.in_weight[:self.left_rows])
        self.right.take_input_weight(self.in_weight[self.left_rows:])

    def forward(self, normed, ctx, entry):
        T = normed.shape[0]
        if self.in_weight is None or any(p.projects_alone(T, normed) for p in (self.left, self.right)):
            left, right = self.left.forward(normed, ctx, entry), self.right.forward(normed, ctx, entry)
        else:
            proj = ops.gemm(normed, self.in_weight, ctx.act)
            left = self.left.forward_projected(proj[:, :self.left_rows], ctx, entry)
            right = self.right.forward_projected(proj[:, self.left_rows:], ctx, entry)
        return ops.Terms.of((self.left_scale, left), (self.right_scale, right))
