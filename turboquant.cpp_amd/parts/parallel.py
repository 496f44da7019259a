"""Two mixers side by side: ``left_scale * left(h) + right_scale * right(h)``, both reading the same h.

Either may keep keys and values and either a state of fixed size, but each kind of storage one of them at most: the schedule
entry has one cache and one state.  In general what the two return stays unsummed (``ops.Terms``): the next norm adds both into
the stream with their scales in float32.  Mixers that are a product of their input, something behind it and an output product
share more, where both offer it:

* ``input_weight`` / ``take_input_weight`` / ``read_out(proj, ...)``: the two input matrices lie one behind the other and one
  product makes both mixers' projections.
* ``output_weight`` / ``writes_into`` and one side's ``scale_output``: both write their rows side by side into one matrix and one
  product over both output matrices, side by side along k, makes the sum; the ratio of the two scales is then multiplied into
  that side's last step in float32 and the other scale stays with the sum.
* ``kv_write`` / ``takes_kv_write``: in a decode step one side's launch lays out the other's queries, keys and values.
"""
from __future__ import annotations

import math

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
        # made by prepare(): the two mixers' input matrices as one, and their output matrices side by side
        self.in_weight = self.out_weight = None
        self.left_rows = self.left_columns = 0
        self.sum_scale = 1.0        # the factor on the product over both output matrices
        self._prepared = False

    def children(self):
        return {"left": self.left, "right": self.right}

    def cache_need(self):
        own = self.left.cache_need()
        return own if own is not None else self.right.cache_need()

    def state_need(self):
        own = self.left.state_need()
        return own if own is not None else self.right.state_need()

    def prepare(self, device, act):
        if self._prepared:
            return
        self._prepared = True
        sides = (self.left, self.right)
        for part in sides:
            part.prepare(device, act)
        if not all(hasattr(p, "read_out") for p in sides):
            return
        ins, outs = [p.input_weight() for p in sides], [p.output_weight() for p in sides]
        if any(w is None for w in ins + outs) or len({w.dtype for w in ins}) != 1:
            return
        self.in_weight, self.left_rows = torch.cat(ins).contiguous(), ins[0].shape[0]
        self.left.take_input_weight(self.in_weight[:self.left_rows])
        self.right.take_input_weight(self.in_weight[self.left_rows:])
        self._join_outputs(outs, act)

    def _join_outputs(self, outs, act) -> None:
        scales = {"left": self.left_scale, "right": self.right_scale}
        if len({w.dtype for w in outs}) != 1 or any(w.shape[1] % 8 for w in outs) or not all(p.writes_into(act) for p in (self.left, self.right)):
            return
        for side, other in (("right", "left"), ("left", "right")):
            ratio = scales[side] / scales[other] if scales[other] != 0.0 else math.inf
            if hasattr(getattr(self, side), "scale_output") and abs(ratio) < 1e6:
                getattr(self, side).scale_output(ratio)
                self.sum_scale = scales[other]
                self.out_weight, self.left_columns = torch.cat(outs, dim=1).contiguous(), outs[0].shape[1]
                self.left.out_weight = self.right.out_weight = None
                return

    def forward(self, normed, ctx, entry):
        if self.in_weight is None:
            left, right = self.left.forward(normed, ctx, entry), self.right.forward(normed, ctx, entry)
            return ops.Terms.of((self.left_scale, left), (self.right_scale, right))
        proj = ops.gemm(normed, self.in_weight, ctx.act)
        rows, n = None, self.left_columns
        into = {"left": {}, "right": {}}
        if self.out_weight is not None:
            rows = torch.empty((proj.shape[0], self.out_weight.shape[1]), dtype=normed.dtype, device=normed.device)
            into = {"left": {"out": rows[:, :n]}, "right": {"out": rows[:, n:]}}
        own = {"left": proj[:, :self.left_rows], "right": proj[:, self.left_rows:]}
        made = {}
        for writer, keeper in (("right", "left"), ("left", "right")):
            w, k = getattr(self, writer), getattr(self, keeper)
            if not (hasattr(k, "kv_write") and hasattr(w, "takes_kv_write") and w.takes_kv_write(own[writer], ctx)):
                continue
            job = k.kv_write(own[keeper], ctx, entry)
            if job is not None:
                made[writer] = w.read_out(own[writer], ctx, entry, kv_write=job, **into[writer])
                made[keeper] = k.read_out(own[keeper], ctx, entry, q=job.q, **into[keeper])
                break
        else:
            made = {side: getattr(self, side).read_out(own[side], ctx, entry, **into[side]) for side in ("left", "right")}
        if rows is not None:
            return ops.Terms.of((self.sum_scale, ops.gemm(rows, self.out_weight, ctx.act, partial_sums=True)))
        return ops.Terms.of(*((scale, ops.gemm(made[side], getattr(self, side).out_weight, ctx.act, partial_sums=True))
                              for side, scale in (("left", self.left_scale), ("right", self.right_scale))))
