"""Feed-forward parts: a dense gated one, a dense one with an activation and no gate, and a sparse one with routed
experts and a shared expert.

Dense (/root/reference/src/engine/tq_transformer.c:2707-2824): ``down(silu(gate x) * (up x))``, no biases; the
gate's activation is an argument (``silu``, ``gelu_tanh`` as /root/reference/src/engine/tq_ops.c:1482-1484, ``relu2``)
that the products' epilogues take.  ``pair_limit`` L: ``down(f(min(gate x, L)) * (clamp(up x, -L, L) + 1))``.
Sparse (/root/reference/src/engine/tq_moe.c:600-1059): router logits in float32, top-k with the highest index
winning ties, weights from a softmax; every chosen expert is the dense formula with its own matrices, summed
with its weight in the order chosen; the shared expert, scaled by ``sigmoid(x . shared_scale)``, is added
last.  ``renormalize`` false keeps the softmax over all experts un-normalised for the chosen ones; true is
the reference's softmax over the chosen logits.  ``router_bias``: a number per expert is added to its logit before the
choice.  ``pair_limit`` L: an expert is ``down(f(min(gate x, L)) * (clamp(up x, -L, L) + 1))``.  ``groups`` (count, keep): the experts form ``count`` equal groups of
neighbours, a group's score is the largest score in it (``pair_groups``: the sum of its two largest), and only experts of
the ``keep`` best groups can be chosen.  ``sigmoid_scores``: an expert's score is the sigmoid of its logit, the choice is by
score, and the weights are the chosen scores over (their sum + 1e-20), times ``weight_scale`` (which the softmax over the
chosen logits may have too).  ``shared_limit`` L: the
shared expert's pair is clamped as ``pair_limit`` clamps the experts' (the two may differ).
``gated`` false: an expert is ``down(f(up x))``, two matrices and no gate.  ``score_correction``: the softmax runs over all
of the router's rows, the choice is by score plus a learned number per row, and the weights are the scores themselves,
not renormalised.  ``identity`` n (with ``score_correction``): the router has n more rows than there are experts with
matrices; a token that chooses one of them gets its own input back, times the weight.
"""
from __future__ import annotations

import torch

from ..csrc import ops
from .base import ParamSpec, Part, register_part


SIDE_STREAM_FROM = 320      # tokens of an eager step from which the shared expert goes to a second stream
# The same border where the step executor issues the launches: forking and joining cost it two events a layer, not the
# 2.6 ms a step that they cost a step issued from Python, so the second stream pays from far fewer tokens on (measured
# on 24 layers, one prompt, with and without it: 48 tokens 4.32 against 4.36 ms, 96 tokens 5.27 against 5.73, 192 tokens
# 5.39 against 6.44, 320 tokens 6.31 against 7.71, 512 tokens 8.06 against 9.06; 24 tokens 3.59 against 3.46).
SIDE_STREAM_FROM_IN_EXECUTOR = 64


@register_part("ffn", "dense_swiglu")
class DenseSwiGLU(Part):
    graph_safe = True
    wants_f32 = False

    def __init__(self, hidden_size: int, inner_size: int, activation: str = "silu", pair_limit: float | None = None):
        if activation not in ops.GATES:
            raise ValueError(f"unknown activation {activation!r}; known: {', '.join(sorted(ops.GATES))}")
        if pair_limit is not None and not pair_limit > 0:
            raise ValueError(f"pair_limit must be positive, got {pair_limit}")
        self.hidden_size, self.inner_size, self.activation, self.pair_limit = hidden_size, inner_size, activation, pair_limit
        self.gate = self.up = self.down = None

    def param_specs(self):
        return {"gate": ParamSpec((self.inner_size, self.hidden_size)),
                "up": ParamSpec((self.inner_size, self.hidden_size)),
                "down": ParamSpec((self.hidden_size, self.inner_size))}

    def prepare(self, device, act):
        # gate and up side by side: a long prompt's pair may then go out as one product over both
        self.gate, self.up = ops.side_by_side(self.gate, self.up)

    def native(self):
        from ..csrc import host_api
        if self.pair_limit is not None:
            return None                  # the executor's pairs have no limit
        return host_api.DenseFfnDesc(self.hidden_size, self.inner_size, ops.GATES[self.activation], host_api.weight(self.gate),
                                     host_api.weight(self.up), host_api.weight(self.down))

    def forward(self, normed, normed32, ctx):
        h = ops.gemm(normed, self.gate, ctx.act, w2=self.up, out_act=True, activation=self.activation,
                     **({} if self.pair_limit is None else {"pair_limit": self.pair_limit}))
        return ops.gemm(h, self.down, ctx.act, partial_sums=True)


@register_part("ffn", "dense_act")
class DenseActivated(Part):
    """Two matrices and an activation between them, no gate and no biases: ``down(f(up x))``, f one of the activations
    of ``ops.GATES`` (``relu2``: the square of relu)."""
    graph_safe = True
    wants_f32 = False

    def __init__(self, hidden_size: int, inner_size: int, activation: str = "relu2"):
        if activation not in ops.GATES:
            raise ValueError(f"unknown activation {activation!r}; known: {', '.join(sorted(ops.GATES))}")
        self.hidden_size, self.inner_size, self.activation = hidden_size, inner_size, activation
        self.up = self.down = None

    def param_specs(self):
        return {"up": ParamSpec((self.inner_size, self.hidden_size)),
                "down": ParamSpec((self.hidden_size, self.inner_size))}

    def forward(self, normed, normed32, ctx):
        h = ops.gemm(normed, self.up, ctx.act, activation=self.activation, act_alone=True)
        return ops.gemm(h, self.down, ctx.act, partial_sums=True)


@register_part("ffn", "moe_swiglu")
class SparseMoE(Part):
    graph_safe = True
    wants_f32 = True    # the router reads the normalised activations in float32

    def __init__(self, hidden_size: int, num_experts: int, top_k: int, expert_size: int, shared_size: int = 0,
                 shared_gated: bool = True, renormalize: bool = False, activation: str = "silu",
                 groups: tuple[int, int] | None = None, router_bias: bool = False, pair_limit: float | None = None,
                 gated: bool = True, score_correction: bool = False, identity: int = 0, sigmoid_scores: bool = False,
                 weight_scale: float = 1.0, pair_groups: bool = False, shared_limit: float | None = None):
        if sigmoid_scores and (score_correction or not renormalize or not gated):
            raise ValueError("sigmoid scores are renormalised over the chosen experts, which are gated pairs, and come without a correction")
        if not sigmoid_scores and pair_groups:
            raise ValueError("groups by their two best scores go with sigmoid scores")
        if weight_scale != 1.0 and (not renormalize or score_correction or not gated):
            raise ValueError("a weight scale goes with weights renormalised over the chosen experts, which are gated pairs")
        if shared_limit is not None and not (shared_size > 0 and shared_limit > 0):
            raise ValueError(f"shared_limit is for a shared expert and positive, got {shared_limit}")
        self.sigmoid_scores, self.weight_scale, self.pair_groups = sigmoid_scores, float(weight_scale), bool(pair_groups)
        self.shared_limit = shared_limit
        if score_correction and (renormalize or groups is not None or router_bias or shared_size > 0):
            raise ValueError("a choice by corrected scores goes with plain softmax weights over all rows, without groups, "
                             "a router bias or a shared expert")
        if identity < 0 or (identity and not score_correction):
            raise ValueError("experts that are the identity come with a choice by corrected scores")
        if not gated and pair_limit is not None:
            raise ValueError("a limit is for gated pairs")
        self.gated, self.score_correction, self.identity, self.correction = gated, score_correction, int(identity), None
        if pair_limit is not None and not pair_limit > 0:
            raise ValueError(f"pair_limit must be positive, got {pair_limit}")
        self.has_router_bias, self.pair_limit, self.router_bias = router_bias, pair_limit, None
        if not 1 <= top_k <= num_experts + identity:
            raise ValueError(f"top_k {top_k} must be within 1..{num_experts + identity}, the router's rows")
        if groups is not None:
            count, keep = groups
            if count < 1 or num_experts % count or not 1 <= keep <= count or top_k > keep * (num_experts // count):
                raise ValueError(f"{count} groups of which {keep} are kept do not fit {num_experts} experts with {top_k} per token")
            groups = None if count == 1 else (int(count), int(keep))
        self.groups = groups
        if activation not in ops.GATES:
            raise ValueError(f"unknown activation {activation!r}; known: {', '.join(sorted(ops.GATES))}")
        self.activation = activation
        self.hidden_size, self.num_experts, self.top_k = hidden_size, num_experts, top_k
        self.expert_size, self.shared_size = expert_size, shared_size
        self.shared_gated, self.renormalize = shared_gated and shared_size > 0, renormalize
        self.router = self.expert_gate = self.expert_up = self.expert_down = None
        self.shared_gate = self.shared_up = self.shared_down = self.shared_scale = None

    def param_specs(self):
        E, H, I, S = self.num_experts, self.hidden_size, self.expert_size, self.shared_size
        specs = {"router": ParamSpec((E + self.identity, H), role="router"),
                 "expert_gate": ParamSpec((E, I, H)), "expert_up": ParamSpec((E, I, H)),
                 "expert_down": ParamSpec((E, H, I))}
        if not self.gated:
            del specs["expert_gate"]
        if self.score_correction:
            specs["correction"] = ParamSpec((E + self.identity,), role="bias")
        if self.has_router_bias:
            specs["router_bias"] = ParamSpec((E,), role="bias")
        if S > 0:
            specs.update({"shared_gate": ParamSpec((S, H)), "shared_up": ParamSpec((S, H)),
                          "shared_down": ParamSpec((H, S))})
            if self.shared_gated:
                specs["shared_scale"] = ParamSpec((1, H), role="router")
        return specs

    def prepare(self, device, act):
        if self.has_router_bias:     # it enters float arithmetic only
            self.router_bias = self.router_bias.float().contiguous()
        if self.score_correction:
            self.correction = self.correction.float().contiguous()
        if self.shared_size > 0:     # as in the dense part; the experts' products never leave this library's kernels
            self.shared_gate, self.shared_up = ops.side_by_side(self.shared_gate, self.shared_up)

    def native(self):
        from ..csrc import host_api
        w = host_api.weight
        if (self.groups is not None or self.has_router_bias or self.pair_limit is not None or not self.gated or self.score_correction
                or self.sigmoid_scores or self.shared_limit is not None or self.weight_scale != 1.0):
            return None                  # the executor chooses among all experts, by logits without a bias, for plain pairs
        return host_api.MoeFfnDesc(self.hidden_size, self.num_experts, self.top_k, self.expert_size, self.shared_size,
                                   int(self.renormalize), ops.GATES[self.activation], w(self.router),
                                   w(self.shared_scale if self.shared_gated else None), w(self.expert_gate), w(self.expert_up),
                                   w(self.expert_down), w(self.shared_gate), w(self.shared_up), w(self.shared_down))

    def forward(self, normed, normed32, ctx):
        T = normed.shape[0]
        unit = ops.expert_tile_rows(T * self.top_k, self.num_experts, ctx.act, normed, self.expert_gate if self.gated else self.expert_up,
                                    **({} if self.expert_size % 8 == 0 else {"w_behind": self.expert_down}))
        if self.score_correction or not self.gated:
            return self._forward_scored(normed, normed32, ctx, unit)
        route = lambda: ops.route(normed32, self.router, self.shared_scale if self.shared_gated else None,
                                  self.top_k, self.renormalize, unit, ctx.act,
                                  **({} if self.groups is None else {"groups": self.groups}),
                                  **({} if self.router_bias is None else {"bias": self.router_bias}),
                                  **({} if self.weight_scale == 1.0 else {"weight_scale": self.weight_scale}),
                                  **({} if not self.sigmoid_scores else {"sigmoid": True, "pair_groups": self.pair_groups}))
        limit = {} if self.pair_limit is None else {"pair_limit": self.pair_limit}
        if self.shared_size > 0 and T <= 16 and unit == 16:
            # a handful of tokens: the shared expert's two products ride in the launches of the routed experts'
            _, weights, gate, sorted_token, pair_slot, tile_expert, n_tiles = route()
            experts = dict(a_rows=sorted_token, tile_group=tile_expert, n_tiles=n_tiles, tile_rows=unit)
            h, hs = ops.gemm_pair(dict(a=normed, w=self.expert_gate, w2=self.expert_up, out_act=True,
                                       activation=self.activation, **experts, **limit),
                                  dict(a=normed, w=self.shared_gate, w2=self.shared_up, out_act=True,
                                       activation=self.activation, **self._shared_limit()), ctx.act)
            y, shared = ops.gemm_pair(dict(a=h, w=self.expert_down, gather=False, **experts),
                                      dict(a=hs, w=self.shared_down, partial_sums=True), ctx.act)
            return ops.GatheredSum(y, pair_slot, weights, shared, gate)
        # The shared expert needs nothing from the router: it may run on a second stream beside the routed experts.
        # That pays while its products are a few passes of tiles over the chip, whose ends the other stream's work
        # fills (2,048 tokens of width 5,632: 5 % of the step; 512 tokens: 10 %); with eight passes and more the two
        # only disturb each other (2,048 tokens of width 20,480: 2 % slower).
        shared, side = None, None
        if self.shared_size > 0:
            tiles = -(-T // 128) * -(-self.shared_size // 128)
            # Below some 300 tokens the host's part of forking and joining (2.6 ms of a step of 24 layers, which is
            # then as long on the host as on the chip) is more than the second stream gains: a prompt step of 65 tokens
            # took 6.8 ms with it and 5.4 without, one of 200 tokens 6.8 and 6.3, of 320 tokens 7.15 and 7.2, of 512
            # tokens 7.9 and 8.8.  A step that is being captured pays the host once and is replayed with the two
            # streams (64 sequences: 10.8 ms a step with them, 11.15 without).
            worth = T >= SIDE_STREAM_FROM or getattr(ctx, "capturing", False)
            side = ctx.fork() if hasattr(ctx, "fork") and worth and tiles < 8 * 256 else None
            if side is not None:
                with torch.cuda.stream(side):
                    shared = self._shared(normed, ctx)
            else:
                shared = self._shared(normed, ctx)
        _, weights, gate, sorted_token, pair_slot, tile_expert, n_tiles = route()
        rows = ops.expert_product_rows(unit, T * self.top_k, self.num_experts)
        h = ops.gemm(normed, self.expert_gate, ctx.act, w2=self.expert_up, out_act=True, a_rows=sorted_token,
                     tile_group=tile_expert, n_tiles=n_tiles, tile_rows=rows, activation=self.activation, **limit)
        y = ops.gemm(h, self.expert_down, ctx.act, a_rows=sorted_token, tile_group=tile_expert, n_tiles=n_tiles,
                     tile_rows=rows, gather=False)
        if side is not None:
            ctx.join()
        # the weighted sum over the chosen experts and the shared expert is left to the next norm
        return ops.GatheredSum(y, pair_slot, weights, shared, gate)

    def _forward_scored(self, normed, normed32, ctx, unit):
        """Experts of two matrices, and routers that choose by corrected scores with experts that are the identity."""
        T = normed.shape[0]
        extra = {"correction": self.correction, "identity": self.identity} if self.score_correction else \
            ({} if self.groups is None else {"groups": self.groups}) | ({} if self.router_bias is None else {"bias": self.router_bias})
        _, weights, own, sorted_token, pair_slot, tile_expert, n_tiles = ops.route(
            normed32, self.router, None, self.top_k, self.renormalize, unit, ctx.act, **extra)
        rows = ops.expert_product_rows(unit, T * self.top_k, self.num_experts)
        order = dict(a_rows=sorted_token, tile_group=tile_expert, n_tiles=n_tiles, tile_rows=rows)
        if self.gated:
            h = ops.gemm(normed, self.expert_gate, ctx.act, w2=self.expert_up, out_act=True, activation=self.activation,
                         **order, **({} if self.pair_limit is None else {"pair_limit": self.pair_limit}))
        else:
            h = ops.gemm(normed, self.expert_up, ctx.act, out_act=True, activation=self.activation, act_alone=True, **order)
        y = ops.gemm(h, self.expert_down, ctx.act, gather=False, **order)
        # a token's weights for the experts that are the identity multiply its own float32 row, which rides where a shared
        # expert's output would
        return ops.GatheredSum(y, pair_slot, weights, normed32[None] if self.identity else None, own if self.identity else None)

    def _shared_limit(self) -> dict:
        return {} if self.shared_limit is None else {"pair_limit": self.shared_limit}

    def _shared(self, normed, ctx):
        hs = ops.gemm(normed, self.shared_gate, ctx.act, w2=self.shared_up, out_act=True, activation=self.activation,
                      **self._shared_limit())
        return ops.gemm(hs, self.shared_down, ctx.act, partial_sums=True)
