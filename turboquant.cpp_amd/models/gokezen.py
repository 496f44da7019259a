"""Gokezen: a small decoder-only design whose layers are listed one by one in config.json.

What is specific to the design and lives here: the keys of its config.json, its tensor names, which part serves which
kind of layer.  The mechanisms themselves are parts with their constants as arguments (``parts/``): one norm in front of a
mixer and a feed-forward that run side by side (``parallel`` blocks); a mixer of two mixers side by side with a factor each,
attention with grouped heads, a window and no rotation, and a matrix memory with exponential gates; a dense gated
feed-forward and one of routed experts whose pairs are clamped, chosen by sigmoid scores within the groups with the best two
scores, with a shared expert beside them; a learned vector per position; layers that run several times in a row with the same
weights, each pass with a cache and a state of its own and with a learned vector added to the stream before it.

config.json: ``architecture`` "Gokezen", ``vocab``, ``width``, ``max_positions``, ``norm.eps``, optionally ``loop`` (``start``,
``stop``, ``times``: layers start .. stop - 1 run ``times`` times in a row) and ``layers``, a list whose entries give ``type``
("parallel"), the mixer (``mixer.left``: ``heads``, ``kv_heads``, ``dim``, ``vdim``, ``scale``, ``mask.size`` (absent: no window);
``mixer.right``: ``heads``, ``dim``, ``vdim``, ``gate_cap``; ``left_scale``, ``right_scale``) and the feed-forward (``mlp``: ``kind``
"dense" with ``ff``, or "moe" with ``router`` (``experts``, ``top``, ``scale``, ``groups.count`` and ``groups.keep`` (absent: one
group)), ``expert`` and ``shared`` (``ff`` and ``limit`` each; ``shared`` absent: none); null for a layer without one).  Layer i's
tensors are named ``l<i>.*``; a linear weight is stored [out, in].  The logits are the embedding table's products.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass, field

from ..config.base import ConfigError, KeyReader, require
from ..config.plan import LayerSpec, ModelPlan, PartSpec, ScheduleEntry, Source
from ..config.registry import Architecture, register_architecture

ARCHITECTURE = "Gokezen"
PARALLEL = "parallel"
EXPERT_ACTIVATION = "swish1702"     # g sigmoid(1.702 g): fixed by the design


@dataclass
class AttentionMixer:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: int | None


@dataclass
class MemoryMixer:
    heads: int
    dim: int
    vdim: int
    gate_cap: float


@dataclass
class SideBySide:
    left: AttentionMixer
    right: MemoryMixer
    left_scale: float
    right_scale: float


@dataclass
class DenseFfn:
    ff: int


@dataclass
class Expert:
    ff: int
    limit: float


@dataclass
class ExpertsFfn:
    experts: int
    top: int
    scale: float
    groups: tuple[int, int] | None      # count, keep; None: the choice is among all experts
    expert: Expert
    shared: Expert | None


@dataclass
class GokezenLayer:
    type: str
    mixer: SideBySide
    mlp: DenseFfn | ExpertsFfn | None


@dataclass
class Loop:
    start: int
    stop: int
    times: int


@dataclass
class GokezenConfig:
    vocab: int
    width: int
    max_positions: int
    eps: float
    loop: Loop | None = None
    layers: list[GokezenLayer] = field(default_factory=list)


def _object(data: dict, key: str, where: str, optional: bool = False) -> dict | None:
    v = data.get(key)
    if v is None and optional:
        return None
    if not isinstance(v, dict):
        raise ConfigError(f"{where}: key {key!r} must be an object, got {v!r}")
    return v


def _mixer(m: dict, where: str) -> SideBySide:
    a, b = _object(m, "left", where), _object(m, "right", where)
    l, r, s = KeyReader(a, where + ".left"), KeyReader(b, where + ".right"), KeyReader(m, where)
    heads, kv = l.integer("heads", minimum=1), l.integer("kv_heads", minimum=1)
    require(heads % kv == 0, f"{where}.left: heads {heads} is not a multiple of kv_heads {kv}")
    mask = _object(a, "mask", where + ".left", optional=True)
    window = KeyReader(mask, where + ".left.mask").integer("size", minimum=1) if mask is not None else None
    left = AttentionMixer(heads, kv, l.integer("dim", minimum=1), l.integer("vdim", minimum=1), l.number("scale"), window)
    cap = r.number("gate_cap")
    require(cap > 0, f"{where}.right: gate_cap must be positive")
    right = MemoryMixer(r.integer("heads", minimum=1), r.integer("dim", minimum=1), r.integer("vdim", minimum=1), cap)
    return SideBySide(left, right, s.number("left_scale"), s.number("right_scale"))


def _expert(f: dict, key: str, where: str) -> Expert:
    r = KeyReader(_object(f, key, where), f"{where}.{key}")
    limit = r.number("limit")
    require(limit > 0, f"{where}.{key}: limit must be positive")
    return Expert(r.integer("ff", minimum=1), limit)


def _mlp(f: dict | None, where: str) -> DenseFfn | ExpertsFfn | None:
    if f is None:
        return None
    kind = f.get("kind")
    require(kind in ("dense", "moe"), f"{where}: feed-forward kind {kind!r} is not implemented (dense and moe are)")
    if kind == "dense":
        return DenseFfn(KeyReader(f, where).integer("ff", minimum=1))
    router = _object(f, "router", where)
    r = KeyReader(router, where + ".router")
    experts, top = r.integer("experts", minimum=1), r.integer("top", minimum=1)
    require(top <= experts, f"{where}: top {top} exceeds experts {experts}")
    groups = None
    if router.get("groups") is not None:
        g = KeyReader(_object(router, "groups", where + ".router"), where + ".router.groups")
        count, keep = g.integer("count", minimum=1), g.integer("keep", minimum=1)
        require(experts % count == 0 and keep <= count and top <= keep * (experts // count),
                f"{where}: {count} groups of which {keep} are kept do not fit {experts} experts with {top} per token")
        groups = (count, keep)
    return ExpertsFfn(experts, top, r.number("scale", 1.0), groups, _expert(f, "expert", where),
                      None if f.get("shared") is None else _expert(f, "shared", where))


def config_from_json(data: dict) -> GokezenConfig:
    r = KeyReader(data)
    cfg = GokezenConfig(vocab=r.integer("vocab", minimum=1), width=r.integer("width", minimum=1),
                        max_positions=r.integer("max_positions", minimum=1),
                        eps=KeyReader(_object(data, "norm", "config.json"), "config.json: norm").number("eps"))
    require(cfg.eps > 0, "norm.eps must be positive")
    layers = data.get("layers")
    require(isinstance(layers, list) and layers, "key 'layers' must be a list with at least one layer")
    for i, entry in enumerate(layers):
        where = f"config.json: layers[{i}]"
        require(isinstance(entry, dict), f"layers[{i}] must be an object")
        kind = entry.get("type")
        require(kind == PARALLEL, f"layers[{i}].type {kind!r} is not implemented ({PARALLEL} is)")
        cfg.layers.append(GokezenLayer(kind, _mixer(_object(entry, "mixer", where), where + ".mixer"),
                                       _mlp(_object(entry, "mlp", where, optional=True), where + ".mlp")))
    loop = _object(data, "loop", "config.json", optional=True)
    if loop is not None:
        l = KeyReader(loop, "config.json: loop")
        cfg.loop = Loop(l.integer("start", minimum=0), l.integer("stop", minimum=1), l.integer("times", minimum=1))
        require(cfg.loop.start < cfg.loop.stop <= len(layers),
                f"loop: layers {cfg.loop.start} .. {cfg.loop.stop} - 1 are not among the {len(layers)} layers")
    return cfg


def complete(cfg: GokezenConfig, shapes: dict) -> GokezenConfig:
    """How many positions the table of learned position vectors has, if that is not what config.json says."""
    cfg = copy.deepcopy(cfg)
    if len(shapes.get("pos", ())) == 2:
        cfg.max_positions = int(shapes["pos"][0])
    return cfg


def config_to_json(c: GokezenConfig) -> dict:
    layers = []
    for layer in c.layers:
        m, f = layer.mixer, layer.mlp
        left = {"heads": m.left.heads, "kv_heads": m.left.kv_heads, "dim": m.left.dim, "vdim": m.left.vdim, "scale": m.left.scale}
        if m.left.window is not None:
            left["mask"] = {"size": m.left.window}
        right = {"heads": m.right.heads, "dim": m.right.dim, "vdim": m.right.vdim, "gate_cap": m.right.gate_cap}
        if f is None:
            mlp = None
        elif isinstance(f, DenseFfn):
            mlp = {"kind": "dense", "ff": f.ff}
        else:
            router = {"experts": f.experts, "top": f.top, "scale": f.scale}
            if f.groups is not None:
                router["groups"] = {"count": f.groups[0], "keep": f.groups[1]}
            mlp = {"kind": "moe", "router": router, "expert": {"ff": f.expert.ff, "limit": f.expert.limit}}
            if f.shared is not None:
                mlp["shared"] = {"ff": f.shared.ff, "limit": f.shared.limit}
        layers.append({"type": layer.type, "mlp": mlp,
                       "mixer": {"left": left, "right": right, "left_scale": m.left_scale, "right_scale": m.right_scale}})
    out = {"architecture": ARCHITECTURE, "vocab": c.vocab, "width": c.width, "max_positions": c.max_positions,
           "norm": {"eps": c.eps}, "layers": layers}
    if c.loop is not None:
        out["loop"] = {"start": c.loop.start, "stop": c.loop.stop, "times": c.loop.times}
    return out


def plan(c: GokezenConfig) -> ModelPlan:
    def norm(name: str) -> PartSpec:
        return PartSpec(kind="rmsnorm", args=dict(size=c.width, eps=c.eps), tensors={"weight": Source.single(name)})

    layers = []
    for i, layer in enumerate(c.layers):
        m, f = layer.mixer, layer.mlp
        p = f"l{i}.mix.left."
        left = PartSpec(
            kind="gqa_attention",
            args=dict(hidden_size=c.width, num_heads=m.left.heads, num_kv_heads=m.left.kv_heads, head_dim=m.left.dim,
                      value_dim=m.left.vdim, scale=m.left.scale, window=m.left.window, separate_qkv=True,
                      position=PartSpec(kind="none")),
            tensors={"q_weight": Source.single(p + "q"), "k_weight": Source.single(p + "k"), "v_weight": Source.single(p + "v"),
                     "out_weight": Source.single(p + "o")})
        p = f"l{i}.mix.right."
        right = PartSpec(
            kind="matrix_memory",
            args=dict(hidden_size=c.width, num_heads=m.right.heads, head_dim=m.right.dim, value_dim=m.right.vdim,
                      gate_cap=m.right.gate_cap, eps=c.eps),
            tensors={"q_weight": Source.single(p + "q"), "k_weight": Source.single(p + "k"), "v_weight": Source.single(p + "v"),
                     "g_weight": Source.single(p + "g"), "i_weight": Source.single(p + "i"), "f_weight": Source.single(p + "f"),
                     "i_bias": Source.single(p + "i.b"), "f_bias": Source.single(p + "f.b"),
                     "out_norm": Source.single(p + "norm"), "out_weight": Source.single(p + "o")})
        parts = {"norm": norm(f"l{i}.norm1"),
                 "mixer": PartSpec(kind="parallel", args=dict(left=left, right=right, left_scale=m.left_scale,
                                                              right_scale=m.right_scale))}
        q = f"l{i}.mlp."
        if isinstance(f, DenseFfn):
            parts["ffn"] = PartSpec(kind="dense_swiglu", args=dict(hidden_size=c.width, inner_size=f.ff, activation="gelu_tanh"),
                                    tensors={n: Source.single(q + n) for n in ("gate", "up", "down")})
        elif f is not None:
            E = range(f.experts)
            tensors = {"router": Source.single(q + "router")}
            for n in ("gate", "up", "down"):
                tensors[f"expert_{n}"] = Source.stack([f"{q}e{e}.{n}" for e in E])
                if f.shared is not None:
                    tensors[f"shared_{n}"] = Source.single(f"{q}shared.{n}")
            parts["ffn"] = PartSpec(
                kind="moe_swiglu",
                args=dict(hidden_size=c.width, num_experts=f.experts, top_k=f.top, expert_size=f.expert.ff,
                          pair_limit=f.expert.limit, shared_size=0 if f.shared is None else f.shared.ff, shared_gated=False,
                          shared_limit=None if f.shared is None else f.shared.limit, renormalize=True,
                          activation=EXPERT_ACTIVATION, groups=f.groups, sigmoid_scores=True, weight_scale=f.scale,
                          pair_groups=True),
                tensors=tensors)
        layers.append(LayerSpec(block="parallel", parts=parts))
    n = len(layers)
    loop = c.loop if c.loop is not None else Loop(n, n, 0)
    schedule = [ScheduleEntry(layer=i) for i in range(loop.start)]
    for t in range(loop.times):       # every pass is a run of its own: with its own cache and state, its vector before it
        schedule += [ScheduleEntry(layer=i, step_vector=t if i == loop.start else None) for i in range(loop.start, loop.stop)]
    schedule += [ScheduleEntry(layer=i) for i in range(loop.stop, n)]
    return ModelPlan(
        architecture=ARCHITECTURE,
        vocab_size=c.vocab,
        hidden_size=c.width,
        layers=layers,
        schedule=schedule,
        final_norm=norm("final.norm"),
        embedding=Source.single("embed"),
        lm_head=None,
        max_positions=c.max_positions,
        position_table=Source.single("pos"),
        step_vectors=Source.single("loop.step") if c.loop is not None else None,
        n_step_vectors=loop.times,
    )


register_architecture(Architecture(
    name=ARCHITECTURE,
    config_from_json=config_from_json,
    plan=plan,
    config_to_json=config_to_json,
    complete=complete,
))
