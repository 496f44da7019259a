"""Pumozen: a small decoder-only design whose layers are listed one by one in config.json.

What is specific to the design and lives here: the keys of its config.json, its tensor names, which part serves which kind of
layer.  The mechanisms themselves are parts with their constants as arguments (``parts/``): a layer norm on every part's output
only (``outnorm`` blocks: the parts read the residual stream itself); attention whose queries and keys are normed over all heads
together, whose values are its keys as projected and whose softmax has one added to its denominator; differential attention
with a temperature by position, an output gate and layers on another layer's keys and values; selective state spaces in their
dual form (Mamba-2); clamped gated pairs, dense and as experts by softmax scores renormalised over the chosen, with a gated
shared one; a vector per token and layer that joins the stream behind the feed-forward, gated by the stream.

config.json: ``architecture`` "Pumozen", ``vocab``, ``width``, ``norm.eps``, ``token_side.dim`` (absent: no such vectors) and
``layers``, a list whose entries give ``type``, the mixer's sizes and constants (``mixer``) and the feed-forward (``mlp``):

* "attention": ``heads``, ``kv_heads``, ``dim``, ``vdim`` (as dim: the values are the keys), ``scale``, ``rot.dims`` and
  ``rot.base`` (absent: no rotation), ``kv_from``;
* "attention_2" (differential): ``heads``, ``kv_heads``, ``dim``, ``vdim``, ``scale``, ``diff``, ``q_temp.coef`` and
  ``q_temp.every`` (absent: none), ``kv_from``;
* "mamba2": ``heads``, ``vdim``, ``state``, ``groups``, ``conv``, ``norm_groups``;
* ``mlp``: ``kind`` "dense" with ``ff`` and ``limit``, or "moe" with ``router`` (``experts``, ``top``, ``scale``), ``expert`` and
  ``shared`` (``ff`` and ``limit`` each; ``shared`` absent: none); null for a layer without one.

A mixer with ``kv_from``: j has no keys and values of its own and reads those that layer j keeps.  Layer i's tensors are named
``l<i>.*``; a linear weight is stored [out, in].  The logits are the embedding table's products.
"""
from __future__ import annotations

from dataclasses import dataclass, field

from ..config.base import ConfigError, KeyReader, require
from ..config.plan import LayerSpec, ModelPlan, PartSpec, ScheduleEntry, Source
from ..config.registry import Architecture, register_architecture

ARCHITECTURE = "Pumozen"
ATTENTION, DIFFERENTIAL, MAMBA = "attention", "attention_2", "mamba2"
PAIR_ACTIVATION = "swish1702"       # g sigmoid(1.702 g): fixed by the design
MAX_POSITIONS = 1 << 24             # the design names no bound of its own: the cache's size is the bound


@dataclass
class AttentionMixer:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot_dims: int               # 0: no rotation
    rot_base: float
    kv_from: int | None


@dataclass
class DifferentialMixer:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    diff: float
    q_temp: tuple[float, float] | None      # coef, every
    kv_from: int | None


@dataclass
class MambaMixer:
    heads: int
    vdim: int
    state: int
    groups: int
    conv: int
    norm_groups: int


@dataclass
class Pair:
    ff: int
    limit: float


@dataclass
class ExpertsFfn:
    experts: int
    top: int
    scale: float
    expert: Pair
    shared: Pair | None


@dataclass
class PumozenLayer:
    type: str
    mixer: AttentionMixer | DifferentialMixer | MambaMixer
    mlp: Pair | ExpertsFfn | None


@dataclass
class PumozenConfig:
    vocab: int
    width: int
    eps: float
    side_dim: int | None
    layers: list[PumozenLayer] = field(default_factory=list)


def _object(data: dict, key: str, where: str, optional: bool = False) -> dict | None:
    v = data.get(key)
    if v is None and optional:
        return None
    if not isinstance(v, dict):
        raise ConfigError(f"{where}: key {key!r} must be an object, got {v!r}")
    return v


def _heads(r: KeyReader, where: str) -> tuple[int, int]:
    heads, kv = r.integer("heads", minimum=1), r.integer("kv_heads", minimum=1)
    require(heads % kv == 0, f"{where}: heads {heads} is not a multiple of kv_heads {kv}")
    return heads, kv


def _attention(m: dict, where: str) -> AttentionMixer:
    r = KeyReader(m, where)
    heads, kv = _heads(r, where)
    dim = r.integer("dim", minimum=1)
    vdim = r.integer("vdim", dim, minimum=1)
    require(vdim == dim, f"{where}: the values are the keys, so vdim {vdim} must be dim {dim}")
    rot = _object(m, "rot", where, optional=True)
    dims, base = 0, 1.0
    if rot is not None:
        q = KeyReader(rot, where + ".rot")
        dims, base = q.integer("dims", minimum=0), q.number("base")
        require(dims % 2 == 0 and dims <= dim, f"{where}.rot: dims {dims} must be even and at most dim {dim}")
        require(base > 0, f"{where}.rot: base must be positive")
    return AttentionMixer(heads, kv, dim, vdim, r.number("scale"), dims, base, r.optional_integer("kv_from"))


def _differential(m: dict, where: str) -> DifferentialMixer:
    r = KeyReader(m, where)
    heads, kv = _heads(r, where)
    temp = _object(m, "q_temp", where, optional=True)
    q_temp = None
    if temp is not None:
        q = KeyReader(temp, where + ".q_temp")
        q_temp = (q.number("coef"), q.number("every"))
        require(q_temp[1] > 0, f"{where}.q_temp: every must be positive")
    return DifferentialMixer(heads, kv, r.integer("dim", minimum=1), r.integer("vdim", minimum=1), r.number("scale"),
                             r.number("diff"), q_temp, r.optional_integer("kv_from"))


def _mamba(m: dict, where: str) -> MambaMixer:
    r = KeyReader(m, where)
    out = MambaMixer(*(r.integer(k, minimum=1) for k in ("heads", "vdim", "state", "groups", "conv", "norm_groups")))
    require(out.heads % out.groups == 0, f"{where}: heads {out.heads} is not a multiple of groups {out.groups}")
    require(out.heads * out.vdim % out.norm_groups == 0,
            f"{where}: {out.heads} heads of {out.vdim} do not fall into {out.norm_groups} equal parts")
    return out


def _pair(f: dict, where: str) -> Pair:
    r = KeyReader(f, where)
    limit = r.number("limit")
    require(limit > 0, f"{where}: limit must be positive")
    return Pair(r.integer("ff", minimum=1), limit)


def _mlp(f: dict | None, where: str) -> Pair | ExpertsFfn | None:
    if f is None:
        return None
    kind = f.get("kind")
    require(kind in ("dense", "moe"), f"{where}: feed-forward kind {kind!r} is not implemented (dense and moe are)")
    if kind == "dense":
        return _pair(f, where)
    r = KeyReader(_object(f, "router", where), where + ".router")
    experts, top = r.integer("experts", minimum=1), r.integer("top", minimum=1)
    require(top <= experts, f"{where}: top {top} exceeds experts {experts}")
    shared = _object(f, "shared", where, optional=True)
    return ExpertsFfn(experts, top, r.number("scale", 1.0), _pair(_object(f, "expert", where), where + ".expert"),
                      None if shared is None else _pair(shared, where + ".shared"))


READERS = {ATTENTION: _attention, DIFFERENTIAL: _differential, MAMBA: _mamba}


def config_from_json(data: dict) -> PumozenConfig:
    r = KeyReader(data)
    side = _object(data, "token_side", "config.json", optional=True)
    cfg = PumozenConfig(vocab=r.integer("vocab", minimum=1), width=r.integer("width", minimum=1),
                        eps=KeyReader(_object(data, "norm", "config.json"), "config.json: norm").number("eps"),
                        side_dim=None if side is None else KeyReader(side, "config.json: token_side").integer("dim", minimum=1))
    require(cfg.eps > 0, "norm.eps must be positive")
    layers = data.get("layers")
    require(isinstance(layers, list) and layers, "key 'layers' must be a list with at least one layer")
    for i, entry in enumerate(layers):
        where = f"config.json: layers[{i}]"
        require(isinstance(entry, dict), f"layers[{i}] must be an object")
        kind = entry.get("type")
        require(kind in READERS, f"layers[{i}].type {kind!r} is not implemented ({', '.join(READERS)} are)")
        m = READERS[kind](_object(entry, "mixer", where), where + ".mixer")
        j = getattr(m, "kv_from", None)
        if j is not None:
            require(0 <= j < i and cfg.layers[j].type == kind and cfg.layers[j].mixer.kv_from is None,
                    f"layers[{i}].mixer.kv_from {j} names no earlier layer of this type with keys and values of its own")
            a = cfg.layers[j].mixer
            require((a.kv_heads, a.dim, a.vdim) == (m.kv_heads, m.dim, m.vdim),
                    f"layers[{i}].mixer.kv_from {j}: the two layers' key and value heads differ")
        cfg.layers.append(PumozenLayer(kind, m, _mlp(_object(entry, "mlp", where, optional=True), where + ".mlp")))
    return cfg


def config_to_json(c: PumozenConfig) -> dict:
    layers = []
    for layer in c.layers:
        m, f = layer.mixer, layer.mlp
        if layer.type == MAMBA:
            mixer = {k: getattr(m, k) for k in ("heads", "vdim", "state", "groups", "conv", "norm_groups")}
        else:
            mixer = {k: getattr(m, k) for k in ("heads", "kv_heads", "dim", "vdim", "scale")}
            if layer.type == ATTENTION and m.rot_dims:
                mixer["rot"] = {"dims": m.rot_dims, "base": m.rot_base}
            if layer.type == DIFFERENTIAL:
                mixer["diff"] = m.diff
                if m.q_temp is not None:
                    mixer["q_temp"] = {"coef": m.q_temp[0], "every": m.q_temp[1]}
            if m.kv_from is not None:
                mixer["kv_from"] = m.kv_from
        mlp = None
        if isinstance(f, Pair):
            mlp = {"kind": "dense", "ff": f.ff, "limit": f.limit}
        elif f is not None:
            mlp = {"kind": "moe", "router": {"experts": f.experts, "top": f.top, "scale": f.scale},
                   "expert": {"ff": f.expert.ff, "limit": f.expert.limit}}
            if f.shared is not None:
                mlp["shared"] = {"ff": f.shared.ff, "limit": f.shared.limit}
        layers.append({"type": layer.type, "mixer": mixer, "mlp": mlp})
    out = {"architecture": ARCHITECTURE, "vocab": c.vocab, "width": c.width, "norm": {"eps": c.eps}, "layers": layers}
    if c.side_dim is not None:
        out["token_side"] = {"dim": c.side_dim}
    return out


def _mixer_spec(c: PumozenConfig, i: int) -> PartSpec:
    layer, p = c.layers[i], f"l{i}.mix."
    m = layer.mixer
    named = lambda **names: {k: Source.single(p + v) for k, v in names.items()}
    if layer.type == MAMBA:
        return PartSpec(kind="ssd",
                        args=dict(hidden_size=c.width, num_heads=m.heads, value_dim=m.vdim, state_dim=m.state, groups=m.groups,
                                  conv_taps=m.conv, norm_parts=m.norm_groups, eps=c.eps),
                        tensors=named(in_weight="in", conv="conv", conv_bias="conv.b", dt_bias="dt_bias", a_log="A_log", skip="D",
                                      out_norm="norm", out_weight="o"))
    own = m.kv_from is None
    if layer.type == ATTENTION:
        tensors = named(q_weight="q", q_norm="q.norm", out_weight="o") | (named(k_weight="k", k_norm="k.norm") if own else {})
        position = PartSpec(kind="none") if m.rot_dims == 0 else \
            PartSpec(kind="rope", args=dict(head_dim=m.dim, rotary_dim=m.rot_dims, theta=m.rot_base, double_table=True))
        return PartSpec(kind="gqa_attention",
                        args=dict(hidden_size=c.width, num_heads=m.heads, num_kv_heads=m.kv_heads, head_dim=m.dim, scale=m.scale,
                                  position=position, separate_qkv=True, row_norm_eps=c.eps, values_are_keys=True, unit_sink=True,
                                  shares_kv=not own),
                        tensors=tensors)
    tensors = named(q_weight="q", q_norm="q.norm", lq1="lq1", lk1="lk1", lq2="lq2", lk2="lk2", g_weight="g", out_weight="o")
    if own:
        tensors |= named(k_weight="k", v_weight="v", k_norm="k.norm")
    return PartSpec(kind="differential_attention",
                    args=dict(hidden_size=c.width, num_heads=m.heads, num_kv_heads=m.kv_heads, head_dim=m.dim, value_dim=m.vdim,
                              eps=c.eps, diff=m.diff, scale=m.scale, temperature=m.q_temp, shares_kv=not own),
                    tensors=tensors)


def _ffn_spec(c: PumozenConfig, i: int) -> PartSpec:
    f, q = c.layers[i].mlp, f"l{i}.mlp."
    if isinstance(f, Pair):
        return PartSpec(kind="dense_swiglu",
                        args=dict(hidden_size=c.width, inner_size=f.ff, activation=PAIR_ACTIVATION, pair_limit=f.limit),
                        tensors={n: Source.single(q + n) for n in ("gate", "up", "down")})
    tensors = {"router": Source.single(q + "router")}
    for n in ("gate", "up", "down"):
        tensors[f"expert_{n}"] = Source.stack([f"{q}e{e}.{n}" for e in range(f.experts)])
        if f.shared is not None:
            tensors[f"shared_{n}"] = Source.single(f"{q}shared.{n}")
    if f.shared is not None:
        tensors["shared_scale"] = Source.single(q + "shared.sg")
    return PartSpec(kind="moe_swiglu",
                    args=dict(hidden_size=c.width, num_experts=f.experts, top_k=f.top, expert_size=f.expert.ff,
                              pair_limit=f.expert.limit, shared_size=0 if f.shared is None else f.shared.ff, shared_gated=True,
                              shared_limit=None if f.shared is None else f.shared.limit, renormalize=True, weight_scale=f.scale,
                              activation=PAIR_ACTIVATION),
                    tensors=tensors)


def plan(c: PumozenConfig) -> ModelPlan:
    def norm(name: str) -> PartSpec:
        return PartSpec(kind="layernorm", args=dict(size=c.width, eps=c.eps),
                        tensors={"weight": Source.single(name), "bias": Source.single(name + ".b")})

    layers, schedule = [], []
    for i, layer in enumerate(c.layers):
        parts = {"mixer": _mixer_spec(c, i), "mixer_norm": norm(f"l{i}.norm1")}
        if layer.mlp is not None:
            parts |= {"ffn": _ffn_spec(c, i), "ffn_norm": norm(f"l{i}.norm2")}
        if c.side_dim is not None:
            parts["side"] = PartSpec(kind="token_side",
                                     args=dict(hidden_size=c.width, dim=c.side_dim, first_column=i * c.side_dim, eps=c.eps),
                                     tensors={n: Source.single(f"l{i}.side.{n}") for n in ("gate", "proj", "norm")})
        layers.append(LayerSpec(block="outnorm", parts=parts))
        schedule.append(ScheduleEntry(layer=i, cache_of=getattr(layer.mixer, "kv_from", None)))
    return ModelPlan(
        architecture=ARCHITECTURE,
        vocab_size=c.vocab,
        hidden_size=c.width,
        layers=layers,
        schedule=schedule,
        final_norm=norm("final.norm"),
        embedding=Source.single("embed"),
        lm_head=None,
        max_positions=MAX_POSITIONS,
        token_table=Source.single("side.embed") if c.side_dim is not None else None,
        token_table_width=len(c.layers) * (c.side_dim or 0),
    )


register_architecture(Architecture(
    name=ARCHITECTURE,
    config_from_json=config_from_json,
    plan=plan,
    config_to_json=config_to_json,
))
