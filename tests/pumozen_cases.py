"""Small Pumozen configurations with sizes and constants of their own, and random weights for them."""
from __future__ import annotations

import json
import os

import numpy as np
import torch


def attention(heads, kv_heads, dim, rot=None, scale=None, kv_from=None):
    """``rot``: (dims, base)."""
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5 if scale is None else scale}
    if rot is not None:
        m["rot"] = {"dims": rot[0], "base": rot[1]}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return "attention", m


def differential(heads, kv_heads, dim, vdim, diff=0.5, temp=None, scale=None, kv_from=None):
    """``temp``: (coef, every)."""
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": dim ** -0.5 if scale is None else scale, "diff": diff}
    if temp is not None:
        m["q_temp"] = {"coef": temp[0], "every": temp[1]}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return "attention_2", m


def mamba(heads, vdim, state, groups=1, conv=4, norm_groups=1):
    return "mamba2", {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": norm_groups}


def dense(ff, limit=2.0):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(experts, top, ff, scale=1.0, limit=2.0, shared=None):
    """``shared``: (ff, limit)."""
    out = {"kind": "moe", "router": {"experts": experts, "top": top, "scale": scale}, "expert": {"ff": ff, "limit": limit}}
    if shared is not None:
        out["shared"] = {"ff": shared[0], "limit": shared[1]}
    return out


def config(width, vocab, layers, side=None, eps=1e-5):
    """``layers``: ((type, mixer), mlp or None); ``side``: the width of a token's own vectors, None: no such vectors."""
    cfg = {"architecture": "Pumozen", "vocab": vocab, "width": width, "norm": {"eps": eps},
           "layers": [{"type": kind, "mixer": m, "mlp": mlp} for (kind, m), mlp in layers]}
    if side is not None:
        cfg["token_side"] = {"dim": side}
    return cfg


CASES = {
    # each mechanism by itself
    "attention_only": config(64, 96, [(attention(4, 2, 16, (16, 1e4)), None)]),
    "differential_only": config(64, 96, [(differential(4, 2, 16, 32, 0.3, (0.4, 20)), None)]),
    "mamba_only": config(64, 96, [(mamba(4, 16, 24, groups=2, norm_groups=2), None)]),
    "side_only": config(40, 50, [(mamba(1, 4, 2), None), (mamba(1, 4, 2), None)], side=8),
    "dense_only": config(40, 50, [(mamba(1, 4, 2), dense(24, 0.7))]),
    "experts_only": config(48, 60, [(mamba(1, 4, 2), moe(12, 3, 20, scale=1.7, limit=0.7, shared=(28, 1.9)))]),
    "shared_keys_only": config(48, 60, [(differential(4, 2, 8, 16, 0.2), None), (differential(2, 2, 8, 16, 0.7, (0.3, 9), kv_from=0), None),
                                        (attention(4, 2, 12, (8, 100.0)), None), (attention(6, 2, 12, (4, 1e3), kv_from=2), None),
                                        (differential(6, 2, 8, 16, 0.5, kv_from=0), None)]),
    # sizes that are no multiples of 16, 8 or 4; values wider and narrower than two maps; rotations of a part, of nothing and of
    # all of a head; one kv head and as many as heads; one tap, many taps; a state of one channel; every head a group, a norm per group of
    # heads; experts: one, all chosen, no shared one; no feed-forward
    "odd": config(72, 101, [
        (attention(6, 3, 20, (12, 5e3), scale=0.31), moe(6, 6, 18, scale=0.6, limit=1.5)),
        (mamba(6, 12, 20, groups=3, conv=7, norm_groups=3), dense(36)),
        (differential(6, 3, 12, 20, 0.3, (0.25, 16), scale=0.4), moe(8, 2, 12, scale=2.2, limit=0.5, shared=(10, 3.0))),
        (differential(3, 3, 12, 20, 0.1, kv_from=2), None),
        (attention(5, 1, 12), dense(20, 0.3)),
        (mamba(3, 14, 1, groups=3, conv=1), moe(1, 1, 10, scale=3.0)),
        (differential(4, 1, 20, 12, 0.35, (-0.2, 40)), dense(33, 5.0)),
    ], side=12),
    # a width that is no multiple of four, heads of 10 and 6, a state space of odd sizes, token vectors of six numbers
    "ragged": config(50, 67, [
        (differential(5, 5, 10, 14, 0.6, (0.5, 7)), dense(10)),
        (mamba(5, 6, 7, groups=5, conv=3, norm_groups=3), moe(9, 4, 14, limit=0.4, shared=(9, 0.9))),
        (attention(4, 4, 6, (2, 10.0)), None),
        (mamba(2, 9, 3, groups=2, conv=2, norm_groups=2), dense(7, 1.1)),
    ], side=6, eps=1e-6),
    # heads as wide as served models have them, and beyond what single kernels take: rows of 64, 128, 256 and 320 for two maps, states
    # of 128, 256 and 300 channels
    "wide": config(256, 300, [
        (attention(4, 1, 128, (64, 1e6)), dense(512, 3.0)),
        (differential(4, 2, 64, 128, 0.6, (0.3, 64)), moe(16, 4, 128, scale=1.5, limit=3.0, shared=(192, 2.0))),
        (mamba(8, 64, 128, groups=2), None),
        (differential(2, 1, 128, 256, 0.4), dense(300)),
        (mamba(2, 40, 256, groups=1, norm_groups=2), None),
        (differential(2, 2, 160, 80, 0.7, (0.1, 50)), None),
        (differential(6, 2, 32, 64, 0.2), None),
        (mamba(3, 20, 300, groups=3, conv=5), None),
    ], side=16),
    # as a served model's layers might be laid out, small
    "regular": config(128, 256, [
        (attention(4, 2, 32, (32, 1e4)), dense(192)),
        (differential(4, 2, 16, 32, 0.6, (0.5, 100)), moe(16, 4, 64, scale=1.5, limit=1.2, shared=(80, 2.5))),
        (mamba(8, 32, 32, groups=2, norm_groups=2), dense(320)),
        (differential(4, 2, 16, 32, 0.6, (0.5, 100), kv_from=1), moe(8, 2, 64, scale=1.2, shared=(64, 1.2))),
    ], side=24),
}


def random_case(seed: int) -> dict:
    """A configuration drawn from sizes of many kinds."""
    rng = np.random.default_rng(7000 + seed)
    pick = lambda xs: xs[int(rng.integers(len(xs)))]
    divisors = lambda n: [d for d in range(1, n + 1) if n % d == 0]
    layers = []
    for i in range(int(rng.integers(1, 7))):
        kind = pick(["attention", "attention_2", "mamba2"])
        heads = pick([1, 2, 3, 4, 6, 8])
        if kind == "mamba2":
            V = pick([3, 4, 8, 16, 24, 32, 64, 96])
            mixer = mamba(heads, V, pick([2, 4, 8, 16, 20, 32, 48, 64, 96]), pick(divisors(heads)), pick([1, 2, 3, 4, 4, 5, 8]),
                          pick(divisors(heads * V)) if rng.random() < 0.5 else pick(divisors(heads)))
        else:
            owners = [j for j, ((k, m), _) in enumerate(layers) if k == kind and "kv_from" not in m]
            j = pick(owners) if owners and rng.random() < 0.6 else None
            kv = layers[j][0][1]["kv_heads"] if j is not None else pick(divisors(heads))
            heads = heads if j is None else kv * pick([1, 2, 3])
            if kind == "attention":
                dim = layers[j][0][1]["dim"] if j is not None else pick([4, 8, 10, 16, 24, 32, 40, 48, 64, 80, 96])
                rot = None if rng.random() < 0.25 else (2 * int(rng.integers(1, dim // 2 + 1)), pick([10.0, 500.0, 1e4, 1e6]))
                mixer = attention(heads, kv, dim, rot, float(rng.uniform(0.5, 1.5)) * dim ** -0.5, j)
            else:
                dim, vdim = (layers[j][0][1][k] for k in ("dim", "vdim")) if j is not None else (pick([4, 8, 12, 16, 24, 32, 48, 64]),
                                                                                                 pick([4, 8, 16, 24, 32, 64, 96, 128]))
                temp = None if rng.random() < 0.3 else (float(rng.uniform(-0.3, 0.6)), pick([1, 5, 16, 33, 64, 100]))
                mixer = differential(heads, kv, dim, vdim, float(rng.uniform(0.1, 0.9)), temp, float(rng.uniform(0.5, 1.5)) * dim ** -0.5, j)
        mlp = None
        if rng.random() < 0.4:
            mlp = dense(pick([8, 20, 24, 40, 64, 100, 130]), pick([0.5, 1.0, 2.0, 7.0]))
        elif rng.random() < 0.8:
            experts = pick([1, 2, 4, 6, 8, 12, 16])
            mlp = moe(experts, int(rng.integers(1, experts + 1)), pick([8, 12, 24, 40, 72]), scale=pick([0.5, 1.0, 2.5]),
                      limit=pick([0.5, 1.0, 2.0, 7.0]), shared=None if rng.random() < 0.3 else (pick([8, 16, 30, 64]), pick([0.6, 1.0, 5.0])))
        layers.append((mixer, mlp))
    return config(pick([40, 56, 64, 90, 96, 120, 160, 200, 256]), int(rng.integers(50, 500)), layers,
                  side=None if rng.random() < 0.2 else pick([1, 4, 8, 10, 16, 24]), eps=pick([1e-5, 1e-6, 1e-3]))


def tensors(cfg: dict, seed: int, peaky: float = 1.0) -> dict[str, np.ndarray]:
    """Random weights as float64 arrays whose values are bfloat16 numbers.  ``peaky`` scales the attentions' query norms, so
    that single keys decide a row of the softmax."""
    rng = np.random.default_rng(seed)
    W = cfg["width"]
    out = {}

    def put(name, shape, std=1.0, mean=0.0):
        v = torch.tensor(rng.normal(mean, std, size=shape), dtype=torch.float32).to(torch.bfloat16)
        out[name] = v.to(torch.float64).numpy()

    def norm(name):
        put(name, (W,), 0.1, 1.0)
        put(name + ".b", (W,), 0.2)

    put("embed", (cfg["vocab"], W), 0.7)
    side = cfg.get("token_side")
    if side is not None:
        put("side.embed", (cfg["vocab"], side["dim"] * len(cfg["layers"])), 1.0)
    for i, layer in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", layer["mixer"], layer["mlp"]
        norm(p + "norm1")
        if layer["type"] == "mamba2":
            H, V, N, G, K = (m[k] for k in ("heads", "vdim", "state", "groups", "conv"))
            C = H * V + 2 * G * N
            put(p + "mix.in", (H * V + C + H, W), W ** -0.5)
            put(p + "mix.conv", (C, K), K ** -0.5)
            put(p + "mix.conv.b", (C,), 0.3)
            put(p + "mix.dt_bias", (H,), 1.5, -1.0)         # some heads forget within a few tokens, some keep hundreds
            put(p + "mix.A_log", (H,), 1.5, -0.5)
            put(p + "mix.D", (H,), 0.5, 1.0)
            put(p + "mix.norm", (H * V,), 0.1, 1.0)
            put(p + "mix.o", (W, H * V), (H * V) ** -0.5)
        else:
            H, G, D, V = (m[k] for k in ("heads", "kv_heads", "dim", "vdim"))
            own, maps = "kv_from" not in m, 2 if layer["type"] == "attention_2" else 1
            put(p + "mix.q", (H * maps * D, W), W ** -0.5)
            put(p + "mix.q.norm", (H * D if maps == 1 else D,), 0.2 * peaky, peaky)
            if own:
                put(p + "mix.k", (G * maps * D, W), W ** -0.5)
                put(p + "mix.k.norm", (G * D if maps == 1 else D,), 0.2, 1.0)
            if maps == 2:
                if own:
                    put(p + "mix.v", (G * V, W), W ** -0.5)
                for n in ("lq1", "lk1", "lq2", "lk2"):
                    put(p + "mix." + n, (D,), 0.3)
                put(p + "mix.g", (H * V, W), W ** -0.5)
            put(p + "mix.o", (W, H * V), (H * V) ** -0.5)
        if f is not None:
            norm(p + "norm2")
            named = [("", f["ff"])] if f["kind"] == "dense" else [(f"e{e}.", f["expert"]["ff"]) for e in range(f["router"]["experts"])]
            if f.get("shared") is not None:
                named.append(("shared.", f["shared"]["ff"]))
                put(p + "mlp.shared.sg", (1, W), W ** -0.5)
            for n, ff in named:
                put(f"{p}mlp.{n}gate", (ff, W), 2.0 * W ** -0.5)      # wide enough for the limits to bite
                put(f"{p}mlp.{n}up", (ff, W), 2.0 * W ** -0.5)
                put(f"{p}mlp.{n}down", (W, ff), ff ** -0.5)
            if f["kind"] == "moe":
                put(p + "mlp.router", (f["router"]["experts"], W), 1.5 * W ** -0.5)
        if side is not None:
            put(p + "side.gate", (side["dim"], W), W ** -0.5)
            put(p + "side.proj", (W, side["dim"]), side["dim"] ** -0.5)
            put(p + "side.norm", (W,), 0.1, 0.5)
    norm("final.norm")
    return out


def write_folder(path: str, cfg: dict, w: dict[str, np.ndarray]) -> str:
    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: torch.tensor(v, dtype=torch.float64).to(torch.bfloat16).contiguous() for k, v in w.items()},
              os.path.join(path, "model.safetensors"))
    return path


def tokens(cfg: dict, n: int, seed: int) -> list[int]:
    return np.random.default_rng(1000 + seed).integers(0, cfg["vocab"], n).tolist()
