"""Small Gokezen configurations with sizes and constants of their own, and random weights for them."""
from __future__ import annotations

import json
import os

import numpy as np
import torch


def mixer(left, right, left_scale=1.0, right_scale=1.0):
    """``left``: (heads, kv_heads, dim, vdim, window or None[, scale]); ``right``: (heads, dim, vdim[, gate_cap])."""
    heads, kv, dim, vdim, window, *scale = left
    a = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale[0] if scale else dim ** -0.5}
    if window is not None:
        a["mask"] = {"size": window}
    h, d, v, *cap = right
    return {"left": a, "right": {"heads": h, "dim": d, "vdim": v, "gate_cap": cap[0] if cap else 15.0},
            "left_scale": left_scale, "right_scale": right_scale}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, groups=None, scale=1.0, limit=2.0, shared=None):
    """``groups``: (count, keep); ``shared``: (ff, limit)."""
    router = {"experts": experts, "top": top, "scale": scale}
    if groups is not None:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    out = {"kind": "moe", "router": router, "expert": {"ff": ff, "limit": limit}}
    if shared is not None:
        out["shared"] = {"ff": shared[0], "limit": shared[1]}
    return out


def config(width, vocab, layers, loop=None, eps=1e-5, max_positions=600):
    """``layers``: (mixer, mlp or None); ``loop``: (start, stop, times)."""
    cfg = {"architecture": "Gokezen", "vocab": vocab, "width": width, "max_positions": max_positions, "norm": {"eps": eps},
           "layers": [{"type": "parallel", "mixer": m, "mlp": mlp} for m, mlp in layers]}
    if loop is not None:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


CASES = {
    # each mechanism by itself: the other half's factor is zero
    "attention_only": config(64, 96, [(mixer((4, 2, 16, 16, 40), (1, 8, 8), 1.0, 0.0), None)]),
    "memory_only": config(64, 96, [(mixer((1, 1, 8, 8, 5), (4, 16, 24), 0.0, 1.0), None)]),
    "dense_only": config(40, 50, [(mixer((1, 1, 8, 8, 4), (1, 4, 4), 0.0, 0.0), dense(24))]),
    "experts_only": config(48, 60, [(mixer((1, 1, 8, 8, 4), (1, 4, 4), 0.0, 0.0),
                                     moe(12, 3, 20, groups=(4, 2), scale=1.7, limit=0.7, shared=(28, 1.9)))]),
    "loop_only": config(32, 40, [(mixer((2, 1, 8, 8, 3), (2, 8, 8), 0.5, 1.5), None)], loop=(0, 1, 3)),
    # sizes that are no multiples of 16, 8 or 4; value widths other than key widths; one kv head and as many as heads; windows
    # below and above a page, and none; negative and equal factors; a loop over some of the layers; groups of one expert, of two,
    # all groups kept, no groups; one expert, all experts chosen; with and without a shared expert; no feed-forward
    "odd": config(72, 101, [
        (mixer((6, 3, 20, 28, 70, 0.31), (3, 20, 12, 4.0), 1.3, -0.7), moe(6, 6, 18, groups=(3, 3), scale=0.6, limit=1.5)),
        (mixer((3, 3, 24, 8, 9), (2, 12, 36, 30.0), 0.4, 0.4), dense(36)),
        (mixer((5, 1, 12, 20, 100), (1, 40, 4), -1.0, 2.0), moe(8, 2, 12, groups=(8, 4), scale=2.2, limit=0.5, shared=(10, 3.0))),
        (mixer((2, 2, 8, 8, None), (6, 4, 8, 1.5), 0.9, 1.1), moe(10, 3, 16, groups=(5, 2), shared=(33, 0.8))),
        (mixer((6, 2, 20, 28, 1), (3, 20, 12)), moe(1, 1, 10, scale=3.0)),
    ], loop=(1, 4, 2)),
    # a width that is no multiple of four, heads of 10, three numbers of a head's memory, windows of a page and around it; a loop
    # that reaches the last layer and runs once
    "ragged": config(50, 67, [
        (mixer((5, 5, 10, 10, 64), (3, 3, 5, 8.0), 1.0, 1.0), dense(10)),
        (mixer((2, 1, 6, 14, 65), (1, 10, 7), 0.8, 1.2), moe(9, 4, 14, groups=(3, 2), limit=0.4, shared=(9, 0.9))),
        (mixer((4, 4, 2, 2, 63), (5, 2, 2, 2.0), 1.5, 0.5), None),
    ], loop=(1, 3, 1), eps=1e-6),
    # heads as wide as served models have them, and memories beyond what the matrix-core form takes
    "wide": config(256, 300, [
        (mixer((4, 1, 128, 128, 200), (2, 128, 128), 0.7, 1.2), dense(512)),
        (mixer((2, 2, 64, 128, 130), (1, 256, 40), 1.0, 0.6), moe(16, 4, 128, groups=(4, 2), scale=2.0, limit=3.0, shared=(192, 2.0))),
        (mixer((4, 2, 32, 32, None), (1, 300, 20), 1.0, 1.0), None),
    ], loop=(0, 2, 2)),
    # as a served model's layers might be laid out, small
    "regular": config(128, 256, [
        (mixer((4, 2, 32, 32, 80), (2, 32, 32), 1.1, 0.6), dense(192)),
        (mixer((4, 2, 32, 32, 80), (2, 32, 48), 1.1, 0.6), moe(16, 4, 64, groups=(4, 2), scale=1.5, limit=1.2, shared=(80, 2.5))),
        (mixer((4, 1, 32, 64, 50), (4, 32, 32), 0.9, 0.8), moe(8, 2, 64, scale=1.2, shared=(64, 1.2))),
        (mixer((4, 4, 32, 32, 80), (2, 64, 32), 1.0, 1.0), dense(320)),
    ], loop=(1, 3, 3), max_positions=1100),
}


def random_case(seed: int) -> dict:
    """A configuration drawn from sizes of many kinds."""
    rng = np.random.default_rng(9000 + seed)
    pick = lambda xs: xs[int(rng.integers(len(xs)))]
    divisors = lambda n: [d for d in range(1, n + 1) if n % d == 0]
    layers = []
    for _ in range(int(rng.integers(1, 5))):
        heads, dim = pick([1, 2, 3, 4, 6, 8]), pick([4, 8, 12, 16, 24, 32, 40, 48, 64, 80, 96])
        left = (heads, pick(divisors(heads)), dim, pick([4, 8, 16, 24, 32, 48, 64, 72, 96]),
                pick([None, 1, 2, 31, 64, 65, 100, 128]), float(rng.uniform(0.5, 1.5)) * dim ** -0.5)
        right = (pick([1, 2, 3, 5, 8]), pick([2, 4, 8, 16, 20, 32, 48, 64, 96]), pick([3, 4, 8, 16, 24, 32, 64, 96]),
                 pick([2.0, 5.0, 15.0, 30.0]))
        mlp = None
        if rng.random() < 0.4:
            mlp = dense(pick([8, 20, 24, 40, 64, 100, 130]))
        elif rng.random() < 0.8:
            experts = pick([1, 2, 4, 6, 8, 12, 16])
            count = pick(divisors(experts))
            keep = int(rng.integers(1, count + 1))
            mlp = moe(experts, int(rng.integers(1, keep * (experts // count) + 1)), pick([8, 12, 24, 40, 72]),
                      groups=None if count == 1 and rng.random() < 0.5 else (count, keep), scale=pick([0.5, 1.0, 2.5]),
                      limit=pick([0.5, 1.0, 2.0, 7.0]), shared=None if rng.random() < 0.3 else (pick([8, 16, 30, 64]), pick([0.6, 1.0, 5.0])))
        layers.append((mixer(left, right, float(rng.uniform(0.3, 1.5)), float(rng.uniform(0.3, 1.5))), mlp))
    n = len(layers)
    start = int(rng.integers(n))
    loop = None if rng.random() < 0.3 else (start, int(rng.integers(start + 1, n + 1)), int(rng.integers(1, 4)))
    return config(pick([40, 56, 64, 90, 96, 120, 160, 200, 256]), int(rng.integers(50, 500)), layers, loop=loop,
                  eps=pick([1e-5, 1e-6, 1e-3]))


def tensors(cfg: dict, seed: int, peaky: float = 1.0) -> dict[str, np.ndarray]:
    """Random weights as float64 arrays whose values are bfloat16 numbers.  ``peaky`` scales the attentions' queries, so that
    single keys decide a row of the softmax."""
    rng = np.random.default_rng(seed)
    W = cfg["width"]
    out = {}

    def put(name, shape, std=1.0, mean=0.0):
        v = torch.tensor(rng.normal(mean, std, size=shape), dtype=torch.float32).to(torch.bfloat16)
        out[name] = v.to(torch.float64).numpy()

    put("embed", (cfg["vocab"], W), 0.5)
    put("pos", (cfg["max_positions"], W), 0.3)
    if cfg.get("loop") is not None:
        put("loop.step", (cfg["loop"]["times"], W), 0.4)
    for i, layer in enumerate(cfg["layers"]):
        p, a, b = f"l{i}.", layer["mixer"]["left"], layer["mixer"]["right"]
        put(p + "norm1", (W,), 0.1, 1.0)
        H, G, D, V = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
        put(p + "mix.left.q", (H * D, W), peaky * W ** -0.5)
        put(p + "mix.left.k", (G * D, W), W ** -0.5)
        put(p + "mix.left.v", (G * V, W), W ** -0.5)
        put(p + "mix.left.o", (W, H * V), (H * V) ** -0.5)
        H, D, V = b["heads"], b["dim"], b["vdim"]
        for n, rows in (("q", H * D), ("k", H * D), ("v", H * V), ("g", H * V), ("i", H), ("f", H)):
            put(f"{p}mix.right.{n}", (rows, W), W ** -0.5)
        put(p + "mix.right.i.b", (H,), 1.0, -0.5)
        put(p + "mix.right.f.b", (H,), 1.5, 2.5)        # some heads forget within a few tokens, some keep hundreds
        put(p + "mix.right.norm", (H * V,), 0.1, 1.0)
        put(p + "mix.right.o", (W, H * V), (H * V) ** -0.5)
        f = layer["mlp"]
        if f is None:
            continue
        if f["kind"] == "dense":
            put(p + "mlp.gate", (f["ff"], W), W ** -0.5)
            put(p + "mlp.up", (f["ff"], W), W ** -0.5)
            put(p + "mlp.down", (W, f["ff"]), f["ff"] ** -0.5)
        else:
            named = [(f"e{e}", f["expert"]["ff"]) for e in range(f["router"]["experts"])]
            if f.get("shared") is not None:
                named.append(("shared", f["shared"]["ff"]))
            for n, ff in named:
                put(f"{p}mlp.{n}.gate", (ff, W), 2.0 * W ** -0.5)      # wide enough for the limits to bite
                put(f"{p}mlp.{n}.up", (ff, W), 2.0 * W ** -0.5)
                put(f"{p}mlp.{n}.down", (W, ff), ff ** -0.5)
            put(p + "mlp.router", (f["router"]["experts"], W), 1.5 * W ** -0.5)
    put("final.norm", (W,), 0.1, 1.0)
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
