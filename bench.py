"""Decode and prefill throughput of the engine on one MI355X, at Qwen1.5-MoE-A2.7B layer sizes with random weights.

    python bench.py [--gpus 1] [--steps K] [--warmup W] [--layers L] [--batch B] [--context C]

A step is one decode step of the whole batch: the step function, greedy sampling on the GPU and the copy of the
chosen tokens to the host, exactly what the generation loop runs.  Prints one JSON line.

    python bench.py --sizes a14b --workload unequal         # 8 prompts of 512 to 4,096 tokens, then 256 decode steps
    python bench.py --dtype float32 --workload unequal      # true 32-bit: 64 prompts of 1 to 2,048 tokens, 64 steps

time the other two workloads: a batch of prompts of unequal lengths in one prompt step, then decode steps.

    python bench.py --design felepel [--design-sizes small,medium] [--layers 8]

times the Felepel design (delta-rule and chunked-attention layers, experts chosen within groups) beside Qwen2-MoE at
equal sizes: prompt steps of 512 and 2,048 tokens, decode steps at batch 1 and 8, and where each model's time goes,
kernel by kernel.  The default run and its line are not touched by it.

    python bench.py --design taminex [--design-sizes small,medium] [--layers 8]

does the same for the Taminex design (a norm on every part's output only; attention with head norms, partial rotation
and a sink; the delta rule with a decay per head; attention over a latent per position, shared between layers; a
feed-forward of two matrices with squared relu) beside Qwen2-MoE with dense feed-forwards of as many weights.

    python bench.py --design beronex [--design-sizes small,medium] [--layers 8]

does it for the Beronex design (norms around every part; attention over a latent with a rotated key part and a latent for
the queries; lightning attention; windowed attention with head norms behind a YaRN rotation, a gate per head and layers on
another layer's keys and values; dense gated feed-forwards and clamped experts in turn) beside Qwen2-MoE with dense
feed-forwards and experts in turn.

    python bench.py --design bosalix [--design-sizes small,medium] [--layers 8]

does it for the Bosalix design (a norm on every part's output only and a mixer input blended with the token before;
windowed attention over a latent with a rotated key part; attention with head norms, unit values mixed between layers,
sigmoid weights and a window that keeps the first positions in sight; experts of two matrices chosen by corrected scores,
some of them the identity) beside Qwen2-MoE with experts in every layer and as many weights.

    python bench.py --design gokezen [--design-sizes small,medium] [--layers 8]

does it for the Gokezen design (mixer and feed-forward side by side behind one norm; windowed attention beside a matrix memory
with exponential gates; dense gated feed-forwards and clamped experts with a shared one, chosen by sigmoid scores within
groups, in turn; a vector added before a looped pass) beside Qwen2-MoE with dense feed-forwards and experts with a shared one
in turn.  A layer of the design has the memory's matrices over those of the layer beside it.

    python bench.py --design pumozen [--design-sizes small,medium] [--layers 8]

does it for the Pumozen design (a layer norm on every part's output only; attention normed over all heads whose values are its
keys, differential attention, Mamba-2; clamped pairs and experts; a vector per token and layer) beside Qwen2-MoE with dense
feed-forwards and experts with a shared one in turn.
"""
from __future__ import annotations

import argparse
import json
import os
import sys
import time

ROOT = os.path.dirname(os.path.abspath(__file__))
sys.path.insert(0, ROOT)

# Qwen1.5-MoE-A2.7B layer sizes
A27B = {
    "architectures": ["Qwen2MoeForCausalLM"], "model_type": "qwen2_moe",
    "vocab_size": 151936, "hidden_size": 2048, "num_hidden_layers": 24, "num_attention_heads": 16,
    "num_key_value_heads": 16, "intermediate_size": 5632, "moe_intermediate_size": 1408,
    "shared_expert_intermediate_size": 5632, "num_experts": 60, "num_experts_per_tok": 4, "norm_topk_prob": False,
    "decoder_sparse_step": 1, "mlp_only_layers": [], "rope_theta": 1000000.0, "rms_norm_eps": 1e-6,
    "use_sliding_window": False, "sliding_window": 32768, "max_window_layers": 24, "max_position_embeddings": 8192,
    "tie_word_embeddings": False, "torch_dtype": "bfloat16",
}
# the other Qwen2-MoE checkpoint's sizes, about 115 GB of bfloat16 weights (`--sizes a14b`)
A14B = dict(A27B, hidden_size=3584, num_hidden_layers=28, num_attention_heads=28, num_key_value_heads=4,
            intermediate_size=18944, moe_intermediate_size=2560, shared_expert_intermediate_size=20480, num_experts=64,
            num_experts_per_tok=8, sliding_window=131072, max_window_layers=28, max_position_embeddings=32768)
SIZES = {"a27b": (A27B, "Qwen1.5-MoE-A2.7B"), "a14b": (A14B, "Qwen2-57B-A14B")}
PEAK_HBM_GBS = 8000.0
PEAK_FLOPS = {"bf16": 2.5e15, "fp32": 157.3e12}
PREFILL_TOKENS = 2048


def layer_weight_elems(c, experts_used: float) -> float:
    H, Q = c["hidden_size"], c["num_attention_heads"] * (c["hidden_size"] // c["num_attention_heads"])
    KV = c["num_key_value_heads"] * (c["hidden_size"] // c["num_attention_heads"])
    attn = H * (Q + 2 * KV) + (Q + 2 * KV) + Q * H
    moe = c["num_experts"] * H + H + 3 * H * c["shared_expert_intermediate_size"] + experts_used * 3 * H * c["moe_intermediate_size"]
    return attn + moe + 2 * H


def decode_bytes(c, layers: int, batch: int, context: float, wbytes: int = 2, used: float | None = None) -> float:
    """Bytes a decode step has to read: every weight it uses once (`used` experts a layer, counted in a step of
    the run; without a count, what a batch of uniformly routed tokens reaches in expectation) and the keys and
    values of the live requests."""
    E, k = c["num_experts"], c["num_experts_per_tok"]
    if used is None:
        used = E * (1.0 - (1.0 - k / E) ** batch)
    hd = c["hidden_size"] // c["num_attention_heads"]
    w = layers * layer_weight_elems(c, used) + c["vocab_size"] * c["hidden_size"] + c["hidden_size"]
    kv = batch * context * layers * 2 * c["num_key_value_heads"] * hd
    return wbytes * (w + kv)


def prefill_flops(c, layers: int, T: int, rows_out: int = 1) -> float:
    H, nh = c["hidden_size"], c["num_attention_heads"]
    hd = H // nh
    Q, KV = nh * hd, c["num_key_value_heads"] * hd
    per_layer = (2 * T * H * (Q + 2 * KV) + 2 * T * Q * H + 4 * nh * hd * T * (T + 1) / 2
                 + 2 * T * H * (c["num_experts"] + 1)
                 + 2 * T * c["num_experts_per_tok"] * 3 * H * c["moe_intermediate_size"]
                 + 2 * T * 3 * H * c["shared_expert_intermediate_size"])
    return layers * per_layer + 2 * rows_out * H * c["vocab_size"]


def probe() -> int:
    """The measured counterparts of the published peaks: one JSON line."""
    import torch
    from turboquant_cpp_amd.csrc import ops
    dev = "cuda:0"

    def timed(fn, reps):
        fn()
        torch.cuda.synchronize()
        a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
        a.record()
        for _ in range(reps):
            fn()
        b.record()
        torch.cuda.synchronize()
        return a.elapsed_time(b) * 1e-3 / reps

    buf = torch.randint(0, 2 ** 31 - 1, (2 ** 28,), dtype=torch.int32, device=dev)      # 1 GiB
    nbytes = buf.numel() * 4
    out = {"metric": "measured peaks", "read_bytes": nbytes}
    for name, once in (("read_GBs", False), ("read_once_hint_GBs", True)):
        out[name] = round(nbytes / timed(lambda: ops.probe_stream(buf, once), 10) / 1e9, 0)
    del buf
    for shape in (32, 16):
        for name, seed in (("same_values", 0), ("random_values", 12345)):
            flop = [0.0]

            def run():
                flop[0] = ops.probe_mfma(shape, 512, 20000, seed, dev)
            t = timed(run, 3)
            out[f"mfma_{shape}_{name}_TFLOPs"] = round(flop[0] / t / 1e12, 0)
    out["published"] = {"hbm_GBs": PEAK_HBM_GBS, "bf16_TFLOPs": PEAK_FLOPS["bf16"] / 1e12}
    print(json.dumps(out))
    return 0


def plain_products(short: str) -> str:
    """Whose kernels run the plain products of a long prompt step (decode steps always run this library's own)."""
    from turboquant_cpp_amd.csrc import ops
    if short == "bf16" and ops._VENDOR:
        return f"hipBLASLt from {ops.VENDOR_MIN_ROWS} rows (TQ_PLAIN_PRODUCTS=own: this library's)"
    return "own kernels"


def count_experts(fn, engine):
    """Runs fn() (an eager decode step, part by part so that the routing can be watched) and returns the mean number of
    distinct experts a layer's router picked."""
    import torch
    from turboquant_cpp_amd.csrc import ops
    picked = []
    route = ops.route

    def counting_route(*a, **k):
        out = route(*a, **k)
        picked.append(int(torch.unique(out[0]).numel()))
        return out

    ops.route = counting_route
    executor, engine.native = engine.native, None
    try:
        result = fn()
    finally:
        ops.route = route
        engine.native = executor
    return result, sum(picked) / max(len(picked), 1)


def unequal_defaults(sizes: str) -> dict:
    """The two stated workloads of unequal prompts: the larger checkpoint's sizes in bfloat16 (8 prompts of 512 to 4,096
    tokens, seed 3, 256 decode steps) and the headline sizes in true 32-bit (64 prompts of 1 to 2,048, seed 4, 64 steps)."""
    big = sizes == "a14b"
    return {"batch": 8 if big else 64, "lo": 512 if big else 1, "hi": 4096 if big else 2048, "steps": 256 if big else 64,
            "seed": 3 if big else 4}


def unequal_workload(sizes: str, act: str, layers: int | None, wl: dict) -> dict:
    """A batch of prompts of unequal lengths in one prompt step, then decode steps; builds its own model with random
    weights and returns the record (the keys of the default run's line)."""
    import torch
    from turboquant_cpp_amd.csrc import ops
    from turboquant_cpp_amd.engine.model import random_model
    from turboquant_cpp_amd.engine.step import Engine
    from turboquant_cpp_amd.sampling.sampler import TokenFetch
    cfg, model_name = dict(SIZES[sizes][0]), SIZES[sizes][1]
    full_layers = cfg["num_hidden_layers"]
    layers = full_layers if layers is None else layers
    cfg["num_hidden_layers"] = cfg["max_window_layers"] = layers
    cfg["max_position_embeddings"] = wl["hi"] + wl["steps"] + 64
    short = "bf16" if act == "bfloat16" else "fp32"
    wbytes = 2 if act == "bfloat16" else 4
    dev = "cuda:0"
    t0 = time.time()
    model = random_model(cfg, seed=wl["seed"], act=act, device=dev)
    torch.cuda.synchronize()
    print(f"[bench] {model_name} sizes, {layers} layers, {short}: random weights on the device in {time.time() - t0:.1f}s "
          f"({model.weight_bytes / 1e9:.1f} GB)", file=sys.stderr, flush=True)
    V = cfg["vocab_size"]
    B = wl["batch"]
    g = torch.Generator().manual_seed(wl["seed"])
    lens = torch.randint(wl["lo"], wl["hi"] + 1, (B,), generator=g).tolist()
    prompts = [torch.randint(0, V, (n,), generator=g).tolist() for n in lens]
    page = 64
    engine = Engine(model, max_tokens=sum(-(-(n + wl["steps"] + 1) // page) * page for n in lens), page_size=page, max_slots=B)
    fetch = TokenFetch(dev, B)
    best = None
    for rep in range(2):                  # the first pass loads kernels and captures the decode graphs
        slots = engine.open(B)
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        logits = engine.step(slots, prompts)
        torch.cuda.synchronize()
        t_prompt = time.perf_counter() - t0
        tokens = ops.argmax(logits, act)
        used = None
        t0 = time.perf_counter()
        for i in range(wl["steps"]):
            fetch.start(tokens)
            if rep == 1 and i == 0:       # an eager step of the timed pass also counts the experts that are read
                graphs, engine.graphs = engine.graphs, None
                lg, used = count_experts(lambda: engine.step_from_device(slots, tokens), engine)
                engine.graphs = graphs
            else:
                lg = engine.step_from_device(slots, tokens)
            fetch.wait()
            tokens = ops.argmax(lg, act)
        torch.cuda.synchronize()
        t_decode = time.perf_counter() - t0
        engine.close(slots)
        best = (t_prompt, t_decode, used)
    t_prompt, t_decode, used = best
    T = sum(lens)
    sec = t_decode / wl["steps"]
    mean_total_ctx = T + B * (wl["steps"] + 1) / 2.0
    read = decode_bytes(cfg, layers, B, mean_total_ctx / B, wbytes, used)
    flops = sum(prefill_flops(cfg, layers, n, 0) for n in lens) + 2.0 * B * cfg["hidden_size"] * V
    out = {
        "metric": f"decode tok/s, batch {B} of unequal prompts ({wl['lo']}..{wl['hi']} tokens), {wl['steps']} steps "
                  f"({model_name} layer sizes, random weights)",
        "value": round(B / sec, 1), "unit": "tok/s", "n_gpus": 1, "steps": wl["steps"], "warmup": 0,
        "ms_per_step": round(sec * 1e3, 4), "higher_is_better": True, "scaling": "weak", "vs_baseline": None,
        "dtype": short, "data": "synthetic",
        "config": {"model": f"{model_name} sizes", "layers": layers, "layers_of_full_model": full_layers,
                   "hidden": cfg["hidden_size"], "heads": cfg["num_attention_heads"], "kv_heads": cfg["num_key_value_heads"],
                   "head_dim": cfg["hidden_size"] // cfg["num_attention_heads"], "vocab": V, "experts": cfg["num_experts"],
                   "top_k": cfg["num_experts_per_tok"], "expert_inner": cfg["moe_intermediate_size"],
                   "shared_inner": cfg["shared_expert_intermediate_size"], "global_batch": B,
                   "prompt_tokens": T, "longest_prompt": max(lens), "shortest_prompt": min(lens),
                   "weights": f"random N(0,0.02) seed {wl['seed']}", "kv_cache": short,
                   "experts_read_per_layer": round(used, 1), "parallelism": "single GPU"},
        "prefill": {"value": round(T / t_prompt, 1), "tokens": T, "ms": round(t_prompt * 1e3, 3),
                    "frac": round(flops / t_prompt / PEAK_FLOPS[short], 4), "plain_products": plain_products(short)},
        "roofline": {"bound": "hbm", "achieved": round(read / sec / 1e9, 1), "peak": PEAK_HBM_GBS, "unit": "GB/s",
                     "frac": round(read / sec / 1e9 / PEAK_HBM_GBS, 4)},
        "decode": {"ms_total": round(t_decode * 1e3, 2), "gb_per_step": round(read / 1e9, 2)},
    }
    return out



# ---------------------------------------------------------------- the Felepel design beside Qwen2-MoE at equal sizes
# name -> width, heads, kv heads of the attention, head size, experts, groups, kept groups, experts per token, expert width;
# for Taminex the width of a dense gated feed-forward and the latent's size
DESIGN_SIZES = {
    "small": dict(width=1024, heads=8, kv_heads=2, dim=128, experts=32, groups=4, keep=2, top=4, ff=768, vocab=32000,
                  dense_ff=2816, kv_rank=256),
    "medium": dict(width=2048, heads=16, kv_heads=4, dim=128, experts=64, groups=8, keep=2, top=4, ff=1408, vocab=32000,
                   dense_ff=5632, kv_rank=512),
    "large": dict(width=4096, heads=32, kv_heads=8, dim=128, experts=32, groups=4, keep=1, top=2, ff=4096, vocab=32000,
                  dense_ff=11008, kv_rank=512),
}


def felepel_config(z: dict, layers: int, max_positions: int) -> dict:
    """`layers` layers in the order delta rule, attention, attention, each with tensors of its own, so that the model has
    as many matrices of the same sizes as the Qwen2-MoE model beside it."""
    moe = {"kind": "moe", "expert": {"ff": z["ff"]},
           "router": {"experts": z["experts"], "top": z["top"], "groups": {"count": z["groups"], "keep": z["keep"]}}}
    delta = {"type": "channel_delta", "mlp": moe,
             "mixer": {"heads": z["heads"], "kv_heads": z["heads"], "dim": z["dim"], "vdim": z["dim"], "conv": 4,
                       "decay_rank": 64, "gate_rank": 64}}
    attn = {"type": "attention", "mlp": moe,
            "mixer": {"heads": z["heads"], "kv_heads": z["kv_heads"], "dim": z["dim"], "vdim": z["dim"],
                      "scale": z["dim"] ** -0.5, "softcap": 50.0, "mask": {"size": 1024}}}
    out = []
    for i in range(layers):
        out.append(dict(delta if i % 3 == 0 else attn))
    return {"architecture": "Felepel", "vocab": z["vocab"], "width": z["width"], "max_positions": max_positions,
            "norm": {"eps": 1e-5}, "layers": out}


def taminex_config(z: dict, layers: int, max_positions: int) -> dict:
    """`layers` layers in the order delta rule, attention, latent attention, latent attention on the layer before's
    latents; a feed-forward of two matrices, half as wide again as the gated one of three beside it."""
    mlp = {"kind": "dense", "ff": z["dense_ff"] * 3 // 2}
    H, G, D = z["heads"], z["kv_heads"], z["dim"]
    kinds = [
        {"type": "delta", "mixer": {"heads": H, "kv_heads": H, "dim": D, "vdim": D, "conv": 4}},
        {"type": "attention", "mixer": {"heads": H, "kv_heads": G, "dim": D, "vdim": D, "scale": D ** -0.5,
                                        "rot": {"dims": D // 2, "base": 1e6}}},
        {"type": "latent_attention", "mixer": {"heads": H, "dim": D, "vdim": D, "kv_rank": z["kv_rank"], "scale": D ** -0.5}},
        {"type": "latent_attention", "mixer": {"heads": H, "dim": D, "vdim": D, "kv_rank": z["kv_rank"], "scale": D ** -0.5}},
    ]
    out = []
    for i in range(layers):
        layer = {"type": kinds[i % 4]["type"], "mixer": dict(kinds[i % 4]["mixer"]), "mlp": mlp}
        if i % 4 == 3:
            layer["mixer"]["kv_from"] = i - 1
        out.append(layer)
    return {"architecture": "Taminex", "vocab": z["vocab"], "width": z["width"], "norm": {"eps": 1e-5}, "logit_scale": 1.0,
            "logit_softcap": 40.0, "layers": out}


def qwen_dense_config_like(z: dict, layers: int, max_positions: int) -> dict:
    """Qwen2-MoE's layers with the dense gated feed-forward in every layer (`mlp_only_layers`)."""
    return dict(A27B, vocab_size=z["vocab"], hidden_size=z["width"], num_hidden_layers=layers, num_attention_heads=z["heads"],
                num_key_value_heads=z["kv_heads"], head_dim=z["dim"], intermediate_size=z["dense_ff"],
                mlp_only_layers=list(range(layers)), max_window_layers=layers, max_position_embeddings=max_positions)


def beronex_config(z: dict, layers: int, max_positions: int) -> dict:
    """`layers` layers in the order latent attention (queries through a latent, a rotated key part), lightning attention,
    attention with a window, attention on that layer's keys and values; dense gated feed-forwards and routed experts in
    turn.  The cached row of a latent layer is the latent and the rotated part, 512 numbers at most."""
    H, G, D = z["heads"], z["kv_heads"], z["dim"]
    dense = {"kind": "dense", "ff": z["dense_ff"]}
    moe = {"kind": "moe", "router": {"experts": z["experts"], "top": z["top"]}, "expert": {"ff": z["ff"], "limit": 7.0}}
    yarn = {"factor": 8.0, "original": 4096, "fast": 32.0, "slow": 1.0}
    rank = min(z["kv_rank"], 512 - D // 2)
    kinds = [
        ("latent_attention", {"heads": H, "dim": D, "rot_dim": D // 2, "vdim": D, "kv_rank": rank, "q_rank": 3 * z["kv_rank"] // 2,
                              "scale": (D + D // 2) ** -0.5, "rot": {"dims": D // 2, "base": 1e4, "scaling": yarn}}, dense),
        ("lightning", {"heads": H, "dim": D, "vdim": D, "decay": [1.0 - 2.0 ** (-5.0 - 4.0 * h / H) for h in range(H)]}, moe),
        ("attention", {"heads": H, "kv_heads": G, "dim": D, "vdim": D, "scale": D ** -0.5, "mask": {"size": 1024},
                       "rot": {"dims": D, "base": 1e6, "scaling": yarn}}, dense),
        ("attention", {"heads": H, "kv_heads": G, "dim": D, "vdim": D, "scale": D ** -0.5, "mask": {"size": 1024},
                       "rot": {"dims": D, "base": 1e6, "scaling": yarn}}, moe),
    ]
    out = []
    for i in range(layers):
        kind, mixer, mlp = kinds[i % 4]
        out.append({"type": kind, "mixer": dict(mixer, kv_from=i - 1) if i % 4 == 3 else dict(mixer), "mlp": mlp})
    return {"architecture": "Beronex", "vocab": z["vocab"], "width": z["width"], "norm": {"eps": 1e-5},
            "embedding": {"scale": 1.0}, "layers": out}


def bosalix_config(z: dict, layers: int, max_positions: int) -> dict:
    """`layers` layers in the order latent attention, latent attention, attention, attention (the attention layers mix their
    values with the first one's), all with a window of 1,024, every one followed by routed experts of two matrices (half as
    wide again as the gated experts beside them, so that a layer has as many weights) with a quarter as many identity experts.
    The cached row of a latent layer is the latent and the rotated part, 512 numbers at most."""
    H, G, D = z["heads"], z["kv_heads"], z["dim"]
    moe = {"kind": "moe", "router": {"experts": z["experts"], "identity": z["experts"] // 4, "top": z["top"]},
           "expert": {"ff": z["ff"] * 3 // 2}}
    rank = min(z["kv_rank"], 512 - D // 2)
    kinds = [
        ("latent_attention", {"heads": H, "dim": D, "rot_dim": D // 2, "vdim": D, "kv_rank": rank, "q_rank": 3 * z["kv_rank"] // 2,
                              "scale": (D + D // 2) ** -0.5, "mask": {"size": 1024}, "rot": {"dims": D // 2, "base": 1e4}}),
        ("attention", {"heads": H, "kv_heads": G, "dim": D, "vdim": D, "scale": D ** -0.5, "mask": {"size": 1024, "keep_first": 4},
                       "v_mix": True, "rot": {"dims": D // 2, "base": 1e6,
                                              "scaling": {"factor": 8.0, "original": 4096, "low": 1.0, "high": 4.0}}}),
    ]
    out = [{"type": kinds[i % 4 // 2][0], "mixer": dict(kinds[i % 4 // 2][1]), "mlp": moe} for i in range(layers)]
    return {"architecture": "Bosalix", "vocab": z["vocab"], "width": z["width"], "norm": {"eps": 1e-5}, "residual_mult": 0.5,
            "embedding": {"scale": 1.0}, "layers": out}


def gokezen_config(z: dict, layers: int, max_positions: int) -> dict:
    """`layers` layers, dense gated feed-forwards and routed experts with a shared one in turn, each with windowed attention and a
    matrix memory of half as many heads side by side; all but the first and the last are a loop of one pass, so that every
    run has tensors of its own."""
    H, G, D = z["heads"], z["kv_heads"], z["dim"]
    mixer = {"left": {"heads": H, "kv_heads": G, "dim": D, "vdim": D, "scale": D ** -0.5, "mask": {"size": 1024}},
             "right": {"heads": H // 2, "dim": D, "vdim": D, "gate_cap": 15.0}, "left_scale": 1.0, "right_scale": 0.5}
    dense = {"kind": "dense", "ff": z["dense_ff"]}
    moe = {"kind": "moe", "expert": {"ff": z["ff"], "limit": 7.0}, "shared": {"ff": z["ff"], "limit": 7.0},
           "router": {"experts": z["experts"], "top": z["top"], "scale": 2.5, "groups": {"count": z["groups"], "keep": z["keep"]}}}
    return {"architecture": "Gokezen", "vocab": z["vocab"], "width": z["width"], "max_positions": max_positions,
            "norm": {"eps": 1e-5}, "loop": {"start": 1, "stop": layers - 1, "times": 1},
            "layers": [{"type": "parallel", "mixer": mixer, "mlp": moe if i % 2 else dense} for i in range(layers)]}


def pumozen_config(z: dict, layers: int, max_positions: int) -> dict:
    """`layers` layers in the order attention (norm over all heads, values that are the keys), differential attention, Mamba-2,
    differential attention on that layer's keys and values; dense clamped pairs and routed experts with a gated shared one in
    turn; a vector of a sixteenth of the width per token and layer.  A map of the differential attention is half as wide as a
    head (two maps and their values are a head each); the state space has twice the width in heads of half a head, with a state
    of 128 channels and one group."""
    H, G, D, W = z["heads"], z["kv_heads"], z["dim"], z["width"]
    dense = {"kind": "dense", "ff": z["dense_ff"], "limit": 7.0}
    moe = {"kind": "moe", "expert": {"ff": z["ff"], "limit": 7.0}, "shared": {"ff": z["ff"], "limit": 7.0},
           "router": {"experts": z["experts"], "top": z["top"], "scale": 1.5}}
    diff = {"heads": H, "kv_heads": G, "dim": D // 2, "vdim": D, "scale": (D // 2) ** -0.5, "diff": 0.6,
            "q_temp": {"coef": 0.1, "every": 1024}}
    kinds = [
        ("attention", {"heads": H, "kv_heads": G, "dim": D, "vdim": D, "scale": D ** -0.5, "rot": {"dims": D, "base": 1e4}}, dense),
        ("attention_2", diff, moe),
        ("mamba2", {"heads": 4 * W // D, "vdim": D // 2, "state": 128, "groups": 1, "conv": 4, "norm_groups": 1}, dense),
        ("attention_2", diff, moe),
    ]
    out = []
    for i in range(layers):
        kind, mixer, mlp = kinds[i % 4]
        out.append({"type": kind, "mixer": dict(mixer, kv_from=i - 2) if i % 4 == 3 else dict(mixer), "mlp": mlp})
    return {"architecture": "Pumozen", "vocab": z["vocab"], "width": W, "norm": {"eps": 1e-5}, "token_side": {"dim": W // 16},
            "layers": out}


def qwen_mixed_shared_config_like(z: dict, layers: int, max_positions: int) -> dict:
    """The mixed layers with a shared expert as wide as a routed one beside the routed experts."""
    return dict(qwen_mixed_config_like(z, layers, max_positions), shared_expert_intermediate_size=z["ff"])


def qwen_mixed_config_like(z: dict, layers: int, max_positions: int) -> dict:
    """Qwen2-MoE's layers with the dense gated feed-forward in every other layer and routed experts in the rest."""
    return dict(qwen_config_like(z, layers, max_positions), intermediate_size=z["dense_ff"],
                mlp_only_layers=list(range(0, layers, 2)))


def qwen_config_like(z: dict, layers: int, max_positions: int) -> dict:
    return dict(A27B, vocab_size=z["vocab"], hidden_size=z["width"], num_hidden_layers=layers, num_attention_heads=z["heads"],
                num_key_value_heads=z["kv_heads"], head_dim=z["dim"], moe_intermediate_size=z["ff"],
                shared_expert_intermediate_size=0, num_experts=z["experts"], num_experts_per_tok=z["top"],
                max_window_layers=layers, max_position_embeddings=max_positions)


def design_comparison(args) -> int:
    import torch
    from turboquant_cpp_amd.csrc import ops
    from turboquant_cpp_amd.engine.model import random_model
    from turboquant_cpp_amd.engine.step import Engine
    act, dev = args.dtype, "cuda:0"
    short = "bf16" if act == "bfloat16" else "fp32"
    layers = args.layers or (6 if args.design == "felepel" else 8)
    context, prompts_at, batches = 2048, (512, 2048), (1, 8)
    design = {"felepel": ("Felepel", felepel_config, qwen_config_like),
              "taminex": ("Taminex", taminex_config, qwen_dense_config_like),
              "beronex": ("Beronex", beronex_config, qwen_mixed_config_like),
              "bosalix": ("Bosalix", bosalix_config, qwen_config_like),
              "gokezen": ("Gokezen", gokezen_config, qwen_mixed_shared_config_like),
              "pumozen": ("Pumozen", pumozen_config, qwen_mixed_shared_config_like)}[args.design]
    out = {"metric": f"{design[0]} beside Qwen2-MoE at equal sizes: prompt and decode tok/s, and milliseconds by kernel",
           "unit": "tok/s", "dtype": short, "layer_runs": layers, "data": "synthetic", "sizes": {}}

    def measure(cfg):
        model = random_model(cfg, seed=2, act=act, device=dev)
        V = model.plan.vocab_size
        gen = torch.Generator().manual_seed(5)
        rec = {"weights_gb": round(model.weight_bytes / 1e9, 2), "prefill": {}, "decode": {}, "kernels_ms": {}}
        for T in prompts_at:
            engine = Engine(model, max_tokens=T + 64, page_size=64, max_slots=1)
            prompt = torch.randint(0, V, (T,), generator=gen).tolist()
            best = None
            for _ in range(4):
                slot = engine.open(1)
                torch.cuda.synchronize()
                t = time.perf_counter()
                engine.step(slot, [prompt])
                torch.cuda.synchronize()
                dt = time.perf_counter() - t
                engine.close(slot)
                best = dt if best is None else min(best, dt)
            rec["prefill"][str(T)] = {"tok_s": round(T / best, 1), "ms": round(best * 1e3, 3)}
            # where the time goes: part by part on one stream, an event behind every launch
            executor, engine.native, engine.side_stream = engine.native, None, None
            slot = engine.open(1)
            ops.profile_begin()
            engine.step(slot, [prompt])
            prof = ops.profile_end()
            engine.close(slot)
            engine.native = executor
            rec["kernels_ms"][f"prefill_{T}"] = {k: [n, round(ms, 3)] for k, (n, ms) in sorted(prof["kernels"].items())}
            del engine
        for B in batches:
            steps, warm = 32, 4
            engine = Engine(model, max_tokens=(context + 64) * B, page_size=64, max_slots=B)
            slots = engine.open(B)
            for sl in slots:
                engine.step([sl], [torch.randint(0, V, (context - steps - warm,), generator=gen).tolist()])
            tokens = torch.randint(0, V, (B,), generator=gen, dtype=torch.int32).to(dev)
            for _ in range(warm):
                tokens = ops.argmax(engine.step_from_device(slots, tokens), act)
            torch.cuda.synchronize()
            t = time.perf_counter()
            for _ in range(steps):
                tokens = ops.argmax(engine.step_from_device(slots, tokens), act)
            torch.cuda.synchronize()
            sec = (time.perf_counter() - t) / steps
            rec["decode"][f"b{B}_ctx{context}"] = {"tok_s": round(B / sec, 1), "ms_per_step": round(sec * 1e3, 4)}
            graphs, engine.graphs, executor, engine.native = engine.graphs, None, engine.native, None
            ops.profile_begin()
            engine.step_from_device(slots, tokens)
            prof = ops.profile_end()
            engine.graphs, engine.native = graphs, executor
            rec["kernels_ms"][f"decode_b{B}"] = {k: [n, round(ms, 3)] for k, (n, ms) in sorted(prof["kernels"].items())}
            engine.close(slots)
            del engine
        del model
        torch.cuda.empty_cache()
        return rec

    for name in args.design_sizes.split(","):
        z = DESIGN_SIZES[name]
        out["sizes"][name] = {"config": z,
                              args.design: measure(design[1](z, layers, context + 64)),
                              "qwen2_moe": measure(design[2](z, layers, context + 64))}
        print(f"[bench] {name} done", file=sys.stderr, flush=True)
    print(json.dumps(out), flush=True)
    return 0


def main() -> int:
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=64)
    ap.add_argument("--warmup", type=int, default=8)
    ap.add_argument("--sizes", default="a27b", choices=sorted(SIZES), help="whose layer sizes (default: the headline model's)")
    ap.add_argument("--layers", type=int, default=None, help="fewer layers than the model has (default: all)")
    ap.add_argument("--batch", type=int, default=8)
    ap.add_argument("--context", type=int, default=8192)
    ap.add_argument("--points-context", type=int, default=2048)
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    ap.add_argument("--no-points", action="store_true")
    ap.add_argument("--prefill-only", action="store_true", help="time only the prompt step (for profiles)")
    ap.add_argument("--prefill-tokens", type=int, default=PREFILL_TOKENS,
                    help="length of the timed prompt (the contract's line has 2,048; other lengths are for profiles)")
    ap.add_argument("--one-stream", action="store_true",
                    help="no second stream in prompt steps: kernels run one after the other, so that a profile shows "
                         "each kernel's own time")
    ap.add_argument("--generate", action="store_true",
                    help="time the generation loop instead of bare steps: --batch prompts of 512 tokens, 256 new tokens "
                         "each, greedy and with the default sampling (temperature 0.7, top-p 0.9, repetition penalty)")
    ap.add_argument("--probe", action="store_true",
                    help="no model: what this GPU reaches on a plain read of memory and on the matrix instructions alone")
    ap.add_argument("--workload", default="steps", choices=["steps", "unequal"],
                    help="unequal: a batch of prompts of unequal lengths in one prompt step, then decode steps "
                         "(defaults per model: a14b 8 prompts of 512..4096, seed 3, 256 steps; float32 64 prompts of "
                         "1..2048, seed 4, 64 steps)")
    ap.add_argument("--prompt-min", type=int, default=None)
    ap.add_argument("--prompt-max", type=int, default=None)
    ap.add_argument("--decode-steps", type=int, default=None)
    ap.add_argument("--seed", type=int, default=None)
    ap.add_argument("--no-workloads", action="store_true",
                    help="leave out the two workloads of unequal prompts that the default run adds under \"workloads\"")
    ap.add_argument("--design", default=None, choices=["felepel", "taminex", "beronex", "bosalix", "gokezen", "pumozen"],
                    help="time this design beside Qwen2-MoE at equal sizes instead of the default workload")
    ap.add_argument("--design-sizes", default="small,medium", help="of " + ", ".join(DESIGN_SIZES))
    args = ap.parse_args()
    if args.gpus != 1:
        print(f"bench.py measures one GPU; --gpus {args.gpus} is not supported (this engine runs on a single device)")
        return 2
    if args.probe:
        return probe()
    if args.design:
        from turboquant_cpp_amd.csrc import ops as _ops
        _ops.library(args.dtype)
        return design_comparison(args)

    import torch
    from turboquant_cpp_amd.csrc import ops
    from turboquant_cpp_amd.engine.model import random_model
    from turboquant_cpp_amd.engine.step import Engine
    from turboquant_cpp_amd.sampling.sampler import TokenFetch

    cfg, model_name = dict(SIZES[args.sizes][0]), SIZES[args.sizes][1]
    full_layers = cfg["num_hidden_layers"]
    args.layers = full_layers if args.layers is None else args.layers
    cfg["num_hidden_layers"] = args.layers
    cfg["max_window_layers"] = args.layers
    n_prefill = args.prefill_tokens
    cfg["max_position_embeddings"] = max(args.context, args.points_context, n_prefill)
    act = args.dtype
    short = "bf16" if act == "bfloat16" else "fp32"
    dev = "cuda:0"
    ops.library(act)
    if args.workload == "unequal":
        wl = unequal_defaults(args.sizes)
        if args.batch != 8:
            wl["batch"] = args.batch
        for key, given in (("lo", args.prompt_min), ("hi", args.prompt_max), ("steps", args.decode_steps), ("seed", args.seed)):
            if given is not None:
                wl[key] = given
        print(json.dumps(unequal_workload(args.sizes, act, args.layers, wl)), flush=True)
        return 0
    t0 = time.time()
    model = random_model(cfg, seed=2, act=act, device=dev)
    torch.cuda.synchronize()
    print(f"[bench] {args.layers}-layer model with random weights on the device in {time.time() - t0:.1f}s "
          f"({model.weight_bytes / 1e9:.1f} GB)", file=sys.stderr, flush=True)
    V = cfg["vocab_size"]
    gen = torch.Generator().manual_seed(2)

    if args.generate:
        from turboquant_cpp_amd.engine.generate import GenerationOptions, generate
        P, N, B = 512, 256, args.batch
        engine = Engine(model, max_tokens=(P + N + 64) * B, page_size=64, max_slots=B)
        prompts = [torch.randint(0, V, (P,), generator=gen).tolist() for _ in range(B)]
        out = {"metric": f"generated tok/s, {B} prompts of {P} tokens, {N} new tokens each ({model_name}, random weights)",
               "unit": "tok/s", "dtype": short, "layers": args.layers}
        for name, opts in (("greedy", dict(temperature=0.0, rep_penalty=1.0)), ("default_sampling", dict())):
            for _ in range(2):      # the first pass loads kernels and captures the decode step
                torch.cuda.synchronize()
                t0 = time.perf_counter()
                res = generate(engine, prompts, GenerationOptions(max_tokens=N, max_batch=B, loop_detection=False, **opts))
                torch.cuda.synchronize()
                dt = time.perf_counter() - t0
            n = sum(len(r.tokens) for r in res)
            out[name] = {"value": round(n / dt, 1), "tokens": n, "seconds": round(dt, 3)}
        print(json.dumps(out))
        return 0

    wbytes = 2 if act == "bfloat16" else 4

    def run_decode(batch: int, context: int, steps: int, warmup: int):
        """Prefills `batch` prompts so that the timed steps end at `context`, then times `steps` decode steps."""
        prompt_len = context - steps - warmup
        page = 64
        per_seq = -(-context // page) * page
        engine = Engine(model, max_tokens=per_seq * batch, page_size=page, max_slots=batch)
        if args.one_stream:
            engine.side_stream = None
        slots = engine.open(batch)
        prompts = [torch.randint(0, V, (prompt_len,), generator=gen).tolist() for _ in range(batch)]
        tp = time.time()
        logits = None
        # prompts go in one sequence at a time to bound the size of the activations
        for s, p in zip(slots, prompts):
            lg = engine.step([s], [p])
            logits = lg if logits is None else torch.cat([logits, lg])
        torch.cuda.synchronize()
        print(f"[bench] prefilled {batch} x {prompt_len} tokens in {time.time() - tp:.1f}s", file=sys.stderr, flush=True)
        tokens = ops.argmax(logits, act)
        fetch = TokenFetch(dev, batch)

        def one_step(ids):
            """As the generation loop does it: the step is issued from the tokens on the device, and the host
            reads those tokens (to look for end tokens) while the step runs."""
            fetch.start(ids)
            lg = engine.step_from_device(slots, ids)
            fetch.wait()
            return ops.argmax(lg, act)

        # the first warm-up step (which runs eagerly) also counts the distinct experts that each layer's router picks
        tokens, experts_used = count_experts(lambda: one_step(tokens), engine)
        for _ in range(warmup - 1):
            tokens = one_step(tokens)
        torch.cuda.synchronize()
        held = lambda: sum(engine.cache.length(s) for s in slots) / batch
        before = held()
        t = time.perf_counter()
        for _ in range(steps):
            tokens = one_step(tokens)
        torch.cuda.synchronize()
        dt = time.perf_counter() - t
        # what a timed step read on average, from the cache's own count of positions: a step that finds L positions
        # writes one and reads L + 1; the first timed step finds `before`, the last one leaves `context`
        mean_ctx = (before + 1 + held()) / 2.0
        if held() != context or before != context - steps:
            raise RuntimeError(f"the timed steps ran from {before} to {held()} positions, not up to {context}")
        engine.close(slots)
        del engine
        torch.cuda.empty_cache()
        return dt / steps, mean_ctx, experts_used

    def run_prefill(T: int):
        engine = Engine(model, max_tokens=T + 64, page_size=64, max_slots=1)
        if args.one_stream:
            engine.side_stream = None
        prompt = torch.randint(0, V, (T,), generator=gen).tolist()
        times = []
        for i in range(4):
            slot = engine.open(1)
            torch.cuda.synchronize()
            t = time.perf_counter()
            engine.step(slot, [prompt])
            host = time.perf_counter() - t      # every launch is made; the chip may still be working
            torch.cuda.synchronize()
            times.append((time.perf_counter() - t, host))
            engine.close(slot)
        del engine
        torch.cuda.empty_cache()
        return min(times[1:])

    pf, pf_host = run_prefill(n_prefill)
    if args.prefill_only:
        print(json.dumps({"metric": f"prefill tok/s at {n_prefill} tokens", "value": round(n_prefill / pf, 1),
                          "unit": "tok/s", "ms": round(pf * 1e3, 3), "host_ms": round(pf_host * 1e3, 3),
                          "layers": args.layers, "dtype": short,
                          "frac": round(prefill_flops(cfg, args.layers, n_prefill) / pf / PEAK_FLOPS[short], 4)}))
        return 0
    sec, mean_ctx, experts_used = run_decode(args.batch, args.context, args.steps, args.warmup)
    value = args.batch / sec
    read = decode_bytes(cfg, args.layers, args.batch, mean_ctx, wbytes, experts_used)
    achieved = read / sec / 1e9

    def point(b, ctx, s, mean, used):
        gb = decode_bytes(cfg, args.layers, b, mean, wbytes, used) / 1e9
        return {"tok_s": round(b / s, 1), "ms_per_step": round(s * 1e3, 4), "gb_per_step": round(gb, 2),
                "frac": round(gb / s / PEAK_HBM_GBS, 4)}

    # decode at batch 1 and 64 at the headline context, and every batch at the shorter context too
    points, detail = {}, {f"decode_b{args.batch}_ctx{args.context}": point(args.batch, args.context, sec, mean_ctx, experts_used)}
    if not args.no_points:
        for b in (1, 64):
            s, mean, used = run_decode(b, args.context, 32, 4)
            points[f"decode_b{b}"] = round(b / s, 1)
            detail[f"decode_b{b}_ctx{args.context}"] = point(b, args.context, s, mean, used)
        if args.points_context != args.context:
            for b in sorted({1, args.batch, 64}):
                s, mean, used = run_decode(b, args.points_context, 32, 4)
                detail[f"decode_b{b}_ctx{args.points_context}"] = point(b, args.points_context, s, mean, used)
    out = {
        "metric": f"decode tok/s at batch {args.batch}, context {args.context} ({model_name} layer sizes, random weights)",
        "value": round(value, 1), "unit": "tok/s", "n_gpus": 1, "steps": args.steps, "warmup": args.warmup,
        "ms_per_step": round(sec * 1e3, 4), "higher_is_better": True, "scaling": "weak", "vs_baseline": None,
        "dtype": short, "data": "synthetic",
        "config": {
            "model": f"{model_name} sizes", "layers": args.layers, "layers_of_full_model": full_layers,
            "hidden": cfg["hidden_size"], "heads": cfg["num_attention_heads"], "kv_heads": cfg["num_key_value_heads"],
            "head_dim": cfg["hidden_size"] // cfg["num_attention_heads"], "vocab": V, "experts": cfg["num_experts"],
            "top_k": cfg["num_experts_per_tok"], "expert_inner": cfg["moe_intermediate_size"],
            "shared_inner": cfg["shared_expert_intermediate_size"], "global_batch": args.batch,
            "seq_len": args.context, "parallelism": "single GPU", "points_context": args.points_context,
            "prefill_tokens": n_prefill, "weights": "random N(0,0.02) seed 2", "kv_cache": short,
            "experts_read_per_layer": round(experts_used, 1),
        },
        "prefill": {"value": round(n_prefill / pf, 1), "tokens": n_prefill, "ms": round(pf * 1e3, 3),
                    "frac": round(prefill_flops(cfg, args.layers, n_prefill) / pf / PEAK_FLOPS[short], 4),
                    "plain_products": plain_products(short)},
        "roofline": {"bound": "hbm", "achieved": round(achieved, 1), "peak": PEAK_HBM_GBS, "unit": "GB/s",
                     "frac": round(achieved / PEAK_HBM_GBS, 4)},
        "points": points,
        "points_detail": detail,
    }
    default_run = (args.sizes == "a27b" and act == "bfloat16" and args.layers == full_layers and not args.no_points
                   and not args.no_workloads)
    if default_run:
        # The two other stated workloads, each with a model of its own, once the headline model has left the device.
        # Whatever happens to them, the headline line is printed.
        import gc
        del model, run_decode, run_prefill
        gc.collect()
        torch.cuda.empty_cache()
        out["workloads"] = {}
        for name, sizes, dtype in (("a14b_bf16_unequal_b8", "a14b", "bfloat16"), ("a27b_fp32_unequal_b64", "a27b", "float32")):
            try:
                out["workloads"][name] = unequal_workload(sizes, dtype, None, unequal_defaults(sizes))
            except Exception as e:      # noqa: BLE001 - the record says what went wrong
                out["workloads"][name] = {"error": f"{type(e).__name__}: {e}"[:300]}
            gc.collect()
            torch.cuda.empty_cache()
    print(json.dumps(out), flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
