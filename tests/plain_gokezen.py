"""A plain, slow implementation of the Gokezen design: float64, whole sequences, no cache, one function per mechanism.

It is written from the design's formulas and shares nothing with the library; the library's logits are held against it.
``w`` maps tensor names to float64 arrays; a linear weight is [out, in] and applied as ``W x``.

embedding:    x = embed[token] + pos[position]
schedule:     the layers in order, except that layers start .. stop - 1 run ``times`` times in a row with the same weights
              (each pass over histories of its own); before pass t the vector loop.step[t] is added to x
A layer:      h = norm1(x);  x <- x + mixer(h) + ff(h)           (one norm, both halves read it; ff optional)
norm:         y / sqrt(mean(y^2) + eps) * weight
mixer:        left_scale * attention(h) + right_scale * matrix_memory(h)
attention:    q, k, v = W h (query head i with key head i // (heads / kv_heads)), score = q . k * scale for
              0 <= i - j < mask.size, softmax, W_o
memory:       q = W_q h dim^-1/2, k = W_k h, v = W_v h;  per head i = cap tanh((W_i h + b_i) / cap),
              f = logsigmoid(cap tanh((W_f h + b_f) / cap));  from m = 0, S = 0, n = 0, token by token
              m' = max(f + m, i);  S <- e^(f + m - m') S + e^(i - m') k v^T;  n likewise with k alone;
              o = S^T q / (max(|n . q|, e^(-m')) + 1e-6);  o / rms(o) per head, times a weight, times sigmoid(W_g h);  W_o
dense ff:     W_down (gelu_tanh(W_gate h) * (W_up h))
experts:      s = sigmoid(W_router h);  a group's score is the sum of its two largest s;  the ``top`` largest s within the
              ``keep`` best groups;  weights s / (their sum + 1e-20) * scale;  a shared expert for every token beside them
an expert:    g = min(W_gate h, limit), u = clamp(W_up h, -limit, limit), W_down (g sigmoid(1.702 g) (u + 1))
logits:       embed . norm(x)
"""
from __future__ import annotations

import math

import numpy as np


def rms_norm(y: np.ndarray, weight, eps: float) -> np.ndarray:
    out = y / np.sqrt(np.mean(y * y, axis=-1, keepdims=True) + eps)
    return out if weight is None else out * weight


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def log_sigmoid(z):
    return -np.logaddexp(0.0, -z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def masked_softmax(scores: np.ndarray, window: int | None) -> np.ndarray:
    """scores [T, T]: row i sees columns j <= i, and with a window only those with i - j < window."""
    T = scores.shape[0]
    out = np.zeros_like(scores)
    for i in range(T):
        lo = 0 if window is None else max(0, i - window + 1)
        row = scores[i, lo:i + 1]
        e = np.exp(row - row.max())
        out[i, lo:i + 1] = e / e.sum()
    return out


def attention(h: np.ndarray, m: dict, w: dict, p: str) -> np.ndarray:
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].T).reshape(T, H, D)
    k = (h @ w[p + "k"].T).reshape(T, G, D)
    v = (h @ w[p + "v"].T).reshape(T, G, V)
    window = m["mask"]["size"] if m.get("mask") is not None else None
    out = np.zeros((T, H, V))
    for head in range(H):
        g = head // (H // G)
        out[:, head] = masked_softmax(q[:, head] @ k[:, g].T * m["scale"], window) @ v[:, g]
    return out.reshape(T, H * V) @ w[p + "o"].T


def memory_gates(h: np.ndarray, m: dict, w: dict, p: str):
    """The logarithms of the input and of the forget gate, [T, heads] each."""
    cap = m["gate_cap"]
    i = cap * np.tanh((h @ w[p + "i"].T + w[p + "i.b"]) / cap)
    f = log_sigmoid(cap * np.tanh((h @ w[p + "f"].T + w[p + "f.b"]) / cap))
    return i, f


def memory_scan(q, k, v, i, f, state=None):
    """q (scaled), k [T, heads, D], v [T, heads, V], gates [T, heads]; ``state``: (S [heads, D, V], n [heads, D], m [heads]).
    Returns the read-outs [T, heads, V] and the state behind the last token."""
    T, H, D = q.shape
    V = v.shape[2]
    S, n, mx = (np.zeros((H, D, V)), np.zeros((H, D)), np.zeros(H)) if state is None else tuple(a.copy() for a in state)
    o = np.zeros((T, H, V))
    for t in range(T):
        for head in range(H):
            new = max(f[t, head] + mx[head], i[t, head])
            keep, add = math.exp(f[t, head] + mx[head] - new), math.exp(i[t, head] - new)
            S[head] = keep * S[head] + add * np.outer(k[t, head], v[t, head])
            n[head] = keep * n[head] + add * k[t, head]
            mx[head] = new
            o[t, head] = S[head].T @ q[t, head] / (max(abs(n[head] @ q[t, head]), math.exp(-new)) + 1e-6)
    return o, (S, n, mx)


def matrix_memory(h: np.ndarray, m: dict, w: dict, p: str, eps: float, state=None, return_state: bool = False):
    T = h.shape[0]
    H, D, V = m["heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].T).reshape(T, H, D) * D ** -0.5
    k = (h @ w[p + "k"].T).reshape(T, H, D)
    v = (h @ w[p + "v"].T).reshape(T, H, V)
    i, f = memory_gates(h, m, w, p)
    o, states = memory_scan(q, k, v, i, f, state)
    o = rms_norm(o, None, eps).reshape(T, H * V) * w[p + "norm"] * sigmoid(h @ w[p + "g"].T)
    out = o @ w[p + "o"].T
    return (out, states) if return_state else out


def mixer(h: np.ndarray, m: dict, w: dict, p: str, eps: float) -> np.ndarray:
    return (m["left_scale"] * attention(h, m["left"], w, p + "left.")
            + m["right_scale"] * matrix_memory(h, m["right"], w, p + "right.", eps))


def dense_ff(h: np.ndarray, w: dict, p: str) -> np.ndarray:
    return (gelu_tanh(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def choose(s: np.ndarray, r: dict, margins: list | None = None):
    """scores [T, experts] -> the chosen experts [T, top] (best first) and their weights; how clear the choices were is
    appended to ``margins``."""
    T, E = s.shape
    top, groups = r["top"], r.get("groups")
    allowed = np.ones((T, E), dtype=bool)
    if groups is not None:
        per = E // groups["count"]
        by_group = np.sort(s.reshape(T, groups["count"], per), axis=-1)[:, :, -2:].sum(-1)
        best = np.argsort(-by_group, axis=-1, kind="stable")[:, :groups["keep"]]
        kept = np.zeros((T, groups["count"]), dtype=bool)
        np.put_along_axis(kept, best, True, axis=-1)
        allowed = np.repeat(kept, per, axis=-1)
    ids = np.argsort(np.where(allowed, -s, np.inf), axis=-1, kind="stable")[:, :top]
    chosen = np.take_along_axis(s, ids, axis=-1)
    if margins is not None:      # by how much the last chosen group and expert were ahead of the first left out
        def ahead(scores, n):
            order = np.sort(scores, axis=-1)[:, ::-1]
            return order[:, n - 1] - order[:, n] if n < scores.shape[1] else np.full(T, np.inf)
        margins.append(ahead(np.where(allowed, s, -np.inf), top))
        if groups is not None:
            margins.append(ahead(by_group, groups["keep"]))
    return ids, chosen / (chosen.sum(-1, keepdims=True) + 1e-20) * r["scale"]


def expert(h: np.ndarray, w: dict, p: str, limit: float) -> np.ndarray:
    g = np.minimum(h @ w[p + "gate"].T, limit)
    u = np.clip(h @ w[p + "up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w[p + "down"].T


def experts_ff(h: np.ndarray, f: dict, w: dict, p: str, margins: list | None = None) -> np.ndarray:
    ids, weights = choose(sigmoid(h @ w[p + "router"].T), f["router"], margins)
    out = np.zeros((h.shape[0], w[p + "e0.down"].shape[0]))
    for t in range(h.shape[0]):
        for e, wt in zip(ids[t], weights[t]):
            out[t] += wt * expert(h[t:t + 1], w, f"{p}e{e}.", f["expert"]["limit"])[0]
    if f.get("shared") is not None:
        out += expert(h, w, p + "shared.", f["shared"]["limit"])
    return out


def runs(cfg: dict) -> list[tuple[int, int | None]]:
    """The layer runs in order: (layer, number of the loop's pass that starts with this run, or None)."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if loop is None:
        return [(i, None) for i in range(n)]
    out = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        out += [(i, t if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
    return out + [(i, None) for i in range(loop["stop"], n)]


def forward(cfg: dict, w: dict, tokens, return_layers: bool = False, return_margins: bool = False):
    """Logits [T, vocab] of a whole sequence (and the residual stream behind every layer run, or per token the smallest margin
    by which any of its choices of experts was made)."""
    eps = cfg["norm"]["eps"]
    x = w["embed"][np.asarray(tokens)] + w["pos"][:len(tokens)]
    streams, margins = [], [np.full(len(tokens), np.inf)]
    for i, step in runs(cfg):
        layer = cfg["layers"][i]
        if step is not None:
            x = x + w["loop.step"][step]
        h = rms_norm(x, w[f"l{i}.norm1"], eps)
        y = mixer(h, layer["mixer"], w, f"l{i}.mix.", eps)
        f = layer.get("mlp")
        if f is not None:
            y = y + (dense_ff(h, w, f"l{i}.mlp.") if f["kind"] == "dense" else experts_ff(h, f, w, f"l{i}.mlp.", margins))
        x = x + y
        streams.append(x.copy())
    logits = rms_norm(x, w["final.norm"], eps) @ w["embed"].T
    if return_margins:
        return logits, np.min(margins, axis=0)
    return (logits, streams) if return_layers else logits
