"""A plain, slow implementation of the Pumozen design: float64, whole sequences, no cache, one function per mechanism.

It is written from the design's formulas and shares nothing with the library; the library's logits are held against it.
``w`` maps tensor names to float64 arrays; a linear weight is [out, in] and applied as ``W x``.

embedding:    x = embed[token]
A layer:      x <- x + ln1(mixer(x));  x <- x + ln2(ff(x)) (ff optional);  then the token's own input:
              e = side.embed[token, i dim : (i + 1) dim],  y = W_proj (gelu_tanh(W_gate x) * e),  x <- x + y / rms(y) * weight
ln:           (y - mean) / sqrt(mean((y - mean)^2) + eps) * weight + bias
attention:    q = W_q h, k = W_k h, v = k;  q / rms(q) * w over all of q's rows together, k alike;  rotation of the first
              rot.dims numbers of a head, number i with i + dims / 2, by p base^(-2 i / dims);  score = q . k * scale;
              weights exp(s_j) / (1 + sum exp(s_j)) over j <= i;  W_o
attention_2:  two maps a head: q, k [heads, 2, dim], each divided by its root mean square over dim, times a weight;
              q times 1 + coef ln(floor((p + 1) / every) + 1);  softmax of q . k * scale per map over the same values;
              o = a1 - lambda a2,  lambda = exp(lq1 . lk1) - exp(lq2 . lk2) + diff;  o / rms(o) * (1 - diff) per head;
              times sigmoid(W_g h);  W_o.  With kv_from the keys and values are those of that layer
mamba2:       W_in h = [z | x | B | C | dt];  x, B, C through a causal convolution with bias and silu;
              dt = softplus(dt + bias);  S <- exp(-exp(A_log) dt) S + dt B x^T,  y = S^T C + D x per head;
              y silu(z), divided by its root mean square in norm_groups equal parts, times a weight;  W_o
pair:         g = min(W_gate h, limit), u = clamp(W_up h, -limit, limit), W_down (g sigmoid(1.702 g) (u + 1))
dense ff:     a pair
experts:      s = softmax(W_router h);  the ``top`` largest;  weights s / (their sum + 1e-20) * scale;  every expert a pair;
              a shared pair for every token beside them, times sigmoid(W_sg h)
logits:       embed . ln(x)
"""
from __future__ import annotations

import math

import numpy as np


def rms_norm(y: np.ndarray, weight, eps: float) -> np.ndarray:
    out = y / np.sqrt(np.mean(y * y, axis=-1, keepdims=True) + eps)
    return out if weight is None else out * weight


def layer_norm(y: np.ndarray, weight, bias, eps: float) -> np.ndarray:
    c = y - np.mean(y, axis=-1, keepdims=True)
    return c / np.sqrt(np.mean(c * c, axis=-1, keepdims=True) + eps) * weight + bias


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def causal_softmax(scores: np.ndarray, sink: bool) -> np.ndarray:
    """scores [T, T]: row i over columns j <= i; with ``sink`` the denominator also holds exp(0)."""
    out = np.zeros_like(scores)
    for i in range(scores.shape[0]):
        row = scores[i, :i + 1]
        top = max(row.max(), 0.0) if sink else row.max()
        e = np.exp(row - top)
        out[i, :i + 1] = e / (e.sum() + (math.exp(-top) if sink else 0.0))
    return out


def rotate(x: np.ndarray, rot: dict | None) -> np.ndarray:
    """x [T, heads, dim], token t at position t."""
    if rot is None:
        return x
    n = rot["dims"] // 2
    a = np.arange(x.shape[0])[:, None] * rot["base"] ** (-2.0 * np.arange(n) / rot["dims"])
    cos, sin = np.cos(a)[:, None, :], np.sin(a)[:, None, :]
    u, v = x[..., :n], x[..., n:2 * n]
    return np.concatenate([u * cos - v * sin, v * cos + u * sin, x[..., 2 * n:]], axis=-1)


def attention_kv(h: np.ndarray, m: dict, w: dict, p: str, eps: float):
    T, G, D = h.shape[0], m["kv_heads"], m["dim"]
    raw = h @ w[p + "k"].T
    return rotate(rms_norm(raw, w[p + "k.norm"], eps).reshape(T, G, D), m.get("rot")), raw.reshape(T, G, D)


def attention(h: np.ndarray, m: dict, w: dict, p: str, eps: float, kv) -> np.ndarray:
    T, H, G, D = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q = rotate(rms_norm(h @ w[p + "q"].T, w[p + "q.norm"], eps).reshape(T, H, D), m.get("rot"))
    k, v = kv
    out = np.zeros((T, H, D))
    for head in range(H):
        g = head // (H // G)
        out[:, head] = causal_softmax(q[:, head] @ k[:, g].T * m["scale"], True) @ v[:, g]
    return out.reshape(T, H * D) @ w[p + "o"].T


def temperature(T: int, t: dict | None) -> np.ndarray:
    if t is None:
        return np.ones(T)
    return 1.0 + t["coef"] * np.log(np.floor((np.arange(T) + 1) / t["every"]) + 1.0)


def differential_kv(h: np.ndarray, m: dict, w: dict, p: str, eps: float):
    T, G, D = h.shape[0], m["kv_heads"], m["dim"]
    k = rms_norm((h @ w[p + "k"].T).reshape(T, G, 2, D), w[p + "k.norm"], eps)
    return k, (h @ w[p + "v"].T).reshape(T, G, m["vdim"])


def lam(m: dict, w: dict, p: str) -> float:
    return float(np.exp(w[p + "lq1"] @ w[p + "lk1"]) - np.exp(w[p + "lq2"] @ w[p + "lk2"]) + m["diff"])


def differential_attention(h: np.ndarray, m: dict, w: dict, p: str, eps: float, kv) -> np.ndarray:
    T, H, G, D, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_norm((h @ w[p + "q"].T).reshape(T, H, 2, D), w[p + "q.norm"], eps)
    q = q * temperature(T, m.get("q_temp"))[:, None, None, None]
    k, v = kv
    lm = lam(m, w, p)
    out = np.zeros((T, H, V))
    for head in range(H):
        g = head // (H // G)
        a1, a2 = (causal_softmax(q[:, head, i] @ k[:, g, i].T * m["scale"], False) @ v[:, g] for i in range(2))
        out[:, head] = rms_norm(a1 - lm * a2, None, eps) * (1.0 - m["diff"])
    return (out.reshape(T, H * V) * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def short_convolution(x: np.ndarray, weight: np.ndarray, bias: np.ndarray, before: np.ndarray | None = None) -> np.ndarray:
    """x [T, channels], weight [channels, taps], the last tap the current token's; ``before`` [taps - 1, channels]: the inputs
    ahead of the first row (zeros for None)."""
    taps = weight.shape[1]
    if before is None:
        before = np.zeros((taps - 1, x.shape[1]))
    full = np.concatenate([before, x])
    return sum(full[j:j + x.shape[0]] * weight[:, j] for j in range(taps)) + bias


def ssd_scan(x, B, C, dt, a_log, D, state=None):
    """x [T, heads, V], B and C [T, groups, N], dt [T, heads] (behind softplus).  Returns y and the states [heads, N, V]."""
    T, H, V = x.shape
    G, N = B.shape[1:]
    S = np.zeros((H, N, V)) if state is None else state.copy()
    y = np.zeros((T, H, V))
    for t in range(T):
        for head in range(H):
            g = head // (H // G)
            S[head] = math.exp(-math.exp(a_log[head]) * dt[t, head]) * S[head] + dt[t, head] * np.outer(B[t, g], x[t, head])
            y[t, head] = S[head].T @ C[t, g] + D[head] * x[t, head]
    return y, S


def mamba2(h: np.ndarray, m: dict, w: dict, p: str, eps: float) -> np.ndarray:
    T, H, V, N, G = h.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * V
    proj = h @ w[p + "in"].T
    z, xbc, dt = proj[:, :inner], proj[:, inner:2 * inner + 2 * G * N], proj[:, 2 * inner + 2 * G * N:]
    xbc = silu(short_convolution(xbc, w[p + "conv"], w[p + "conv.b"]))
    x = xbc[:, :inner].reshape(T, H, V)
    B = xbc[:, inner:inner + G * N].reshape(T, G, N)
    C = xbc[:, inner + G * N:].reshape(T, G, N)
    y, _ = ssd_scan(x, B, C, softplus(dt + w[p + "dt_bias"]), w[p + "A_log"], w[p + "D"])
    y = (y.reshape(T, inner) * silu(z)).reshape(T, m["norm_groups"], inner // m["norm_groups"])
    return (rms_norm(y, None, eps).reshape(T, inner) * w[p + "norm"]) @ w[p + "o"].T


def pair(h: np.ndarray, w: dict, p: str, limit: float) -> np.ndarray:
    g = np.minimum(h @ w[p + "gate"].T, limit)
    u = np.clip(h @ w[p + "up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w[p + "down"].T


def choose(z: np.ndarray, r: dict, margins: list | None = None):
    """Router logits [T, experts] -> the chosen experts [T, top] (best first) and their weights; by how much the last one
    chosen was ahead of the first left out is appended to ``margins``."""
    s = np.exp(z - z.max(-1, keepdims=True))
    s = s / s.sum(-1, keepdims=True)
    ids = np.argsort(-s, axis=-1, kind="stable")[:, :r["top"]]
    chosen = np.take_along_axis(s, ids, axis=-1)
    if margins is not None and r["top"] < z.shape[1]:
        order = np.sort(z, axis=-1)[:, ::-1]
        margins.append(order[:, r["top"] - 1] - order[:, r["top"]])
    return ids, chosen / (chosen.sum(-1, keepdims=True) + 1e-20) * r["scale"]


def experts_ff(h: np.ndarray, f: dict, w: dict, p: str, margins: list | None = None) -> np.ndarray:
    ids, weights = choose(h @ w[p + "router"].T, f["router"], margins)
    out = np.zeros((h.shape[0], w[p + "e0.down"].shape[0]))
    for t in range(h.shape[0]):
        for e, wt in zip(ids[t], weights[t]):
            out[t] += wt * pair(h[t:t + 1], w, f"{p}e{e}.", f["expert"]["limit"])[0]
    if f.get("shared") is not None:
        out += sigmoid(h @ w[p + "shared.sg"].T) * pair(h, w, p + "shared.", f["shared"]["limit"])
    return out


def token_side(x: np.ndarray, tokens, i: int, dim: int, w: dict, eps: float) -> np.ndarray:
    e = w["side.embed"][np.asarray(tokens), i * dim:(i + 1) * dim]
    y = (gelu_tanh(x @ w[f"l{i}.side.gate"].T) * e) @ w[f"l{i}.side.proj"].T
    return x + rms_norm(y, w[f"l{i}.side.norm"], eps)


def forward(cfg: dict, w: dict, tokens, return_layers: bool = False, return_margins: bool = False):
    """Logits [T, vocab] of a whole sequence (and the residual stream behind every layer, or per token the smallest margin by
    which any of its choices of experts was made)."""
    eps = cfg["norm"]["eps"]
    x = w["embed"][np.asarray(tokens)]
    streams, margins, kept = [], [np.full(len(tokens), np.inf)], {}
    for i, layer in enumerate(cfg["layers"]):
        m, f, p = layer["mixer"], layer.get("mlp"), f"l{i}."
        if layer["type"] == "mamba2":
            y = mamba2(x, m, w, p + "mix.", eps)
        else:
            make, mix = ((attention_kv, attention) if layer["type"] == "attention" else (differential_kv, differential_attention))
            kept[i] = kept[m["kv_from"]] if m.get("kv_from") is not None else make(x, m, w, p + "mix.", eps)
            y = mix(x, m, w, p + "mix.", eps, kept[i])
        x = x + layer_norm(y, w[p + "norm1"], w[p + "norm1.b"], eps)
        if f is not None:
            y = pair(x, w, p + "mlp.", f["limit"]) if f["kind"] == "dense" else experts_ff(x, f, w, p + "mlp.", margins)
            x = x + layer_norm(y, w[p + "norm2"], w[p + "norm2.b"], eps)
        if cfg.get("token_side") is not None:
            x = token_side(x, tokens, i, cfg["token_side"]["dim"], w, eps)
        streams.append(x.copy())
    logits = layer_norm(x, w["final.norm"], w["final.norm.b"], eps) @ w["embed"].T
    if return_margins:
        return logits, np.min(margins, axis=0)
    return (logits, streams) if return_layers else logits
