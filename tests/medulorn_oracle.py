"""Plain restatement of the Medulorn design in numpy float64: one function per mechanism, whole sequences from position 0, one query
at a time.  It shares no code with the product: the tests compare the HIP path with it.

Weights are a dict {checkpoint tensor name: array}, every matrix [out, in] and applied as W x; the configuration is the parsed
config.json.
"""
from __future__ import annotations

import numpy as np


def sigmoid(z):
    e = np.exp(-np.abs(z))
    return np.where(z >= 0, 1.0 / (1.0 + e), e / (1.0 + e))


def silu(z):
    return z * sigmoid(z)


def unit_rms(x, eps):
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps)


def scalar_norm(x, g, eps):
    """One weight for all coordinates."""
    return unit_rms(x, eps) * float(np.asarray(g).reshape(()))


def token_shift(h, mu):
    before = np.vstack([np.zeros_like(h[:1]), h[:-1]])
    return h + (before - h) * mu


def frequencies(rot):
    """Turns per position of every pair; wavelengths beyond what a model was made for are stretched (Llama 3.1)."""
    f = rot["base"] ** (-2.0 * np.arange(rot["dims"] // 2) / rot["dims"])
    sc = rot.get("scaling")
    if not sc:
        return f
    out = np.empty_like(f)
    for i, v in enumerate(f):
        wave = 2.0 * np.pi / v
        if wave < sc["original"] / sc["high"]:
            out[i] = v
        elif wave > sc["original"] / sc["low"]:
            out[i] = v / sc["factor"]
        else:
            s = (sc["original"] / wave - sc["low"]) / (sc["high"] - sc["low"])
            out[i] = (1.0 - s) * v / sc["factor"] + s * v
    return out


def rotated(x, rot):
    """x [T, heads, dim]: the first rot.dims dimensions of every head turn, pairs (i, i + dims / 2)."""
    if not rot:
        return x
    half = rot["dims"] // 2
    a = (np.arange(x.shape[0])[:, None] * frequencies(rot)[None, :])[:, None, :]
    u, v = x[..., :half], x[..., half:2 * half]
    return np.concatenate([u * np.cos(a) - v * np.sin(a), v * np.cos(a) + u * np.sin(a), x[..., 2 * half:]], axis=-1)


def chunk_keys(i, mask):
    return np.arange(i // mask["size"] * mask["size"], i + 1)


def window_keys(i, mask):
    j = np.arange(i + 1)
    return j[(i - j < mask["size"]) | (j < mask.get("keep_first", 0))]


def sink_softmax(s, sink):
    """s [heads, keys]; sink [heads]: the score of an entry that takes part in the denominator only."""
    m = np.maximum(s.max(axis=1), sink)[:, None]
    e = np.exp(s - m)
    return e / (np.exp(sink[:, None] - m) + e.sum(axis=1, keepdims=True))


def grouped_attention(q, k, v, scale, keys, sink):
    """q [T, H, dim], k [T, G, dim], v [T, G, vdim]; keys(i): the places query i sees."""
    T, H, _ = q.shape
    share = np.arange(H) // (H // k.shape[1])
    out = np.empty((T, H, v.shape[2]))
    for i in range(T):
        j = keys(i)
        p = sink_softmax(np.einsum("hd,jhd->hj", q[i], k[j][:, share]) * scale, sink)
        out[i] = np.einsum("hj,jhd->hd", p, v[j][:, share])
    return out


def chunked_attention(h, w, mx, eps):
    """Biased projections, norms per head, chunks, and a one in the softmax's denominator."""
    T, H, G = h.shape[0], mx["heads"], mx["kv_heads"]
    q, k, v = (h @ w[n].T + w[n + ".b"] for n in "qkv")
    q = unit_rms(q.reshape(T, H, -1), eps) * w["q.norm"]
    k = unit_rms(k.reshape(T, G, -1), eps) * w["k.norm"]
    mask = mx.get("mask")
    keys = (lambda i: chunk_keys(i, mask)) if mask else (lambda i: np.arange(i + 1))
    o = grouped_attention(rotated(q, mx.get("rot")), rotated(k, mx.get("rot")), v.reshape(T, G, -1), mx["scale"], keys, np.zeros(H))
    return o.reshape(T, -1) @ w["o"].T


def window_attention(h, w, mx, eps):
    """Norms over the whole projections, a window beside kept first tokens, and a learned sink per head."""
    T, H, G = h.shape[0], mx["heads"], mx["kv_heads"]
    q = unit_rms(h @ w["q"].T, eps) * w["q.norm"]
    k = unit_rms(h @ w["k"].T, eps) * w["k.norm"]
    mask = mx.get("mask")
    keys = (lambda i: window_keys(i, mask)) if mask else (lambda i: np.arange(i + 1))
    o = grouped_attention(rotated(q.reshape(T, H, -1), mx.get("rot")), rotated(k.reshape(T, G, -1), mx.get("rot")), (h @ w["v"].T).reshape(T, G, -1),
                          mx["scale"], keys, w["sink"])
    return o.reshape(T, -1) @ w["o"].T


def lightning(q, k, v, decay):
    """q, k [T, H, dim], v [T, H, vdim]: S <- decay S + k v^T, o = S^T q."""
    T, H, D = q.shape
    S, out = np.zeros((H, D, v.shape[2])), np.empty((T, H, v.shape[2]))
    for t in range(T):
        S = np.asarray(decay)[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = np.einsum("hd,hdv->hv", q[t], S)
    return out


def lightning_mixer(h, w, mx, eps):
    T, H = h.shape[0], mx["heads"]
    q, k, v = (silu(h @ w[n].T).reshape(T, H, -1) for n in "qkv")
    o = lightning(q, k, v, mx["decay"]).reshape(T, -1)
    return (unit_rms(o, eps) * w["norm"] * sigmoid(h @ w["g"].T)) @ w["o"].T


def mixer(h, w, ly, eps):
    mx = ly["mixer"]
    if ly["type"] == "attention":
        return chunked_attention(h, w, mx, eps)
    return mx["left_scale"] * window_attention(h, sub(w, "left."), mx["left"], eps) + mx["right_scale"] * lightning_mixer(h, sub(w, "right."), mx["right"], eps)


def relu_glu(h, w):
    return (np.maximum(h @ w["gate"].T, 0.0) * (h @ w["up"].T)) @ w["down"].T


def clamped_glu(h, w, name, limit):
    g = np.minimum(h @ w[name + ".gate"].T, limit)
    u = np.clip(h @ w[name + ".up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w[name + ".down"].T


def choose(z, top):
    """The chosen experts of one token, best first, their weights, and how close the call was."""
    order = np.argsort(-z, kind="stable")
    e = np.exp(z[order[:top]] - z[order[0]])
    return order[:top], e / e.sum(), z[order[top - 1]] - z[order[top]] if top < z.size else np.inf


def experts(h, w, mlp, margins=None):
    z = h @ w["router"].T + w["router.b"]
    out, gaps = np.zeros_like(h), np.empty(h.shape[0])
    for t in range(h.shape[0]):
        chosen, weight, gaps[t] = choose(z[t], mlp["router"]["top"])
        for e, p in zip(chosen, weight):
            out[t] += p * clamped_glu(h[t], w, f"e{e}", mlp["expert"]["limit"])
    if margins is not None:
        margins.append(gaps)
    return out if mlp.get("shared") is None else out + clamped_glu(h, w, "shared", mlp["shared"]["limit"])


def feed_forward(h, w, mlp, margins=None):
    return relu_glu(h, w) if mlp["kind"] == "dense" else experts(h, w, mlp, margins)


def capped(z, cap):
    return cap * np.tanh(z / cap) if cap else z


def sub(weights, prefix):
    return {k[len(prefix):]: np.asarray(v, np.float64) for k, v in weights.items() if k.startswith(prefix)}


def forward(cfg, weights, tokens, return_layers=False, margins=None):
    """Logits [T, vocab] of one sequence (and the residual stream after every layer [layers, T, width]).  margins: a list that gets, for
    every layer with experts, how close each token's choice was."""
    eps, tok, alpha = cfg["norm"]["eps"], np.asarray(tokens), cfg["postln_alpha"]
    x = np.asarray(weights["embed"], np.float64)[tok] * cfg["embedding"]["scale"]
    layers = []
    for i, ly in enumerate(cfg["layers"]):
        w = sub(weights, f"l{i}.")
        x = scalar_norm(alpha * x + mixer(token_shift(x, w["shift"]), sub(w, "mix."), ly, eps), w["norm1"], eps)
        if ly["mlp"] is not None:
            x = scalar_norm(alpha * x + feed_forward(x, sub(w, "mlp."), ly["mlp"], margins), w["norm2"], eps)
        layers.append(x)
    logits = capped(scalar_norm(x, weights["final.norm"], eps) @ np.asarray(weights["head"], np.float64).T, cfg.get("logit_softcap"))
    return (logits, np.stack(layers)) if return_layers else logits
