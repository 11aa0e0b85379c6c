"""Plain restatement of the Bolinex design in numpy float64: one function per mechanism, whole sequences from position 0, one query
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


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def rms_norm(x, w, eps):
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps) * w


def layer_norm(x, w, b, eps):
    d = x - x.mean(axis=-1, keepdims=True)
    return d / np.sqrt((d * d).mean(axis=-1, keepdims=True) + eps) * w + b


def distance_bias(r1, r2, back):
    """What every head takes off the score of a key `back` tokens before the query: [heads, keys]."""
    return r1[:, None] * np.log1p(r2[:, None] * back[None, :])


def capped(s, cap):
    return s if cap is None else cap * np.tanh(s / cap)


def grouped_attention(q, k, v, mx, r1, r2):
    """q [T, H, dim], k [T, G, dim], v [T, G, vdim]; row i sees the window that ends with itself."""
    T, H, _ = q.shape
    share = np.arange(H) // (H // k.shape[1])
    window = T if mx.get("mask") is None else mx["mask"]["size"]
    out = np.empty((T, H, v.shape[2]))
    for i in range(T):
        j = np.arange(max(0, i - window + 1), i + 1)
        s = capped(np.einsum("hd,jhd->hj", q[i], k[j][:, share]) * mx["scale"], mx.get("softcap")) - distance_bias(r1, r2, i - j)
        p = np.exp(s - s.max(axis=1, keepdims=True))
        out[i] = np.einsum("hj,jhd->hd", p / p.sum(axis=1, keepdims=True), v[j][:, share])
    return out


def mixed_values(v, first, lam):
    return v if first is None else (1.0 - lam) * v + lam * first


def attention(h, w, mx, first):
    """Returns the mixer's output and the layer's own values (before mixing)."""
    T, H, G = h.shape[0], mx["heads"], mx["kv_heads"]
    v = h @ w["v"].T
    mixed = mixed_values(v, first, float(w["vmix"])) if mx.get("v_mix") else v
    o = grouped_attention((h @ w["q"].T).reshape(T, H, -1), (h @ w["k"].T).reshape(T, G, -1), mixed.reshape(T, G, -1), mx, w["r1"], w["r2"])
    return (o.reshape(T, -1) * sigmoid(h @ w["g"].T)) @ w["o"].T, v


def squared_relu_ff(h, up, down):
    return np.maximum(h @ up.T, 0.0) ** 2 @ down.T


def gated_ff(h, w, name):
    return (silu(h @ w[name + ".gate"].T) * (h @ w[name + ".up"].T)) @ w[name + ".down"].T


def group_scores(choice, groups):
    return np.sort(choice.reshape(groups["count"], -1), axis=1)[:, -2:].sum(axis=1)


def choose(choice, router):
    """The chosen experts of one token, best first, and how close the call was (the smallest gap that decided something)."""
    gr, E = router.get("groups"), router["experts"]
    ok, gap = np.ones(E, bool), np.inf
    if gr is not None:
        score = group_scores(choice, gr)
        order = np.argsort(-score, kind="stable")
        ok = np.repeat(np.isin(np.arange(gr["count"]), order[:gr["keep"]]), E // gr["count"])
        if gr["keep"] < gr["count"]:
            gap = score[order[gr["keep"] - 1]] - score[order[gr["keep"]]]
    c = np.where(ok, choice, -np.inf)
    order = np.argsort(-c, kind="stable")
    if router["top"] < ok.sum():
        gap = min(gap, c[order[router["top"] - 1]] - c[order[router["top"]]])
    return order[:router["top"]], gap


def experts(h, w, mlp, margins=None):
    s = sigmoid(h @ w["router"].T)
    out, gaps = np.zeros_like(h), np.empty(h.shape[0])
    for t in range(h.shape[0]):
        chosen, gaps[t] = choose(s[t] + w["correction"], mlp["router"])
        for e in chosen:
            out[t] += s[t, e] * gated_ff(h[t], w, f"e{e}")
    if margins is not None:
        margins.append(gaps)
    return out if mlp.get("shared") is None else out + gated_ff(h, w, "shared")


def feed_forward(h, w, mlp, margins=None):
    if mlp is None:
        return 0.0
    return squared_relu_ff(h, w["up"], w["down"]) if mlp["kind"] == "dense" else experts(h, w, mlp, margins)


def token_side(x, e, w, eps):
    return rms_norm((gelu_tanh(x @ w["gate"].T) * e) @ w["proj"].T, w["norm"], eps)


def sub(weights, prefix):
    return {k[len(prefix):]: np.asarray(v, np.float64) for k, v in weights.items() if k.startswith(prefix)}


def forward(cfg, weights, tokens, return_layers=False, margins=None):
    """Logits [T, vocab] of one sequence (and the residual stream after every layer [layers, T, width]).  margins: a list that gets, for
    every layer with experts, how close each token's choice was."""
    eps, tok = cfg["norm"]["eps"], np.asarray(tokens)
    x = np.asarray(weights["embed"], np.float64)[tok] + np.asarray(weights["pos"], np.float64)[:len(tok)]
    layers, first = [], None
    for i, ly in enumerate(cfg["layers"]):
        w = sub(weights, f"l{i}.")
        h = layer_norm(x, w["norm1"], w["norm1.b"], eps)
        y, v = attention(h, sub(weights, f"l{i}.mix."), ly["mixer"], first)
        if ly["mixer"].get("v_mix") and first is None:
            first = v
        x = x + (y + feed_forward(h, sub(weights, f"l{i}.mlp."), ly["mlp"], margins))
        if cfg.get("token_side"):
            n = cfg["token_side"]["dim"]
            x = x + token_side(x, np.asarray(weights["side.embed"], np.float64)[tok, i * n:(i + 1) * n], sub(weights, f"l{i}.side."), eps)
        layers.append(x)
    logits = layer_norm(x, *(np.asarray(weights["final.norm" + b], np.float64) for b in ("", ".b")), eps) @ np.asarray(weights["head"], np.float64).T
    return (logits, np.stack(layers)) if return_layers else logits
