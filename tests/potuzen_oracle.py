"""Plain restatement of the Potuzen design in numpy float64: one function per mechanism, whole sequences from position 0,
token by token where the mechanism is a recurrence.  It shares no code with the product: the tests compare the HIP path with it.

Weights are a dict {checkpoint tensor name: array}, every matrix [out, in] and applied as W x; the configuration is the parsed
config.json.
"""
from __future__ import annotations

import numpy as np


def sigmoid(z):
    return np.where(z >= 0, 1.0 / (1.0 + np.exp(-np.abs(z))), np.exp(-np.abs(z)) / (1.0 + np.exp(-np.abs(z))))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.maximum(z, 0.0) + np.log1p(np.exp(-np.abs(z)))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def rms(x, eps):
    """x over its own root mean square (last axis), eps under the root."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def rms_norm(x, w, eps):
    return rms(x, eps) * w


def gated_mlp(h, gate, up, down):
    return (gelu_tanh(h @ gate.T) * (h @ up.T)) @ down.T


def windowed_softmax_attention(q, k, v, scale, window):
    """q, k [T, heads, dim], v [T, heads, vdim]: query i sees keys i - window + 1 .. i."""
    T = q.shape[0]
    out = np.empty(v.shape)
    for i in range(T):
        lo = max(0, i - window + 1)
        s = np.einsum("hd,jhd->hj", q[i], k[lo:i + 1]) * scale
        p = np.exp(s - s.max(axis=1, keepdims=True))
        p /= p.sum(axis=1, keepdims=True)
        out[i] = np.einsum("hj,jhd->hd", p, v[lo:i + 1])
    return out


def latent_attention(h, w, mx, eps):
    T, H, d, dv = h.shape[0], mx["heads"], mx["dim"], mx["vdim"]
    cq = rms_norm(h @ w["dq"].T, w["dq.norm"], eps)
    c = rms_norm(h @ w["dkv"].T, w["dkv.norm"], eps)
    q = (cq @ w["uq"].T).reshape(T, H, d)
    k = (c @ w["uk"].T).reshape(T, H, d)
    v = (c @ w["uv"].T).reshape(T, H, dv)
    o = windowed_softmax_attention(q, k, v, mx["scale"], mx["mask"]["size"]).reshape(T, H * dv)
    return (o * sigmoid(h @ w["g"].T)) @ w["o"].T


def causal_conv(x, w, b):
    """Per channel: w [channels, taps], the last tap is the current token's; zeros before the sequence."""
    T, taps = x.shape[0], w.shape[1]
    xp = np.concatenate([np.zeros((taps - 1, x.shape[1])), x])
    return sum(xp[i:i + T] * w[:, i] for i in range(taps)) + b


def ssd_recurrence(x, B, C, dt, A_log, D):
    """x [T, heads, vdim], B / C [T, groups, N], dt [T, heads] (after softplus): y [T, heads, vdim]."""
    T, H, P = x.shape
    per = H // B.shape[1]
    S = np.zeros((H, B.shape[2], P))
    y = np.empty(x.shape)
    for t in range(T):
        for hd in range(H):
            g = hd // per
            S[hd] = np.exp(-np.exp(A_log[hd]) * dt[t, hd]) * S[hd] + dt[t, hd] * np.outer(B[t, g], x[t, hd])
            y[t, hd] = S[hd].T @ C[t, g] + D[hd] * x[t, hd]
    return y


def grouped_rms(y, groups, eps):
    T, n = y.shape
    return rms(y.reshape(T, groups, n // groups), eps).reshape(T, n)


def mamba2(h, w, mx, eps):
    T, H, P, N, G = h.shape[0], mx["heads"], mx["vdim"], mx["state"], mx["groups"]
    inner = H * P
    z, xbc, dt = np.split(h @ w["in"].T, [inner, 2 * inner + 2 * G * N], axis=1)
    xbc = silu(causal_conv(xbc, w["conv"], w["conv.b"]))
    x, B, C = np.split(xbc, [inner, inner + G * N], axis=1)
    y = ssd_recurrence(x.reshape(T, H, P), B.reshape(T, G, N), C.reshape(T, G, N), softplus(dt + w["dt_bias"]), w["A_log"], w["D"])
    y = grouped_rms(y.reshape(T, inner) * silu(z), mx["norm_groups"], eps) * w["norm"]
    return y @ w["o"].T


def gla_recurrence(q, k, v, log_alpha):
    """q, k, log_alpha [T, heads, dim], v [T, heads, vdim]: S = diag(alpha) S + k v^T, o = S^T q."""
    T, H, d = q.shape
    S = np.zeros((H, d, v.shape[2]))
    o = np.empty(v.shape)
    for t in range(T):
        S = np.exp(log_alpha[t])[:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = np.einsum("hkv,hk->hv", S, q[t])
    return o


def gla(h, w, mx, eps):
    T, H, d, dv = h.shape[0], mx["heads"], mx["dim"], mx["vdim"]
    q = (h @ w["q"].T).reshape(T, H, d) * d ** -0.5
    k = (h @ w["k"].T).reshape(T, H, d)
    v = (h @ w["v"].T).reshape(T, H, dv)
    z = ((h @ w["a1"].T) @ w["a2"].T + w["a2.b"]).reshape(T, H, d)
    o = gla_recurrence(q, k, v, -softplus(-z) / mx["tau"])
    o = (rms(o, eps) * w["norm"]).reshape(T, H * dv)
    return (o * silu(h @ w["g"].T)) @ w["o"].T


MIXERS = {"latent_attention": latent_attention, "mamba2": mamba2, "gla": gla}


def owner(cfg, i):
    """The layer whose tensors layer i uses."""
    while cfg["layers"][i].get("weights_of") is not None:
        i = cfg["layers"][i]["weights_of"]
    return i


def sub(weights, prefix):
    return {k[len(prefix):]: np.asarray(v, np.float64) for k, v in weights.items() if k.startswith(prefix)}


def forward(cfg, weights, tokens, return_layers=False):
    """Logits [T, vocab] of one sequence (and the residual stream after every layer [layers, T, width])."""
    eps = cfg["norm"]["eps"]
    x = np.asarray(weights["embed"], np.float64)[np.asarray(tokens)]
    layers = []
    for i, ly in enumerate(cfg["layers"]):
        w = sub(weights, f"l{owner(cfg, i)}.")
        mix = {k[4:]: v for k, v in w.items() if k.startswith("mix.")}
        y = MIXERS[ly["type"]](rms_norm(x, w["norm1"], eps), mix, ly["mixer"], eps)
        x = x + rms_norm(y, w["norm1b"], eps)
        if ly["mlp"] is not None:
            y = gated_mlp(rms_norm(x, w["norm2"], eps), w["mlp.gate"], w["mlp.up"], w["mlp.down"])
            x = x + rms_norm(y, w["norm2b"], eps)
        layers.append(x)
    logits = rms_norm(x, np.asarray(weights["final.norm"], np.float64), eps) @ np.asarray(weights["head"], np.float64).T
    return (logits, np.stack(layers)) if return_layers else logits
