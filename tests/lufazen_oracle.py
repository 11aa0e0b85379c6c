"""Plain restatement of the Lufazen design in numpy float64: one function per mechanism, whole sequences from position 0, token by
token where the mechanism is a recurrence.  It shares no code with the product: the tests compare the HIP path with it.

Weights are a dict {checkpoint tensor name: array}, every matrix [out, in] and applied as W x; the configuration is the parsed
config.json.
"""
from __future__ import annotations

import numpy as np

GLU_SLOPE = 1.702
UNIT_EPS = 1e-6


def sigmoid(z):
    e = np.exp(-np.abs(z))
    return np.where(z >= 0, 1.0 / (1.0 + e), e / (1.0 + e))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.maximum(z, 0.0) + np.log1p(np.exp(-np.abs(z)))


def rms(x, eps):
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps)


def rms_norm(x, w, eps):
    return rms(x, eps) * w


def centred_norm(x, w, eps):
    """The norm whose weight is kept as its difference from one."""
    return rms(x, eps) * (1.0 + w)


def unit(x):
    return x / np.sqrt((x * x).sum(axis=-1, keepdims=True) + UNIT_EPS)


def clamped_glu(h, gate, up, down, limit):
    g = np.minimum(h @ gate.T, limit)
    u = np.clip(h @ up.T, -limit, limit)
    return (g * sigmoid(GLU_SLOPE * g) * (u + 1.0)) @ down.T


def frequencies(rot):
    """Angle per position of every rotated pair, and the factor on cos and sin."""
    n, base, sc = rot["dims"], rot["base"], rot.get("scaling")
    i = np.arange(n // 2)
    f = base ** (-2.0 * i / n)
    if sc is None:
        return f, 1.0

    def place(turns):       # the pair that turns this often over the original length
        return n * np.log(sc["original"] / (2 * np.pi * turns)) / (2 * np.log(base))
    lo, hi = max(np.floor(place(sc["fast"])), 0), min(np.ceil(place(sc["slow"])), n - 1)
    ramp = np.clip((i - lo) / max(hi - lo, 0.001), 0, 1)
    return f / sc["factor"] * ramp + f * (1 - ramp), 0.1 * np.log(sc["factor"]) + 1.0


def rotate(x, rot):
    """x [T, ..., n]: row t is position t; dimension i turns with dimension i + n / 2."""
    f, mag = frequencies(rot)
    n = rot["dims"]
    a = np.arange(x.shape[0])[:, None] * f
    shape = (x.shape[0],) + (1,) * (x.ndim - 2) + (n // 2,)
    c, s = (np.cos(a) * mag).reshape(shape), (np.sin(a) * mag).reshape(shape)
    u, v = x[..., :n // 2], x[..., n // 2:n]
    return np.concatenate([u * c - v * s, v * c + u * s, x[..., n:]], axis=-1)


def causal_softmax_attention(q, k, v, scale):
    """q, k [T, heads, dim], v [T, heads, vdim]: query i sees keys 0 .. i."""
    out = np.empty(v.shape)
    for i in range(q.shape[0]):
        s = np.einsum("hd,jhd->hj", q[i], k[:i + 1]) * scale
        p = np.exp(s - s.max(axis=1, keepdims=True))
        out[i] = np.einsum("hj,jhd->hd", p / p.sum(axis=1, keepdims=True), v[:i + 1])
    return out


def latents(h, w, mx, eps):
    """What a layer's cache holds: the normed latent, and the rotated key part that all heads share."""
    kv = h @ w["dkv"].T
    return rms_norm(kv[:, :mx["kv_rank"]], w["dkv.norm"], eps), rotate(kv[:, mx["kv_rank"]:], mx["rot"])


def latent_attention(h, w, mx, eps, cached):
    T, H, d, r, dv = h.shape[0], mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"]
    c, k_rot = cached
    q = (rms_norm(h @ w["dq"].T, w["dq.norm"], eps) @ w["uq"].T).reshape(T, H, d + r)
    q = np.concatenate([q[..., :d], rotate(q[..., d:], mx["rot"])], axis=-1)
    k = np.concatenate([(c @ w["uk"].T).reshape(T, H, d), np.broadcast_to(k_rot[:, None], (T, H, r))], axis=-1)
    o = causal_softmax_attention(q, k, (c @ w["uv"].T).reshape(T, H, dv), mx["scale"])
    o = o * sigmoid(h @ w["g"].T)[:, :, None]
    return o.reshape(T, H * dv) @ w["o"].T


def causal_conv(x, w):
    """Per channel: w [channels, taps], the last tap is the current token's; zeros before the sequence."""
    T, taps = x.shape[0], w.shape[1]
    xp = np.concatenate([np.zeros((taps - 1, x.shape[1])), x])
    return sum(xp[i:i + T] * w[:, i] for i in range(taps))


def delta_recurrence(q, k, v, log_decay, beta):
    """q, k, log_decay [T, heads, dim], v [T, heads, vdim], beta [T, heads]:
    S <- diag(decay) S, u = beta (v - S^T k), S <- S + k u^T, o = S^T q."""
    T, H, d = q.shape
    S = np.zeros((H, d, v.shape[2]))
    o = np.empty(v.shape)
    for t in range(T):
        S = np.exp(log_decay[t])[:, :, None] * S
        u = beta[t][:, None] * (v[t] - np.einsum("hkv,hk->hv", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        o[t] = np.einsum("hkv,hk->hv", S, q[t])
    return o


def channel_decay(h, w, heads, dim):
    z = ((h @ w["a1"].T) @ w["a2"].T + w["dt_bias"]).reshape(-1, heads, dim)
    return -np.exp(w["A_log"])[None, :, None] * softplus(z)


def channel_delta(h, w, mx, eps):
    T, H, G, d, dv = h.shape[0], mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q, k, v = (silu(causal_conv(h @ w[n].T, w[n + ".conv"])) for n in "qkv")
    share = np.arange(H) // (H // G)
    q, k = unit(q.reshape(T, G, d))[:, share] * d ** -0.5, unit(k.reshape(T, G, d))[:, share]
    o = delta_recurrence(q, k, v.reshape(T, H, dv), channel_decay(h, w, H, d), sigmoid(h @ w["b"].T))
    gate = sigmoid((h @ w["g1"].T) @ w["g2"].T)
    return (rms_norm(o, w["norm"], eps).reshape(T, H * dv) * gate) @ w["o"].T


def sub(weights, prefix):
    return {k[len(prefix):]: np.asarray(v, np.float64) for k, v in weights.items() if k.startswith(prefix)}


def forward(cfg, weights, tokens, return_layers=False):
    """Logits [T, vocab] of one sequence (and the residual stream after every layer [layers, T, width])."""
    eps = cfg["norm"]["eps"]
    x = np.asarray(weights["embed"], np.float64)[np.asarray(tokens)]
    layers, cached = [], {}
    for i, ly in enumerate(cfg["layers"]):
        w, mx = sub(weights, f"l{i}."), ly["mixer"]
        mix = {k[4:]: v for k, v in w.items() if k.startswith("mix.")}
        if ly["type"] == "latent_attention":
            j = mx.get("kv_from")
            cached[i] = latents(x, mix, mx, eps) if j is None else cached[j]
            y = latent_attention(x, mix, mx, eps, cached[i])
        else:
            y = channel_delta(x, mix, mx, eps)
        x = x + centred_norm(y, w["norm1"], eps) * w["ls1"]
        if ly["mlp"] is not None:
            y = clamped_glu(x, w["mlp.gate"], w["mlp.up"], w["mlp.down"], ly["mlp"]["limit"])
            x = x + centred_norm(y, w["norm2"], eps) * w["ls2"]
        layers.append(x)
    logits = centred_norm(x, np.asarray(weights["final.norm"], np.float64), eps) @ np.asarray(weights["head"], np.float64).T
    cap = cfg["logit_softcap"]
    logits = cap * np.tanh(logits / cap)
    return (logits, np.stack(layers)) if return_layers else logits
