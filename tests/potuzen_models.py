"""Small Potuzen models for the tests: configurations (parsed config.json), seeded random weights rounded to bf16, and a writer of
the checkpoint folder (config.json + model.safetensors in bf16, or fp32)."""
from __future__ import annotations

import json
import os
import struct

import numpy as np


def bf16_bits(a):
    u = np.ascontiguousarray(a, np.float32).view(np.uint32)
    return ((u + ((u >> 16) & 1) + np.uint32(0x7FFF)) >> 16).astype(np.uint16)


def bf16(a):
    return (bf16_bits(a).astype(np.uint32) << 16).view(np.float32)


def latent(heads=3, dim=40, vdim=24, q_rank=56, kv_rank=72, window=50, scale=0.3, ff=88, **kw):
    return dict(type="latent_attention", mlp=None if ff is None else dict(kind="dense", ff=ff),
                mixer=dict(heads=heads, dim=dim, vdim=vdim, q_rank=q_rank, kv_rank=kv_rank, mask=dict(size=window), scale=scale), **kw)


def mamba2(heads=4, vdim=20, state=24, groups=2, norm_groups=1, conv=3, ff=72, **kw):
    return dict(type="mamba2", mlp=None if ff is None else dict(kind="dense", ff=ff),
                mixer=dict(heads=heads, vdim=vdim, state=state, groups=groups, norm_groups=norm_groups, conv=conv), **kw)


def gla(heads=5, dim=36, vdim=28, tau=12.0, ff=104, **kw):
    return dict(type="gla", mlp=None if ff is None else dict(kind="dense", ff=ff), mixer=dict(heads=heads, dim=dim, vdim=vdim, tau=tau), **kw)


def config(layers, width=160, vocab=331, eps=1e-5):
    return dict(architecture="Potuzen", vocab=vocab, width=width, norm=dict(eps=eps), layers=layers)


def weights(cfg, seed=0, rank=8, decay_bias=0.0):
    """{tensor name: fp32 array whose values are bf16}.  rank: of GLA's decay projection; decay_bias: mean of its bias."""
    g = np.random.default_rng(seed)
    W, V = cfg["width"], cfg["vocab"]
    t = {}

    def mat(name, out, inn, s=1.0):
        t[name] = bf16(g.standard_normal((out, inn)) * (s / np.sqrt(inn)))

    def norm(name, n):
        t[name] = bf16(1.0 + 0.2 * g.standard_normal(n))

    t["embed"] = bf16(g.standard_normal((V, W)))
    mat("head", V, W)
    norm("final.norm", W)
    for i, ly in enumerate(cfg["layers"]):
        if ly.get("weights_of") is not None:
            continue
        p, m, mx = f"l{i}.", f"l{i}.mix.", ly["mixer"]
        H, dv = mx["heads"], mx["vdim"]
        norm(p + "norm1", W)
        norm(p + "norm1b", W)
        if ly["type"] == "latent_attention":
            d, qr, kr = mx["dim"], mx["q_rank"], mx["kv_rank"]
            mat(m + "dq", qr, W); norm(m + "dq.norm", qr); mat(m + "uq", H * d, qr)
            mat(m + "dkv", kr, W); norm(m + "dkv.norm", kr); mat(m + "uk", H * d, kr); mat(m + "uv", H * dv, kr)
            mat(m + "g", H * dv, W); mat(m + "o", W, H * dv)
        elif ly["type"] == "mamba2":
            inner, GN = H * dv, mx["groups"] * mx["state"]
            mat(m + "in", 2 * inner + 2 * GN + H, W)
            t[m + "conv"] = bf16(0.5 * g.standard_normal((inner + 2 * GN, mx["conv"])))
            t[m + "conv.b"] = bf16(0.2 * g.standard_normal(inner + 2 * GN))
            t[m + "dt_bias"] = bf16(g.uniform(-3.0, 0.5, H))
            t[m + "A_log"] = bf16(np.log(g.uniform(0.3, 8.0, H)))
            t[m + "D"] = bf16(1.0 + 0.3 * g.standard_normal(H))
            norm(m + "norm", inner)
            mat(m + "o", W, inner)
        else:
            d = mx["dim"]
            mat(m + "q", H * d, W); mat(m + "k", H * d, W); mat(m + "v", H * dv, W); mat(m + "g", H * dv, W); mat(m + "o", W, H * dv)
            norm(m + "norm", dv)
            mat(m + "a1", rank, W); mat(m + "a2", H * d, rank, 2.0)
            t[m + "a2.b"] = bf16(decay_bias + g.standard_normal(H * d))
        if ly["mlp"] is not None:
            ff = ly["mlp"]["ff"]
            norm(p + "norm2", W)
            norm(p + "norm2b", W)
            mat(p + "mlp.gate", ff, W); mat(p + "mlp.up", ff, W); mat(p + "mlp.down", W, ff)
    return t


def write(dirname, cfg, w):
    os.makedirs(dirname, exist_ok=True)
    with open(os.path.join(dirname, "config.json"), "w") as f:
        json.dump(cfg, f)
    head, blobs, off = {}, [], 0
    for name, a in w.items():
        b = bf16_bits(a).tobytes()
        head[name] = dict(dtype="BF16", shape=list(a.shape), data_offsets=[off, off + len(b)])
        blobs.append(b)
        off += len(b)
    h = json.dumps(head).encode()
    with open(os.path.join(dirname, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(h)) + h + b"".join(blobs))
    return str(dirname)
