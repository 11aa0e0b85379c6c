"""Small Lufazen models for the tests: configurations (parsed config.json) and seeded random weights rounded to bf16.  The checkpoint
folder is written by potuzen_models.write."""
from __future__ import annotations

import numpy as np

from potuzen_models import bf16


def mlp(ff, limit):
    return None if ff is None else dict(kind="dense", ff=ff, limit=limit)


def latent(heads=3, dim=40, rot=48, vdim=24, q_rank=56, kv_rank=72, scale=0.15, base=1000.0, scaling=(3.0, 64, 8.0, 1.0), kv_from=None, ff=88, limit=1.1):
    """scaling: (factor, original, fast, slow) or None."""
    mx = dict(heads=heads, dim=dim, rot_dim=rot, vdim=vdim, q_rank=q_rank, kv_rank=kv_rank, scale=scale,
              rot=dict(base=base, dims=rot, scaling=None if scaling is None else dict(zip(("factor", "original", "fast", "slow"), scaling))))
    if kv_from is not None:
        mx["kv_from"] = kv_from
    return dict(type="latent_attention", mixer=mx, mlp=mlp(ff, limit))


def delta(heads=4, kv_heads=2, dim=36, vdim=28, conv=4, ff=72, limit=0.9):
    return dict(type="channel_delta", mixer=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv), mlp=mlp(ff, limit))


def config(layers, width=160, vocab=331, eps=1e-5, cap=12.0):
    return dict(architecture="Lufazen", vocab=vocab, width=width, norm=dict(eps=eps), logit_softcap=cap, layers=layers)


def weights(cfg, seed=0, a_rank=7, g_rank=11, decay_bias=-1.0, a_log=(0.1, 4.0), rot_scale=1.0):
    """{tensor name: fp32 array whose values are bf16}.  decay_bias: mean of dt_bias; a_log: range of exp(A_log); rot_scale: of the
    rotated queries and keys."""
    g = np.random.default_rng(seed)
    W, V = cfg["width"], cfg["vocab"]
    t = {}

    def mat(name, out, inn, s=1.0):
        t[name] = bf16(g.standard_normal((out, inn)) * (s / np.sqrt(inn)))

    def norm(name, n, mean=1.0):
        t[name] = bf16(mean + 0.2 * g.standard_normal(n))

    t["embed"] = bf16(g.standard_normal((V, W)))
    mat("head", V, W, 4.0)
    norm("final.norm", W, 0.0)
    for i, ly in enumerate(cfg["layers"]):
        p, m, mx = f"l{i}.", f"l{i}.mix.", ly["mixer"]
        H, dv, d = mx["heads"], mx["vdim"], mx["dim"]
        norm(p + "norm1", W, 0.0)
        norm(p + "ls1", W, 0.7)
        if ly["type"] == "latent_attention":
            r, qr, kr = mx["rot_dim"], mx["q_rank"], mx["kv_rank"]
            mat(m + "dq", qr, W); norm(m + "dq.norm", qr); mat(m + "uq", H * (d + r), qr, 1.5)
            t[m + "uq"].reshape(H, d + r, qr)[:, d:] = bf16(t[m + "uq"].reshape(H, d + r, qr)[:, d:] * rot_scale)
            if mx.get("kv_from") is None:
                mat(m + "dkv", kr + r, W); norm(m + "dkv.norm", kr)
                t[m + "dkv"][kr:] = bf16(t[m + "dkv"][kr:] * rot_scale)
            mat(m + "uk", H * d, kr); mat(m + "uv", H * dv, kr); mat(m + "g", H, W); mat(m + "o", W, H * dv)
        else:
            G = mx["kv_heads"]
            for n, ch in (("q", G * d), ("k", G * d), ("v", H * dv)):
                mat(m + n, ch, W)
                t[m + n + ".conv"] = bf16(0.6 * g.standard_normal((ch, mx["conv"])))
            mat(m + "b", H, W); mat(m + "o", W, H * dv); norm(m + "norm", dv)
            t[m + "A_log"] = bf16(np.log(g.uniform(*a_log, H)))
            mat(m + "a1", a_rank, W); mat(m + "a2", H * d, a_rank)
            t[m + "dt_bias"] = bf16(decay_bias + g.standard_normal(H * d))
            mat(m + "g1", g_rank, W); mat(m + "g2", H * dv, g_rank)
        if ly["mlp"] is not None:
            ff = ly["mlp"]["ff"]
            norm(p + "norm2", W, 0.0)
            norm(p + "ls2", W, 0.7)
            mat(p + "mlp.gate", ff, W); mat(p + "mlp.up", ff, W); mat(p + "mlp.down", W, ff)
    return t
