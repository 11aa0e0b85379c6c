"""Small Medulorn models for the tests: configurations (parsed config.json), seeded random weights rounded to bf16, and token sequences
whose expert choices are not close calls.  The checkpoint folder is written by potuzen_models.write."""
from __future__ import annotations

import numpy as np

import medulorn_oracle as O
from potuzen_models import bf16


def dense(ff=88):
    return dict(kind="dense", ff=ff)


def moe(experts=10, top=3, ff=40, limit=1.5, shared=56, shared_limit=2.5):
    return dict(kind="moe", expert=dict(ff=ff, limit=limit), router=dict(experts=experts, top=top),
                shared=None if shared is None else dict(ff=shared, limit=shared_limit))


def rot(dims, base=10000.0, scaling=None):
    """scaling: (factor, low, high, original) or None."""
    return dict(base=base, dims=dims, **({} if scaling is None else dict(scaling=dict(zip(("factor", "low", "high", "original"), scaling)))))


def attention(heads=6, kv_heads=2, dim=40, vdim=24, chunk=50, scale=0.2, turn=rot(40), mlp=dense()):
    mx = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, mask=None if chunk is None else dict(size=chunk), rot=turn)
    return dict(type="attention", mixer=mx, mlp=mlp)


def decays(n):
    return np.round(1.0 - np.geomspace(0.5, 0.004, n), 4).tolist()


def parallel(heads=4, kv_heads=2, dim=24, vdim=40, window=30, keep=3, scale=0.25, turn=rot(16, 5000.0, (8.0, 1.0, 4.0, 60)), left_scale=0.7,
             heads2=3, dim2=20, vdim2=28, decay=None, right_scale=1.4, mlp=dense()):
    left = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, mask=None if window is None else dict(size=window, keep_first=keep), rot=turn)
    right = dict(heads=heads2, dim=dim2, vdim=vdim2, decay=decays(heads2) if decay is None else decay)
    return dict(type="parallel", mixer=dict(left=left, left_scale=left_scale, right=right, right_scale=right_scale), mlp=mlp)


def config(layers, width=160, vocab=331, eps=1e-5, alpha=1.7, scale=6.0, cap=25.0):
    return dict(architecture="Medulorn", vocab=vocab, width=width, norm=dict(eps=eps), embedding=dict(scale=scale), postln_alpha=alpha, logit_softcap=cap, layers=layers)


def weights(cfg, seed=0, sink=(0.0, 1.5), shift=(-0.2, 0.9)):
    """{tensor name: fp32 array whose values are bf16}.  sink: mean and spread; shift: range."""
    g = np.random.default_rng(seed)
    W, V = cfg["width"], cfg["vocab"]
    t = {}

    def mat(name, out, inn, s=1.0):
        t[name] = bf16(g.standard_normal((out, inn)) * (s / np.sqrt(inn)))

    def vec(name, n, mean=1.0, s=0.2):
        t[name] = bf16(mean + s * g.standard_normal(n))

    def one(name):
        t[name] = bf16(np.float32(g.uniform(0.6, 1.5))).reshape(())

    def glu(name, ff):
        mat(name + "gate", ff, W, 1.5); mat(name + "up", ff, W, 1.5); mat(name + "down", W, ff)

    t["embed"] = bf16(g.standard_normal((V, W)) / cfg["embedding"]["scale"])
    mat("head", V, W, 2.0)
    one("final.norm")
    for i, ly in enumerate(cfg["layers"]):
        p, m, f, mx, mlp = f"l{i}.", f"l{i}.mix.", f"l{i}.mlp.", ly["mixer"], ly["mlp"]
        one(p + "norm1")
        t[p + "shift"] = bf16(g.uniform(*shift, W))
        two = ly["type"] == "parallel"
        a, mx = (m + "left.", mx["left"]) if two else (m, mx)
        H, G, d, dv = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
        mat(a + "q", H * d, W); mat(a + "k", G * d, W); mat(a + "v", G * dv, W); mat(a + "o", W, H * dv, 1.5)
        vec(a + "q.norm", H * d if two else d, 1.3, 0.3); vec(a + "k.norm", G * d if two else d, 1.3, 0.3)
        if two:
            vec(a + "sink", H, *sink)
            r, R = m + "right.", ly["mixer"]["right"]
            n, v = R["heads"] * R["dim"], R["heads"] * R["vdim"]
            mat(r + "q", n, W, 1.5); mat(r + "k", n, W, 1.5); mat(r + "v", v, W, 1.5); mat(r + "g", v, W, 1.5); vec(r + "norm", v); mat(r + "o", W, v)
        else:
            vec(a + "q.b", H * d, 0.0, 0.5); vec(a + "k.b", G * d, 0.0, 0.5); vec(a + "v.b", G * dv, 0.0, 0.5)
        if mlp is None:
            continue
        one(p + "norm2")
        if mlp["kind"] == "dense":
            glu(f, mlp["ff"])
            continue
        E = mlp["router"]["experts"]
        for e in range(E):
            glu(f + f"e{e}.", mlp["expert"]["ff"])
        mat(f + "router", E, W, 0.7)
        vec(f + "router.b", E, 0.0, 1.5)
        if mlp["shared"] is not None:
            glu(f + "shared.", mlp["shared"]["ff"])
    return t


def clear_tokens(cfg, w, n, seed, margin=0.014):
    """n random tokens on which no router's choice is closer than `margin`, and their (logits, residual streams)."""
    g = np.random.default_rng(seed)
    tok = g.integers(0, cfg["vocab"], n)
    for _ in range(80):
        close = []
        logits, layers = O.forward(cfg, w, tok, return_layers=True, margins=close)
        bad = np.zeros(n, bool) if not close else np.min(close, axis=0) < margin
        if not bad.any():
            return tok.tolist(), logits, layers
        tok[bad] = g.integers(0, cfg["vocab"], int(bad.sum()))
    raise AssertionError("no sequence without close calls found")
