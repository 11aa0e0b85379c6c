"""Small Bolinex models for the tests: configurations (parsed config.json), seeded random weights rounded to bf16, and token sequences
whose expert choices are not close calls.  The checkpoint folder is written by potuzen_models.write."""
from __future__ import annotations

import numpy as np

import bolinex_oracle as O
from potuzen_models import bf16


def dense(ff=88):
    return dict(kind="dense", ff=ff)


def moe(experts=12, top=3, groups=(4, 2), ff=40, shared=56):
    """groups: (count, keep) or None."""
    out = dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, top=top), shared=None if shared is None else dict(ff=shared))
    out["router"]["groups"] = None if groups is None else dict(count=groups[0], keep=groups[1])
    return out


def attention(heads=6, kv_heads=2, dim=40, vdim=24, window=50, scale=0.2, cap=9.0, v_mix=True, mlp=dense()):
    mx = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, softcap=cap, v_mix=v_mix, mask=None if window is None else dict(size=window))
    return dict(type="attention", mixer=mx, mlp=mlp)


def config(layers, width=160, vocab=331, eps=1e-5, side=20, positions=700):
    return dict(architecture="Bolinex", vocab=vocab, width=width, norm=dict(eps=eps), token_side=None if side is None else dict(dim=side), max_positions=positions, layers=layers)


def weights(cfg, seed=0, r1=(0.02, 2.0), r2=(0.05, 0.5), correction=(-2.2, 0.7)):
    """{tensor name: fp32 array whose values are bf16}.  r1, r2: ranges; correction: mean and spread."""
    g = np.random.default_rng(seed)
    W, V, sd, L = cfg["width"], cfg["vocab"], (cfg["token_side"] or {}).get("dim", 0), len(cfg["layers"])
    t = {}

    def mat(name, out, inn, s=1.0):
        t[name] = bf16(g.standard_normal((out, inn)) * (s / np.sqrt(inn)))

    def norm(name, n, bias=True):
        t[name] = bf16(1.0 + 0.2 * g.standard_normal(n))
        if bias:
            t[name + ".b"] = bf16(0.3 * g.standard_normal(n))

    def glu(name, ff):
        mat(name + ".gate", ff, W); mat(name + ".up", ff, W); mat(name + ".down", W, ff)

    t["embed"] = bf16(g.standard_normal((V, W)))
    t["pos"] = bf16(0.4 * g.standard_normal((cfg["max_positions"], W)))
    if sd:
        t["side.embed"] = bf16(g.standard_normal((V, L * sd)))
    mat("head", V, W, 2.0)
    norm("final.norm", W)
    for i, ly in enumerate(cfg["layers"]):
        p, m, f, mx, mlp = f"l{i}.", f"l{i}.mix.", f"l{i}.mlp.", ly["mixer"], ly["mlp"]
        H, G, d, dv = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
        norm(p + "norm1", W)
        mat(m + "q", H * d, W, 1.5); mat(m + "k", G * d, W, 1.5); mat(m + "v", G * dv, W); mat(m + "g", H * dv, W); mat(m + "o", W, H * dv)
        t[m + "r1"], t[m + "r2"] = bf16(g.uniform(*r1, H)), bf16(g.uniform(*r2, H))
        if mx["v_mix"]:
            t[m + "vmix"] = bf16(np.float32(g.uniform(0.2, 0.8)))
        if sd:
            mat(p + "side.gate", sd, W); mat(p + "side.proj", W, sd); norm(p + "side.norm", W, False)
        if mlp is None:
            continue
        if mlp["kind"] == "dense":
            mat(f + "up", mlp["ff"], W); mat(f + "down", W, mlp["ff"])
            continue
        E = mlp["router"]["experts"]
        for e in range(E):
            glu(f + f"e{e}", mlp["expert"]["ff"])
        mat(f + "router", E, W, 1.5)
        t[f + "correction"] = bf16(correction[0] + correction[1] * g.standard_normal(E))
        if mlp["shared"] is not None:
            glu(f + "shared", mlp["shared"]["ff"])
    return {k: v.reshape(()) if k.endswith("vmix") else v for k, v in t.items()}


def clear_tokens(cfg, w, n, seed, margin=0.012):
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
