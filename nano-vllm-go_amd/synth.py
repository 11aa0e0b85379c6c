"""Synthetic checkpoints for tests and bench: seeded random weights at a model's shapes, produced in
the layout the reference holds AFTER loading (generic_loader.go:353-604): 2-D weights [in, out],
gate|up concatenated, Falcon K|V combined, MoE experts [E, out, in].  Values are rounded to bf16 so
the bf16 device copy is exact (as it is for a real bf16 checkpoint, generic_loader.go:802-805).

Not part of the hot path: an input generator shared by tests/, bench.py and __graft_entry__.smoke().
"""
from __future__ import annotations

import numpy as np


def round_bf16(a: np.ndarray) -> np.ndarray:
    """fp32 -> nearest-even bf16 -> fp32."""
    u = np.ascontiguousarray(a, dtype=np.float32).view(np.uint32)
    r = ((u >> 16) & 1) + np.uint32(0x7FFF)
    return (((u + r) >> 16) << 16).astype(np.uint32).view(np.float32)


def make_weights(cfg: dict, seed: int = 42, scale: float = 0.02, peaked_head: float = 0.0) -> dict:
    """{(slot, layer): fp32 ndarray} in reference post-load layout.  SURVEY.md §8(d): weights
    N(0, scale^2) seeded per layer (seed+layer), norm weights 1+0.02n, biases 0.02n.
    peaked_head > 0 scales an UNTIED LM head (larger logits; used by the greedy fixtures)."""
    H, L, V = cfg["hidden"], cfg["num_layers"], cfg["vocab_size"]
    nH, hd, F = cfg["num_heads"], cfg["head_dim"], cfg["ffn_dim"]
    at = cfg["attention_type"]
    nKV = nH if at == "mha" else (1 if at == "mqa" else cfg["num_kv_heads"])
    ln = cfg["norm_type"] == "layernorm"
    t: dict = {}
    g = np.random.default_rng(seed)

    def w(rng, *shape, s=scale):
        return round_bf16(rng.standard_normal(shape, dtype=np.float32) * np.float32(s))

    def nw(rng, n):
        return round_bf16(1.0 + 0.02 * rng.standard_normal(n, dtype=np.float32))

    def nb(rng, n):
        return round_bf16(0.02 * rng.standard_normal(n, dtype=np.float32))

    emb_scale = scale * (peaked_head if peaked_head > 0 else 1.0)   # LM head only (untied fixtures)
    t[("tok_emb", 0)] = w(g, V, H)
    if cfg["position_type"] == "learned":
        t[("pos_emb", 0)] = w(g, cfg["max_seq_len"], H)
    if not cfg.get("tied_embedding", False):
        t[("lm_head", 0)] = w(g, H, V, s=emb_scale)
    t[("final_norm_w", 0)] = nw(g, H)
    if ln:
        t[("final_norm_b", 0)] = nb(g, H)
    hybrid = cfg.get("hybrid_layers") or []
    for li in range(L):
        r = np.random.default_rng(seed + 1 + li)
        t[("attn_norm_w", li)] = nw(r, H)
        if ln:
            t[("attn_norm_b", li)] = nb(r, H)
        if cfg["block_style"] == "sequential":
            t[("ffn_norm_w", li)] = nw(r, H)
            if ln:
                t[("ffn_norm_b", li)] = nb(r, H)
        if li < len(hybrid) and hybrid[li] in ("mamba", "mamba2"):
            # Mamba2Layer tensors as loadMamba2 leaves them (generic_loader.go:461-512): PyTorch layouts, NOT transposed;
            # the block keeps its shared MLP (loadFFN) and both norms
            EH, nh, ss, ng, K = cfg["mamba_expand"] * H, cfg["mamba_num_heads"], cfg["mamba_state_size"], cfg["mamba_n_groups"], cfg["mamba_conv_kernel"]
            conv_dim = EH + 2 * ng * ss
            t[("mamba_in_proj", li)] = w(r, EH + conv_dim + nh, H)
            t[("mamba_conv_w", li)] = w(r, conv_dim, K, s=0.3)
            t[("mamba_conv_b", li)] = nb(r, conv_dim)
            t[("mamba_a_log", li)] = round_bf16(np.log(r.uniform(1.0, 8.0, nh)).astype(np.float32))
            t[("mamba_d", li)] = nw(r, nh)
            t[("mamba_dt_bias", li)] = round_bf16(r.uniform(-3.0, 0.5, nh).astype(np.float32))
            t[("mamba_norm", li)] = nw(r, EH)
            t[("mamba_out_proj", li)] = w(r, H, EH)
            n1 = 2 * F if cfg["activation_type"] == "swiglu" else F
            t[("w1", li)] = w(r, H, n1)
            t[("w2", li)] = w(r, F, H)
            continue
        t[("wq", li)] = w(r, H, nH * hd)
        if at == "mqa":
            t[("wkv", li)] = w(r, H, 2 * hd)
        else:
            t[("wk", li)] = w(r, H, nKV * hd)
            t[("wv", li)] = w(r, H, nKV * hd)
        t[("wo", li)] = w(r, nH * hd, H)
        if at == "mha":   # GPT-2: attention biases ARE loaded (generic_loader.go:418-441)
            for b, n in (("bq", nH * hd), ("bk", nKV * hd), ("bv", nKV * hd), ("bo", H)):
                t[(b, li)] = nb(r, n)
        if cfg.get("use_moe", False):
            E = cfg["num_experts"]
            t[("router", li)] = w(r, H, E, s=0.5)
            t[("moe_in", li)] = w(r, E, 2 * F, H)
            t[("moe_out", li)] = w(r, E, H, F)
        else:
            n1 = 2 * F if cfg["activation_type"] == "swiglu" else F
            t[("w1", li)] = w(r, H, n1)
            t[("w2", li)] = w(r, F, H)
            # GPT-2 FFN biases exist on disk but the reference never loads them (key built as
            # "...c_fc.weight.bias", generic_loader.go:559-560) -> none here either.
    return t


def tiny_config(family: str, **over) -> dict:
    """Small models of each family for parity tests (shapes legal for the kernels: hd 64, H,F % 64)."""
    base = dict(vocab_size=1000, hidden=128, num_layers=2, num_heads=2, num_kv_heads=2, head_dim=64, ffn_dim=256,
                max_seq_len=256, rope_base=10000.0, norm_eps=1e-5, tied_embedding=False, use_moe=False,
                num_experts=0, num_experts_per_tok=0, embedding_multiplier=0.0, attention_multiplier=0.0,
                residual_multiplier=0.0, logits_scaling=0.0)
    if family == "gpt2":
        base.update(attention_type="mha", norm_type="layernorm", position_type="learned", activation_type="gelu",
                    block_style="sequential", tied_embedding=True, vocab_size=1003)
    elif family == "llama":
        base.update(attention_type="gqa", norm_type="rmsnorm", position_type="rope", activation_type="swiglu",
                    block_style="sequential", num_heads=4, num_kv_heads=2, hidden=256, ffn_dim=512,
                    rope_base=500000.0, tied_embedding=True)
    elif family == "falcon":
        base.update(attention_type="mqa", norm_type="layernorm", position_type="rope", activation_type="gelu",
                    block_style="parallel", num_heads=3, num_kv_heads=1, hidden=192, ffn_dim=768)
    elif family == "granite_moe":
        base.update(attention_type="gqa", norm_type="rmsnorm", position_type="rope", activation_type="swiglu",
                    block_style="sequential", num_heads=4, num_kv_heads=2, hidden=256, ffn_dim=64, use_moe=True,
                    num_experts=8, num_experts_per_tok=2, tied_embedding=True, vocab_size=1027,
                    embedding_multiplier=12.0, attention_multiplier=0.015625, residual_multiplier=0.22,
                    logits_scaling=6.0, norm_eps=1e-6)
    elif family == "granite_hybrid":
        # Granite-4 hybrid (config.go:241-330): GQA attention WITHOUT positional encoding + Mamba2 blocks, shared SwiGLU MLP,
        # muP multipliers; tiny sizes that keep the real ratios (heads x head_dim = expand x hidden)
        base.update(attention_type="gqa", norm_type="rmsnorm", position_type="nope", activation_type="swiglu",
                    block_style="sequential", num_heads=4, num_kv_heads=2, hidden=128, ffn_dim=256, num_layers=4,
                    tied_embedding=True, vocab_size=1019, embedding_multiplier=12.0, attention_multiplier=0.015625,
                    residual_multiplier=0.22, logits_scaling=6.0, norm_eps=1e-5,
                    mamba_expand=2, mamba_state_size=32, mamba_num_heads=8, mamba_head_dim=32, mamba_n_groups=2,
                    mamba_conv_kernel=4, hybrid_layers=["mamba", "attention", "mamba", "mamba"])
    else:
        raise ValueError(family)
    base.update(over)
    return base


def layered_shapes(cfg: dict, decay_rank: int = 16) -> list:
    """[(slot, layer, shape, kind)] of every tensor of a model described by a list of layers (cfg["layers"]: config.LAYER_FIELDS
    dicts); kind: matrix | norm | norm0 (kept as a difference from one) | conv | bias | dt_bias | a_log | decay (0 .. 0.5) — how a synthetic checkpoint
    should draw it.  decay_rank: of the low-rank decay (and gate) projections whose rank the configuration leaves open."""
    H, V, post, par, side = cfg["hidden"], cfg["vocab_size"], cfg["block_style"] == "post", cfg["block_style"] == "parallel", cfg.get("side_dim", 0)
    ln = cfg["norm_type"] == "layernorm"
    norm = "norm0" if cfg.get("norm_weight_offset") else "norm"
    sums = cfg["block_style"] == "sum_norm"
    n1 = 1 if cfg["norm_type"] == "rmsnorm_scalar" else H       # a norm's weights
    out = [("tok_emb", 0, (V, H), "matrix"), ("lm_head", 0, (V, H), "matrix"), ("final_norm_w", 0, (n1,), norm)]
    if ln:
        out.append(("final_norm_b", 0, (H,), "bias"))
    if cfg["position_type"] == "learned":
        out.append(("pos_emb", 0, (cfg["max_seq_len"], H), "matrix"))
    if side:
        out.append(("side_emb", 0, (V, len(cfg["layers"]) * side), "matrix"))
    for i, c in enumerate(cfg["layers"]):
        if c["weights_of"] >= 0:
            continue
        h, d, dv = c["heads"], c["dim"], c["vdim"]
        t = [("mix_scale", (H,), "norm")] if post else [] if sums else [("attn_norm_w", (n1,), norm)]
        t += [("shift", (H,), "decay")] if cfg.get("token_shift") else []
        t += [("attn_norm_b", (H,), "bias")] if ln else []
        t += [] if par else [("mix_post_norm", (n1,), norm)]
        t += [("side_gate", (side, H), "matrix"), ("side_proj", (H, side), "matrix"), ("side_norm", (H,), "norm")] if side else []
        if c["mixer"] == "latent_attention":
            qr, kr, rot = c["q_rank"], c["kv_rank"], c["rot_dim"]
            t += [("lat_dq", (qr, H), "matrix"), ("lat_dq_norm", (qr,), "norm"), ("lat_uq", (h * (d + rot), qr), "matrix"), ("lat_uk", (h * d, kr), "matrix"),
                  ("lat_uv", (h * dv, kr), "matrix"), ("mix_gate", (h if c["gate_per_head"] else h * dv, H), "matrix"), ("wo", (H, h * dv), "matrix")]
            if c["kv_from"] < 0:
                t += [("lat_dkv", (kr + rot, H), "matrix"), ("lat_dkv_norm", (kr,), "norm")]
        elif c["mixer"] == "attention":
            g = c["kv_heads"]
            t += [("wq", (h * d, H), "matrix"), ("wk", (g * d, H), "matrix"), ("wv", (g * dv, H), "matrix"), ("wo", (H, h * dv), "matrix")]
            t += [] if c["ungated"] else [("mix_gate", (h * dv, H), "matrix")]
            t += [("bias_r1", (h,), "norm"), ("bias_r2", (h,), "decay")] if par else []
            t += [("v_mix", (1,), "decay")] if c["v_mix"] else []
            t += [("bq", (h * d,), "bias"), ("bk", (g * d,), "bias"), ("bv", (g * dv,), "bias")] if c["qkv_bias"] else []
            if c["qk_norm"]:
                t += [("q_norm", (d if c["qk_norm"] == 1 else h * d,), "norm"), ("k_norm", (d if c["qk_norm"] == 1 else g * d,), "norm")]
            t += [("sink", (h,), "bias")] if c["sink"] == 2 else []
            if c["mixer2"]:
                qk2, v2 = c["heads2"] * c["dim2"], c["heads2"] * c["vdim2"]
                t += [("lin_q", (qk2, H), "matrix"), ("lin_k", (qk2, H), "matrix"), ("lin_v", (v2, H), "matrix"), ("lin_gate", (v2, H), "matrix"),
                      ("lin_norm", (v2,), "norm"), ("lin_o", (H, v2), "matrix")]
        elif c["mixer"] == "channel_delta":
            qk, r = c["kv_heads"] * d, c["decay_rank"] or decay_rank
            t += [("wq", (qk, H), "matrix"), ("wk", (qk, H), "matrix"), ("wv", (h * dv, H), "matrix"), ("wo", (H, h * dv), "matrix"),
                  ("delta_conv", ((2 * qk + h * dv) * c["conv_taps"],), "conv"), ("delta_beta", (h, H), "matrix"), ("mamba_a_log", (h,), "a_log"),
                  ("gla_norm", (dv,), "norm"), ("gla_a1", (r, H), "matrix"), ("gla_a2", (h * d, r), "matrix"), ("gla_a2_b", (h * d,), "dt_bias"),
                  ("delta_g1", (r, H), "matrix"), ("delta_g2", (h * dv, r), "matrix")]
        elif c["mixer"] == "mamba2":
            inner, conv = h * dv, h * dv + 2 * c["groups"] * c["state"]
            t += [("mamba_in_proj", (inner + conv + h, H), "matrix"), ("mamba_conv_w", (conv * c["conv_taps"],), "conv"), ("mamba_conv_b", (conv,), "bias"),
                  ("mamba_dt_bias", (h,), "dt_bias"), ("mamba_a_log", (h,), "a_log"), ("mamba_d", (h,), "norm"), ("mamba_norm", (inner,), "norm"),
                  ("mamba_out_proj", (H, inner), "matrix")]
        else:
            t += [("wq", (h * d, H), "matrix"), ("wk", (h * d, H), "matrix"), ("wv", (h * dv, H), "matrix"), ("mix_gate", (h * dv, H), "matrix"),
                  ("wo", (H, h * dv), "matrix"), ("gla_norm", (dv,), "norm"), ("gla_a1", (decay_rank, H), "matrix"),
                  ("gla_a2", (h * d, decay_rank), "matrix"), ("gla_a2_b", (h * d,), "bias")]
        if c["experts"]:
            E, I = c["experts"], c["expert_dim"]
            t += [("router", (E, H), "matrix"), ("router_bias", (E,), "bias"), ("moe_in", (E * 2 * I, H), "matrix"), ("moe_out", (E * H, I), "matrix")]
        if sums and (c["ffn_dim"] or c["experts"]):
            t.append(("ffn_post_norm", (n1,), norm))
            t += [("w1", (2 * c["ffn_dim"], H), "matrix"), ("w2", (H, c["ffn_dim"]), "matrix")] if c["ffn_dim"] else []
        elif c["ffn_dim"] and par:
            F, gated = c["ffn_dim"], c["ffn_act"] != 0 or cfg["activation_type"] != "relu2"      # (a layer's own activation here: SwiGLU)
            t += [("w1", ((2 if gated else 1) * F, H), "matrix"), ("w2", (H, F), "matrix")]
        elif c["ffn_dim"]:
            F = c["ffn_dim"]
            t += [("ffn_scale", (H,), "norm")] if post else [("ffn_norm_w", (n1,), norm)]
            t += [("ffn_post_norm", (n1,), norm), ("w1", (2 * F, H), "matrix"), ("w2", (H, F), "matrix")]
        out += [(slot, i, shape, kind) for slot, shape, kind in t]
    return out


def _potuzen(width: int, layers: int, heads: int, q_rank: int, ff: int, window: int = 1024) -> dict:
    """A Potuzen model at a real model's layer sizes: latent attention, Mamba-2 and gated linear attention in turn."""
    from .config import LAYER_FIELDS
    kinds = [dict(mixer="latent_attention", heads=heads, dim=128, vdim=128, q_rank=q_rank, kv_rank=512, window=window, scale=128 ** -0.5),
             dict(mixer="mamba2", heads=width // 32, vdim=64, state=128, groups=1, norm_groups=1, conv_taps=4),
             dict(mixer="gla", heads=heads, dim=128, vdim=128, tau=16.0)]
    return dict(vocab_size=32000, hidden=width, num_layers=layers, num_heads=0, num_kv_heads=0, head_dim=0, ffn_dim=0, max_seq_len=4096,
                attention_type="gqa", norm_type="rmsnorm", position_type="nope", activation_type="geglu", block_style="sandwich",
                rope_base=0.0, norm_eps=1e-6, tied_embedding=False, layers=[dict(LAYER_FIELDS, ffn_dim=ff, **kinds[i % 3]) for i in range(layers)])


def _lufazen(width: int, layers: int, heads: int, q_rank: int, ff: int) -> dict:
    """A Lufazen model at a real model's layer sizes: rotated latent attention (every other one reads the latents of the one before it)
    and two channel-wise delta rules in turn."""
    from .config import LAYER_FIELDS
    lat = dict(mixer="latent_attention", heads=heads, dim=128, vdim=128, q_rank=q_rank, kv_rank=512, scale=192 ** -0.5, rot_dim=64, gate_per_head=1,
               rot_base=1e6, rot_factor=4.0, rot_original=4096.0, rot_fast=32.0, rot_slow=1.0)
    delta = dict(mixer="channel_delta", heads=heads, kv_heads=heads, dim=128, vdim=128, conv_taps=4, decay_rank=128)
    kinds = [lat, delta, delta]
    ls = [dict(LAYER_FIELDS, ffn_dim=ff, ffn_limit=7.0, **kinds[i % 3]) for i in range(layers)]
    for i in range(3, layers, 6):
        ls[i]["kv_from"] = i - 3
    return dict(vocab_size=32000, hidden=width, num_layers=layers, num_heads=0, num_kv_heads=0, head_dim=0, ffn_dim=0, max_seq_len=4096,
                attention_type="gqa", norm_type="rmsnorm", position_type="nope", activation_type="clamped_glu", block_style="post",
                rope_base=0.0, norm_eps=1e-5, tied_embedding=False, norm_weight_offset=1.0, logit_softcap=30.0, layers=ls)


def _bolinex(width: int, layers: int, heads: int, ff: int, expert_ff: int, window: int = 1024) -> dict:
    """A Bolinex model at a real model's layer sizes: grouped attention with a window, dense and expert feed-forwards in turn."""
    from .config import ACT_SWIGLU, LAYER_FIELDS
    att = dict(mixer="attention", heads=heads, kv_heads=heads // 4, dim=128, vdim=128, window=window, scale=128 ** -0.5, softcap=30.0, v_mix=1)
    kinds = [dict(ffn_dim=ff), dict(ffn_dim=expert_ff, ffn_act=ACT_SWIGLU, experts=32, top_k=8, expert_dim=expert_ff, expert_groups=8, groups_kept=4)]
    return dict(vocab_size=32000, hidden=width, num_layers=layers, num_heads=0, num_kv_heads=0, head_dim=0, ffn_dim=0, max_seq_len=4096,
                attention_type="gqa", norm_type="layernorm", position_type="learned", activation_type="relu2", block_style="parallel",
                rope_base=0.0, norm_eps=1e-6, tied_embedding=False, side_dim=256, layers=[dict(LAYER_FIELDS, **att, **kinds[i % 2]) for i in range(layers)])


def _medulorn(width: int, layers: int, heads: int, ff: int, expert_ff: int, window: int = 1024) -> dict:
    """A Medulorn model at a real model's layer sizes: chunked attention with dense feed-forwards, and windowed beside lightning attention with
    experts, in turn."""
    from .config import ACT_CLAMPED_GLU, LAYER_FIELDS, MIXER_LIGHTNING, QK_NORM_HEAD, QK_NORM_ROW, SINK_LEARNED, SINK_ZERO
    att = dict(mixer="attention", heads=heads, kv_heads=heads // 4, dim=128, vdim=128, scale=128 ** -0.5, ungated=1, rot_dim=128, rot_base=1e5)
    kinds = [dict(att, chunk=window, qk_norm=QK_NORM_HEAD, sink=SINK_ZERO, qkv_bias=1, ffn_dim=ff),
             dict(att, window=window, keep_first=8, qk_norm=QK_NORM_ROW, sink=SINK_LEARNED, rot_factor=8.0, rot_low=1.0, rot_high=4.0, rot_original=2048.0, out_scale=0.9,
                  mixer2=MIXER_LIGHTNING, heads2=heads, dim2=128, vdim2=128, out_scale2=0.7, decay=[1.0 - 0.5 ** (1.0 + 7.0 * h / heads) for h in range(heads)],
                  ffn_dim=expert_ff, ffn_act=ACT_CLAMPED_GLU, ffn_limit=7.0, experts=32, top_k=8, expert_dim=expert_ff, expert_groups=1, groups_kept=1, route_softmax=1, expert_limit=7.0)]
    return dict(vocab_size=32000, hidden=width, num_layers=layers, num_heads=0, num_kv_heads=0, head_dim=0, ffn_dim=0, max_seq_len=4096,
                attention_type="gqa", norm_type="rmsnorm_scalar", position_type="nope", activation_type="reglu", block_style="sum_norm",
                rope_base=0.0, norm_eps=1e-6, tied_embedding=False, embedding_multiplier=width ** 0.5, stream_scale=2.0, token_shift=1, logit_softcap=40.0,
                layers=[dict(LAYER_FIELDS, **kinds[i % 2]) for i in range(layers)])


def _gqa(hidden: int, layers: int, heads: int, ff: int, experts: bool = False) -> dict:
    """The grouped-query attention families at the same sizes: dense feed-forwards (Llama), or 32 experts of which a token takes 8 (Granite)."""
    return dict(vocab_size=32000, hidden=hidden, num_layers=layers, num_heads=heads, num_kv_heads=heads // 4, head_dim=128, ffn_dim=ff, max_seq_len=4096,
                attention_type="gqa", norm_type="rmsnorm", position_type="rope", activation_type="swiglu", block_style="sequential", norm_eps=1e-6,
                tied_embedding=False, **(dict(use_moe=True, num_experts=32, num_experts_per_tok=8) if experts else {}))


def _hybrid(hidden: int, layers: int, heads: int, ff: int) -> dict:
    """The attention + Mamba-2 hybrid family at the same sizes (its attention where _potuzen has latent attention, Mamba-2 elsewhere)."""
    return dict(vocab_size=32000, hidden=hidden, num_layers=layers, num_heads=heads, num_kv_heads=heads // 4, head_dim=128, ffn_dim=ff,
                max_seq_len=4096, attention_type="gqa", norm_type="rmsnorm", position_type="nope", activation_type="swiglu",
                block_style="sequential", norm_eps=1e-5, tied_embedding=False, mamba_expand=2, mamba_state_size=128,
                mamba_num_heads=hidden // 32, mamba_head_dim=64, mamba_n_groups=1, mamba_conv_kernel=4,
                hybrid_layers=["attention" if i % 3 == 0 else "mamba" for i in range(layers)])


FULL_CONFIGS = {
    # the reference families' headline shapes
    "gpt2": dict(vocab_size=50257, hidden=768, num_layers=12, num_heads=12, num_kv_heads=12, head_dim=64,
                 ffn_dim=3072, max_seq_len=1024, attention_type="mha", norm_type="layernorm",
                 position_type="learned", activation_type="gelu", block_style="sequential", norm_eps=1e-5,
                 tied_embedding=True),
    "llama-3.2-1b": dict(vocab_size=128256, hidden=2048, num_layers=16, num_heads=32, num_kv_heads=8, head_dim=64,
                         ffn_dim=8192, max_seq_len=4096, attention_type="gqa", norm_type="rmsnorm",
                         position_type="rope", activation_type="swiglu", block_style="sequential",
                         rope_base=500000.0, norm_eps=1e-5, tied_embedding=True),
    "falcon-7b": dict(vocab_size=65024, hidden=4544, num_layers=32, num_heads=71, num_kv_heads=1, head_dim=64,
                      ffn_dim=18176, max_seq_len=2048, attention_type="mqa", norm_type="layernorm",
                      position_type="rope", activation_type="gelu", block_style="parallel", norm_eps=1e-5,
                      tied_embedding=False),
    "granite-3.0-1b-a400m": dict(vocab_size=49155, hidden=1024, num_layers=24, num_heads=16, num_kv_heads=8,
                                 head_dim=64, ffn_dim=512, max_seq_len=4096, attention_type="gqa",
                                 norm_type="rmsnorm", position_type="rope", activation_type="swiglu",
                                 block_style="sequential", rope_base=10000.0, norm_eps=1e-6, tied_embedding=True,
                                 use_moe=True, num_experts=32, num_experts_per_tok=8, embedding_multiplier=12.0,
                                 attention_multiplier=0.015625, residual_multiplier=0.22, logits_scaling=6.0),
    "llama-3-8b": dict(vocab_size=128256, hidden=4096, num_layers=32, num_heads=32, num_kv_heads=8, head_dim=128,
                       ffn_dim=14336, max_seq_len=4096, attention_type="gqa", norm_type="rmsnorm",
                       position_type="rope", activation_type="swiglu", block_style="sequential",
                       rope_base=500000.0, norm_eps=1e-5, tied_embedding=False),
    # designs described by a list of layers at a real model's layer sizes, and the closest other family at the same sizes
    "medulorn-2k": _medulorn(2048, 12, 16, 6144, 512), "medulorn-4k": _medulorn(4096, 6, 32, 12288, 1024),
    "bolinex-2k": _bolinex(2048, 12, 16, 6144, 512), "bolinex-4k": _bolinex(4096, 6, 32, 12288, 1024),
    "gqa-2k": _gqa(2048, 12, 16, 6144), "gqa-moe-2k": _gqa(2048, 12, 16, 512, True), "gqa-4k": _gqa(4096, 6, 32, 12288), "gqa-moe-4k": _gqa(4096, 6, 32, 1024, True),
    "lufazen-2k": _lufazen(2048, 12, 16, 768, 6144), "lufazen-4k": _lufazen(4096, 6, 32, 1536, 12288),
    "potuzen-2k": _potuzen(2048, 12, 16, 768, 6144), "hybrid-2k": _hybrid(2048, 12, 16, 6144),
    "potuzen-4k": _potuzen(4096, 6, 32, 1536, 12288), "hybrid-4k": _hybrid(4096, 6, 32, 12288),
}
for _c in FULL_CONFIGS.values():
    for _k, _v in dict(use_moe=False, num_experts=0, num_experts_per_tok=0, embedding_multiplier=0.0,
                       attention_multiplier=0.0, residual_multiplier=0.0, logits_scaling=0.0,
                       rope_base=10000.0).items():
        _c.setdefault(_k, _v)
