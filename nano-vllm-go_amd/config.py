"""Mirror of purego/tensor/config.go: ModelConfig (config.go:58-122), the per-architecture
templates (config.go:125-376) and LoadModelConfig (generic_loader.go:808-1007) — the plain-data
input contract of the forward path.  Field names are the Go names in snake_case.
"""
from __future__ import annotations

import json
from dataclasses import asdict, dataclass, field


@dataclass
class ModelConfig:
    architecture: str = "gpt2"
    model_name: str = ""
    vocab_size: int = 0
    hidden: int = 0
    num_layers: int = 0
    num_heads: int = 0
    num_kv_heads: int = 0
    head_dim: int = 0
    ffn_dim: int = 0
    max_seq_len: int = 0
    attention_type: str = "mha"       # mha | mqa | gqa            config.go:18-22
    norm_type: str = "layernorm"      # layernorm | rmsnorm        config.go:27-30
    position_type: str = "learned"    # learned | rope | nope      config.go:35-40
    activation_type: str = "gelu"     # gelu | swiglu              config.go:45-48
    block_style: str = "sequential"   # sequential | parallel      config.go:53-56
    eos_token_id: int = 0
    bos_token_id: int = 0
    pad_token_id: int = 0
    rope_base: float = 10000.0
    norm_eps: float = 1e-5
    tied_embedding: bool = False
    use_moe: bool = False
    num_experts: int = 0
    num_experts_per_tok: int = 0
    embedding_multiplier: float = 0.0
    attention_multiplier: float = 0.0
    residual_multiplier: float = 0.0
    logits_scaling: float = 0.0
    hybrid_layers: list = field(default_factory=list)     # config.go:113: "attention" | "mamba" | "mamba2" per layer
    mamba_expand: int = 0             # config.go:100-106
    mamba_state_size: int = 0
    mamba_num_heads: int = 0
    mamba_head_dim: int = 0
    mamba_n_groups: int = 0
    mamba_conv_kernel: int = 0
    layers: list = field(default_factory=list)            # models described by a list of layers: one dict per layer (LAYER_FIELDS)
    norm_weight_offset: float = 0.0
    logit_softcap: float = 0.0
    side_dim: int = 0                 # per-layer token inputs
    stream_scale: float = 0.0         # norms of sums: factor of the residual stream
    token_shift: int = 0

    @property
    def mamba_layer_mask(self):
        m = [0, 0]
        for i, t in enumerate(self.hybrid_layers[:128]):
            if t in ("mamba", "mamba2"):
                m[i >> 6] |= 1 << (i & 63)
        return m

    def to_dict(self) -> dict:
        return asdict(self)


def new_gpt2_config() -> ModelConfig:           # config.go:125-148
    return ModelConfig(architecture="gpt2", model_name="gpt2", vocab_size=50257, hidden=768, num_layers=12,
                       num_heads=12, num_kv_heads=12, head_dim=64, ffn_dim=3072, max_seq_len=1024,
                       attention_type="mha", norm_type="layernorm", position_type="learned",
                       activation_type="gelu", block_style="sequential", eos_token_id=50256,
                       bos_token_id=50256, pad_token_id=50256, norm_eps=1e-5, tied_embedding=True)


def new_falcon_config(size: str = "7b") -> ModelConfig:   # config.go:151-194
    c = ModelConfig(architecture="falcon", attention_type="mqa", norm_type="layernorm", position_type="rope",
                    activation_type="gelu", block_style="parallel", num_kv_heads=1, rope_base=10000.0,
                    norm_eps=1e-5, tied_embedding=False, eos_token_id=11, bos_token_id=11, pad_token_id=11)
    if size == "40b":
        c.model_name, c.vocab_size, c.hidden, c.num_layers, c.num_heads, c.head_dim, c.ffn_dim, c.max_seq_len = \
            "falcon-40b", 65024, 8192, 60, 128, 64, 32768, 2048
    else:
        c.model_name, c.vocab_size, c.hidden, c.num_layers, c.num_heads, c.head_dim, c.ffn_dim, c.max_seq_len = \
            "falcon-7b", 65024, 4544, 32, 71, 64, 18176, 2048
    return c


def new_llama_config(size: str = "7b") -> ModelConfig:    # config.go:197-242
    c = ModelConfig(architecture="llama", attention_type="gqa", norm_type="rmsnorm", position_type="rope",
                    activation_type="swiglu", block_style="sequential", rope_base=10000.0, norm_eps=1e-6,
                    tied_embedding=False, eos_token_id=2, bos_token_id=1, pad_token_id=0)
    if size == "13b":
        c.model_name, c.vocab_size, c.hidden, c.num_layers, c.num_heads, c.num_kv_heads, c.head_dim, c.ffn_dim, \
            c.max_seq_len = "llama-13b", 32000, 5120, 40, 40, 10, 128, 13824, 4096
    else:
        c.model_name, c.vocab_size, c.hidden, c.num_layers, c.num_heads, c.num_kv_heads, c.head_dim, c.ffn_dim, \
            c.max_seq_len = "llama-7b", 32000, 4096, 32, 32, 8, 128, 11008, 4096
    return c


def new_granite_moe_config(size: str = "350m") -> ModelConfig:   # config.go:333-376
    return ModelConfig(architecture="granite", model_name="granite-moe-350m", attention_type="gqa",
                       norm_type="rmsnorm", position_type="rope", activation_type="swiglu",
                       block_style="sequential", rope_base=10000.0, norm_eps=1e-6, tied_embedding=True,
                       use_moe=False, num_experts=32, num_experts_per_tok=8, vocab_size=49155, hidden=1024,
                       num_layers=24, num_heads=16, num_kv_heads=8, head_dim=64, ffn_dim=512, max_seq_len=4096)


def _infer_config_from_json(raw: dict) -> ModelConfig:    # generic_loader.go:975-1007
    mt = raw.get("model_type")
    if mt == "gpt2":
        return new_gpt2_config()
    if mt in ("falcon", "RefinedWeb", "RefinedWebModel"):
        return new_falcon_config("7b")
    if mt in ("llama", "LlamaForCausalLM"):
        return new_llama_config("7b")
    if mt == "granitemoe":
        return new_granite_moe_config("350m")
    if mt == "granitemoehybrid":                        # :993-1001
        hs = raw.get("hidden_size")
        return new_granite_config("350m" if not isinstance(hs, (int, float)) or hs <= 800 else "1b")
    return new_gpt2_config()


def new_granite_config(size: str = "350m") -> ModelConfig:   # config.go:241-330 (Granite-4 hybrid: attention + Mamba2)
    c = ModelConfig(architecture="granite", attention_type="gqa", norm_type="rmsnorm", position_type="nope",
                    activation_type="swiglu", block_style="sequential", rope_base=10000.0, norm_eps=1e-5, tied_embedding=True,
                    mamba_expand=2, mamba_state_size=128, mamba_conv_kernel=4, mamba_num_heads=48)
    if size == "1b":
        c.model_name, c.vocab_size, c.hidden, c.num_layers, c.num_heads, c.num_kv_heads, c.head_dim, c.ffn_dim, \
            c.max_seq_len = "granite-4.0-h-1b", 49152, 1536, 40, 12, 4, 128, 4096, 128000
        c.mamba_n_groups = 8
        c.hybrid_layers = ["mamba"] * 40
    else:
        c.model_name, c.vocab_size, c.hidden, c.num_layers, c.num_heads, c.num_kv_heads, c.head_dim, c.ffn_dim, \
            c.max_seq_len = "granite-4.0-h-350m", 49152, 768, 32, 12, 4, 64, 2048, 32768
        c.mamba_head_dim, c.mamba_n_groups = 32, 1
        c.hybrid_layers = ["attention" if i in (10, 13, 17, 27) else "mamba" for i in range(32)]
    return c


LAYER_FIELDS = dict(mixer="", weights_of=-1, heads=0, dim=0, vdim=0, q_rank=0, kv_rank=0, window=0, scale=0.0, state=0, groups=0,
                    norm_groups=0, conv_taps=0, tau=0.0, decay_rank=0, ffn_dim=0, ffn_limit=0.0, kv_from=-1, rot_dim=0, gate_per_head=0, kv_heads=0,
                    rot_base=0.0, rot_factor=0.0, rot_original=0.0, rot_fast=0.0, rot_slow=0.0, softcap=0.0, v_mix=0, ffn_act=0, experts=0, top_k=0,
                    expert_dim=0, expert_groups=0, groups_kept=0, chunk=0, keep_first=0, qk_norm=0, sink=0, qkv_bias=0, ungated=0, rot_low=0.0, rot_high=0.0,
                    out_scale=0.0, route_softmax=0, expert_limit=0.0, mixer2=0, heads2=0, dim2=0, vdim2=0, out_scale2=0.0, decay=())      # nvl_layer_config
ACT_SWIGLU, ACT_CLAMPED_GLU = 1, 3                                     # NVL_ACT_* (ffn_act)
QK_NORM_HEAD, QK_NORM_ROW = 1, 2                                       # NVL_QK_NORM_*
SINK_ZERO, SINK_LEARNED = 1, 2                                         # NVL_SINK_*
MIXER_LIGHTNING = 5                                                    # NVL_MIXER_LIGHTNING (mixer2)


def _potuzen_layer(e: dict) -> dict:
    """One entry of a Potuzen config.json's layer list -> the fields of nvl_layer_config."""
    mx, mlp, ty = e["mixer"], e.get("mlp"), e["type"]
    out = dict(LAYER_FIELDS, mixer=ty, heads=mx["heads"], vdim=mx["vdim"])
    if e.get("weights_of") is not None:
        out["weights_of"] = e["weights_of"]
    if ty == "latent_attention":
        out.update(dim=mx["dim"], q_rank=mx["q_rank"], kv_rank=mx["kv_rank"], scale=float(mx["scale"]), window=(mx.get("mask") or {}).get("size", 0))
    elif ty == "mamba2":
        out.update(state=mx["state"], groups=mx["groups"], norm_groups=mx["norm_groups"], conv_taps=mx["conv"])
    elif ty == "gla":
        out.update(dim=mx["dim"], tau=float(mx["tau"]))
    else:
        raise ValueError(f"unknown mixer {ty!r}")
    if mlp is not None:
        if mlp.get("kind", "dense") != "dense":
            raise ValueError(f"unknown feed-forward kind {mlp['kind']!r}")
        out["ffn_dim"] = mlp["ff"]
    return out


def potuzen_config(raw: dict) -> ModelConfig:
    """The Potuzen design: a list of layers (latent attention / Mamba-2 / gated linear attention), sandwich norms, GEGLU.  The
    file names no longest sequence: 4096, as the library's own reader sets it; override max_seq_len as needed."""
    return ModelConfig(architecture="Potuzen", model_name="potuzen", vocab_size=raw["vocab"], hidden=raw["width"],
                       num_layers=len(raw["layers"]), max_seq_len=4096, attention_type="gqa", norm_type="rmsnorm", position_type="nope",
                       activation_type="geglu", block_style="sandwich", rope_base=0.0, norm_eps=float(raw["norm"]["eps"]),
                       layers=[_potuzen_layer(e) for e in raw["layers"]])


def _lufazen_layer(e: dict) -> dict:
    """One entry of a Lufazen config.json's layer list -> the fields of nvl_layer_config."""
    mx, mlp, ty = e["mixer"], e.get("mlp"), e["type"]
    out = dict(LAYER_FIELDS, mixer=ty, heads=mx["heads"], dim=mx["dim"], vdim=mx["vdim"])
    if ty == "latent_attention":
        rot = mx["rot"]
        if rot["dims"] != mx["rot_dim"]:
            raise ValueError("rot.dims differs from rot_dim")
        out.update(q_rank=mx["q_rank"], kv_rank=mx["kv_rank"], scale=float(mx["scale"]), rot_dim=mx["rot_dim"], gate_per_head=1, rot_base=float(rot["base"]))
        if mx.get("kv_from") is not None:
            out["kv_from"] = mx["kv_from"]
        if rot.get("scaling") is not None:
            out.update({"rot_" + k: float(rot["scaling"][k]) for k in ("factor", "original", "fast", "slow")})
    elif ty == "channel_delta":
        out.update(kv_heads=mx["kv_heads"], conv_taps=mx["conv"])
    else:
        raise ValueError(f"unknown mixer {ty!r}")
    if mlp is not None:
        if mlp.get("kind", "dense") != "dense":
            raise ValueError(f"unknown feed-forward kind {mlp['kind']!r}")
        out.update(ffn_dim=mlp["ff"], ffn_limit=float(mlp["limit"]))
    return out


def lufazen_config(raw: dict) -> ModelConfig:
    """The Lufazen design: a list of layers (rotated latent attention / channel-wise gated delta rule), norms on the sublayers' outputs
    whose weights are kept as differences from one, layer scales, clamped gated feed-forwards, capped logits."""
    return ModelConfig(architecture="Lufazen", model_name="lufazen", vocab_size=raw["vocab"], hidden=raw["width"],
                       num_layers=len(raw["layers"]), max_seq_len=4096, attention_type="gqa", norm_type="rmsnorm", position_type="nope",
                       activation_type="clamped_glu", block_style="post", rope_base=0.0, norm_eps=float(raw["norm"]["eps"]),
                       norm_weight_offset=1.0, logit_softcap=float(raw.get("logit_softcap") or 0.0), layers=[_lufazen_layer(e) for e in raw["layers"]])


def _bolinex_layer(e: dict) -> dict:
    """One entry of a Bolinex config.json's layer list -> the fields of nvl_layer_config."""
    mx, mlp, ty = e["mixer"], e.get("mlp"), e["type"]
    if ty != "attention":
        raise ValueError(f"unknown mixer {ty!r}")
    out = dict(LAYER_FIELDS, mixer=ty, heads=mx["heads"], kv_heads=mx["kv_heads"], dim=mx["dim"], vdim=mx["vdim"], scale=float(mx["scale"]),
               softcap=float(mx.get("softcap") or 0.0), v_mix=int(bool(mx.get("v_mix"))), window=(mx.get("mask") or {}).get("size", 0))
    if mlp is None:
        return out
    kind = mlp.get("kind", "dense")
    if kind == "moe":
        ro, groups = mlp["router"], mlp["router"].get("groups") or dict(count=1, keep=1)
        out.update(expert_dim=mlp["expert"]["ff"], experts=ro["experts"], top_k=ro["top"], expert_groups=groups["count"], groups_kept=groups["keep"],
                   ffn_dim=(mlp.get("shared") or {}).get("ff", 0), ffn_act=ACT_SWIGLU)
    elif kind == "dense":
        out["ffn_dim"] = mlp["ff"]
    else:
        raise ValueError(f"unknown feed-forward kind {kind!r}")
    return out


def bolinex_config(raw: dict) -> ModelConfig:
    """The Bolinex design: parallel blocks behind one layer norm, grouped-query attention (capped scores, logarithmic distance bias,
    windows, mixed values, output gate), squared-ReLU or expert feed-forwards, learned positions, per-layer token inputs."""
    return ModelConfig(architecture="Bolinex", model_name="bolinex", vocab_size=raw["vocab"], hidden=raw["width"],
                       num_layers=len(raw["layers"]), max_seq_len=raw["max_positions"], attention_type="gqa", norm_type="layernorm", position_type="learned",
                       activation_type="relu2", block_style="parallel", rope_base=0.0, norm_eps=float(raw["norm"]["eps"]),
                       side_dim=(raw.get("token_side") or {}).get("dim", 0), layers=[_bolinex_layer(e) for e in raw["layers"]])


def _medulorn_attention(mx: dict) -> dict:
    """What the two attentions of the Medulorn design have in common."""
    out = dict(heads=mx["heads"], kv_heads=mx["kv_heads"], dim=mx["dim"], vdim=mx["vdim"], scale=float(mx["scale"]), ungated=1)
    rot = mx.get("rot")
    if rot is not None:
        out.update(rot_dim=rot["dims"], rot_base=float(rot["base"]))
        sc = rot.get("scaling")
        if sc is not None:
            out.update({"rot_" + k: float(sc[k]) for k in ("factor", "original", "low", "high")})
    return out


def _medulorn_layer(e: dict) -> dict:
    """One entry of a Medulorn config.json's layer list -> the fields of nvl_layer_config."""
    mx, mlp, ty = e["mixer"], e.get("mlp"), e["type"]
    out = dict(LAYER_FIELDS, mixer="attention")
    if ty == "attention":
        out.update(_medulorn_attention(mx), qk_norm=QK_NORM_HEAD, sink=SINK_ZERO, qkv_bias=1, chunk=(mx.get("mask") or {}).get("size", 0))
    elif ty == "parallel":
        left, right = mx["left"], mx["right"]
        mask = left.get("mask") or {}
        if len(right["decay"]) != right["heads"]:
            raise ValueError("as many decays as heads expected")
        out.update(_medulorn_attention(left), qk_norm=QK_NORM_ROW, sink=SINK_LEARNED, window=mask.get("size", 0), keep_first=mask.get("keep_first") or 0,
                   out_scale=float(mx["left_scale"]), mixer2=MIXER_LIGHTNING, heads2=right["heads"], dim2=right["dim"], vdim2=right["vdim"],
                   out_scale2=float(mx["right_scale"]), decay=[float(d) for d in right["decay"]])
    else:
        raise ValueError(f"unknown mixer {ty!r}")
    if mlp is None:
        return out
    kind = mlp.get("kind", "dense")
    if kind == "moe":
        out.update(expert_dim=mlp["expert"]["ff"], expert_limit=float(mlp["expert"]["limit"]), experts=mlp["router"]["experts"], top_k=mlp["router"]["top"],
                   expert_groups=1, groups_kept=1, route_softmax=1)
        if mlp.get("shared") is not None:
            out.update(ffn_dim=mlp["shared"]["ff"], ffn_limit=float(mlp["shared"]["limit"]), ffn_act=ACT_CLAMPED_GLU)
    elif kind == "dense":
        out["ffn_dim"] = mlp["ff"]
    else:
        raise ValueError(f"unknown feed-forward kind {kind!r}")
    return out


def medulorn_config(raw: dict) -> ModelConfig:
    """The Medulorn design: norms (one weight each) of alpha x + f(x), token shift in front of every mixer, chunked attention, and windowed
    attention beside lightning attention; ReLU-gated or expert feed-forwards, capped logits."""
    return ModelConfig(architecture="Medulorn", model_name="medulorn", vocab_size=raw["vocab"], hidden=raw["width"],
                       num_layers=len(raw["layers"]), max_seq_len=4096, attention_type="gqa", norm_type="rmsnorm_scalar", position_type="nope",
                       activation_type="reglu", block_style="sum_norm", rope_base=0.0, norm_eps=float(raw["norm"]["eps"]),
                       embedding_multiplier=float(raw["embedding"]["scale"]), stream_scale=float(raw["postln_alpha"]), token_shift=1,
                       logit_softcap=float(raw.get("logit_softcap") or 0.0), layers=[_medulorn_layer(e) for e in raw["layers"]])


LAYERED = {"Medulorn": medulorn_config, "Potuzen": potuzen_config, "Lufazen": lufazen_config, "Bolinex": bolinex_config}      # architectures described by a list of layers


def load_model_config(raw: dict | str) -> ModelConfig:
    """LoadModelConfig (generic_loader.go:808-972) on an already-parsed HF config.json (or its text).
    Reference quirks kept: max_position_embeddings and rope_scaling are never read, so max_seq_len
    stays the template's constant and Llama-3 RoPE frequency scaling is not applied."""
    if isinstance(raw, str):
        raw = json.loads(raw)
    arch = raw.get("architecture")
    if arch in LAYERED:
        return LAYERED[arch](raw)
    if arch == "gpt2":
        c = new_gpt2_config()
    elif arch == "falcon":
        c = new_falcon_config("7b")
    elif arch == "llama":
        c = new_llama_config("7b")
    else:
        c = _infer_config_from_json(raw)

    def num(key):
        v = raw.get(key)
        return v if isinstance(v, (int, float)) and not isinstance(v, bool) else None

    for key, attr in (("vocab_size", "vocab_size"), ("n_embd", "hidden"), ("hidden_size", "hidden"),
                      ("n_layer", "num_layers"), ("num_hidden_layers", "num_layers"), ("num_layers", "num_layers"),
                      ("n_head", "num_heads"), ("num_attention_heads", "num_heads"), ("num_heads", "num_heads"),
                      ("num_key_value_heads", "num_kv_heads"), ("num_kv_heads", "num_kv_heads")):
        v = num(key)
        if v is not None:
            setattr(c, attr, int(v))
    if raw.get("multi_query") is True:
        c.num_kv_heads = 1
    v = num("head_dim")
    if v is not None:
        c.head_dim = int(v)
    if c.head_dim == 0 and c.hidden > 0 and c.num_heads > 0:
        c.head_dim = c.hidden // c.num_heads
    for key, attr in (("eos_token_id", "eos_token_id"), ("bos_token_id", "bos_token_id"),
                      ("pad_token_id", "pad_token_id")):
        v = num(key)
        if v is not None:
            setattr(c, attr, int(v))
    v = num("rope_theta")
    if v is not None:
        c.rope_base = float(v)
    for key in ("rms_norm_eps", "layer_norm_epsilon"):
        v = num(key)
        if v is not None:
            c.norm_eps = float(v)
    for key in ("n_inner", "intermediate_size"):
        v = num(key)
        if v is not None:
            c.ffn_dim = int(v)
    if c.ffn_dim == 0 and c.hidden > 0:
        c.ffn_dim = 4 * c.hidden
    if isinstance(raw.get("tie_word_embeddings"), bool):
        c.tied_embedding = raw["tie_word_embeddings"]
    for key in ("embedding_multiplier", "attention_multiplier", "residual_multiplier", "logits_scaling"):
        v = num(key)
        if v is not None:
            setattr(c, key, float(v))
    if isinstance(raw.get("layer_types"), list):          # :917-925
        c.hybrid_layers = [t if isinstance(t, str) else "" for t in raw["layer_types"]]
    for key, attr in (("mamba_expand", "mamba_expand"), ("mamba_d_state", "mamba_state_size"), ("mamba_n_heads", "mamba_num_heads"),
                      ("mamba_d_head", "mamba_head_dim"), ("mamba_n_groups", "mamba_n_groups"), ("mamba_d_conv", "mamba_conv_kernel")):
        v = num(key)
        if v is not None:
            setattr(c, attr, int(v))
    v = num("num_local_experts")
    if v is not None:
        c.num_experts = int(v)
        # (reference: UseMoE = true for ANY value, 0 included; a hybrid checkpoint says 0 and runs the dense shared MLP —
        # the device library treats 0 experts as "no MoE", and so does this mirror)
        c.use_moe = v > 0
    v = num("num_experts_per_tok")
    if v is not None:
        c.num_experts_per_tok = int(v)
    return c
