// layered.h — models described by a list of layers (nvl_layer_config): every layer names a mixer (latent attention, Mamba-2, gated
// linear attention, channel-wise delta rule, grouped-query attention, the last also with lightning attention beside it), its sizes and its
// feed-forward, with a norm before and after each sublayer (NVL_BLOCK_SANDWICH), after it only (NVL_BLOCK_POST: the sublayers read the
// residual stream itself), of the scaled stream and the sublayer's result together (NVL_BLOCK_SUM_NORM: likewise), or one norm that both
// sublayers read (NVL_BLOCK_PARALLEL).  Host side: creation, tensor staging, freezing into the kernels' layouts, the layer stack of one
// forward pass.  Included by nvllm.hip.
//
// A parallel block's two sublayers end in ONE projection: their operands sit side by side in m->lmix (kd = ko + Fp columns) and W_o
// and W_down side by side in one matrix.  The feed-forward is dense, or a mixture of experts whose shared expert takes the dense one's
// place; the experts' sum joins in the launch that completes the residual.  A per-layer token input (side_dim) follows:
// x += rms(P (gelu(G x) * e_token)) * w.
//
// Two mixers side by side (mixer2) share ONE projection in and ONE out: their operands sit side by side in m->lmix, W_o and W_o2 side by
// side in one matrix, and the factors of their results are applied, in fp32, as the operands are written.
//
// What differs from the fixed-shape models around it:
//   * widths need not be multiples of 64: rows, heads and latents are padded with zeros when the tensors are frozen (m->H is the
//     padded row, m->Hn the real one), so the GEMM and norm kernels run unchanged;
//   * the cache of a sequence is a slot (recurrent states, convolution rows) plus blocks of the library's pool (latents); blocks
//     that no window reaches any more go back to the pool while the sequence runs (pool_trim);
//   * a batch may mix prompt portions and single tokens: latent attention takes the absorbed form for sequences with up to
//     LAT_ABSORB_MAX new tokens and the expanded form for the rest, grouped attention its short form up to GROUPED_SHORT_ROWS
//     query rows; recurrences go token by token up to REC_STEP_MAX.
#pragma once

static int g_grouped_split = 0;      // nvl_set_tuning key 37: key splits of the short grouped attention (1 .. 16); 0 = automatic

namespace {

constexpr int LAT_ABSORB_MAX = 16, LAT_ABSORB_MAX_RP = 512, REC_STEP_MAX = 4;
constexpr int GLU_IN_MAX = 1024;       // widest shared expert whose gate and up columns pass through fp32 rows instead of a launch of their own
constexpr int SHARED_PARTS_MAX = 16;   // widest shared expert, in experts, that joins the masked experts of a decode step
constexpr int GROUPED_SHORT_ROWS = 64, GROUPED_SPLIT_WGS = 512;      // GROUPED_SPLIT_WGS: workgroups of a launch whose keys are split

bool same_rotation(const nvl_layer_config& a, const nvl_layer_config& b) {
    return a.rot_dim == b.rot_dim && a.rot_base == b.rot_base && a.rot_factor == b.rot_factor && a.rot_original == b.rot_original &&
           a.rot_fast == b.rot_fast && a.rot_slow == b.rot_slow && a.rot_low == b.rot_low && a.rot_high == b.rot_high;
}
// unrotated (padded to 32) + rotated part; d + rot = 192 with 256 value channels has no LDS left for its ring of tiles
int pad_rotated(int d, int vp) {
    for (int p : {32, 64, 96, 128, 192, 256}) if (d <= p && !(p == 192 && vp > 128)) return p;
    return (int)round_up(d, 64);
}
int pad_head(int d, int unit) {       // head sizes the attention instances exist for; larger ones take the plain kernel
    for (int p : {32, 64, 128, 256}) if (d <= p) return p;
    return (int)round_up(d, unit);
}

// ------------------------------------------------------------------------------------------
// creation
// ------------------------------------------------------------------------------------------
int layered_create(const nvl_model_config& c, const nvl_layer_config* layers, const nvl_runtime_opts& opts, nvl_model** out) {
    auto bad = [&](const std::string& why) { return fail(nullptr, NVL_ERR_INVALID, "nvl_create_layers: " + why); };
    const bool par = c.block_style == NVL_BLOCK_PARALLEL, sum = c.block_style == NVL_BLOCK_SUM_NORM;
    if (c.block_style != NVL_BLOCK_SANDWICH && c.block_style != NVL_BLOCK_POST && !par && !sum) return bad("block_style NVL_BLOCK_SANDWICH, _POST, _PARALLEL or _SUM_NORM expected");
    auto act_ok = [&](int a) { return par ? a == NVL_ACT_RELU2 || a == NVL_ACT_SWIGLU : a == (sum ? NVL_ACT_REGLU : NVL_ACT_GEGLU) || a == NVL_ACT_CLAMPED_GLU; };
    if (!act_ok(c.activation_type)) return bad("activation_type does not fit the block style (NVL_ACT_GEGLU, NVL_ACT_CLAMPED_GLU; parallel: NVL_ACT_RELU2, NVL_ACT_SWIGLU; norms of sums: NVL_ACT_REGLU, NVL_ACT_CLAMPED_GLU)");
    if (sum && !(c.stream_scale != 0.f)) return bad("stream_scale is zero");
    if (c.token_shift && !sum && c.block_style != NVL_BLOCK_POST) return bad("token_shift needs mixers that read the residual stream itself");
    if (!par && ((c.norm_type != NVL_NORM_RMS && c.norm_type != NVL_NORM_RMS_SCALAR) || c.position_type != NVL_POS_NONE || c.side_dim)) return bad("layer norms, learned positions and side_dim need NVL_BLOCK_PARALLEL");
    if ((c.norm_type != NVL_NORM_RMS && c.norm_type != NVL_NORM_RMS_SCALAR && c.norm_type != NVL_NORM_LAYER) || (c.position_type != NVL_POS_NONE && c.position_type != NVL_POS_LEARNED)) return bad("bad norm_type / position_type");
    if (c.norm_type == NVL_NORM_LAYER && c.norm_weight_offset != 0.f) return bad("layer norms take their weights as they are");
    if (c.side_dim < 0 || c.side_dim > 8192) return bad("bad side_dim");
    if (!(c.logit_softcap >= 0.f)) return bad("logit_softcap is negative");
    if (c.hidden <= 0 || c.num_layers <= 0 || c.vocab_size <= 0 || c.max_seq_len <= 0) return bad("non-positive model dimension");
    if (c.hidden > 20480) return bad("hidden larger than 20480");
    if (opts.max_seqs <= 0) return bad("max_seqs must be >= 1");
    if (opts.max_batch_tokens < 0 || opts.kv_num_blocks < 0 || opts.kv_block_size < 0 || opts.kv_block_size % 64) return bad("bad max_batch_tokens / kv_num_blocks / kv_block_size");
    if (opts.tp_size > 1 || opts.tp_force_single) return bad("tensor parallelism does not cover models described by a list of layers");
    const int L = c.num_layers;
    for (int i = 0; i < L; i++) {
        const nvl_layer_config& l = layers[i];
        const std::string at = "layer " + std::to_string(i) + ": ";
        if (l.heads <= 0 || l.vdim <= 0 || l.vdim > 2048 || l.ffn_dim < 0) return bad(at + "bad heads / vdim / ffn_dim");
        if (l.ffn_dim && (l.ffn_act ? l.ffn_act : c.activation_type) == NVL_ACT_CLAMPED_GLU && !(l.ffn_limit > 0.f)) return bad(at + "ffn_limit is not positive");
        if (l.ffn_act && !act_ok(l.ffn_act)) return bad(at + "ffn_act does not fit the block style");
        if (l.experts) {
            if (!par && !sum) return bad(at + "experts need NVL_BLOCK_PARALLEL or NVL_BLOCK_SUM_NORM");
            if (!(l.expert_limit >= 0.f)) return bad(at + "expert_limit is negative");
            if (l.route_softmax && l.expert_groups != 1) return bad(at + "softmax routing has no expert groups");
            if (par && (l.route_softmax || l.expert_limit > 0.f)) return bad(at + "softmax routing and clamped experts need NVL_BLOCK_SUM_NORM");
            if (l.experts < 0 || l.experts > std::min(MOE_MAX_E, ROUTE_MAX_E) || l.expert_dim <= 0 || l.expert_groups <= 0 || l.experts % l.expert_groups || l.groups_kept <= 0 ||
                l.groups_kept > l.expert_groups || l.top_k <= 0 || l.top_k > l.groups_kept * (l.experts / l.expert_groups)) return bad(at + "bad expert sizes");
        }
        if (l.mixer != NVL_MIXER_ATTENTION && (l.chunk || l.keep_first || l.qk_norm || l.sink || l.qkv_bias || l.ungated || l.mixer2)) return bad(at + "chunks, kept tokens, query/key norms, sinks, biases and a second mixer belong to NVL_MIXER_ATTENTION");
        if (l.rot_dim < 0 || l.rot_dim % 2 || l.rot_dim > 1024 || (l.rot_dim && !(l.rot_base > 1.0)) || (l.rot_factor != 0.0 && !(l.rot_factor > 0.0 && l.rot_original > 0.0)) ||
            (l.rot_high != 0.0 ? !(l.rot_factor > 0.0 && l.rot_low > 0.0 && l.rot_high > l.rot_low) : l.rot_factor != 0.0 && !(l.rot_fast > 0.0 && l.rot_slow > 0.0))) return bad(at + "bad rotation");
        switch (l.mixer) {
            case NVL_MIXER_LATENT_ATTENTION:
                if (l.kv_from >= 0) {
                    if (l.kv_from >= i) return bad(at + "kv_from names no earlier layer");
                    const nvl_layer_config& s = layers[l.kv_from];
                    if (s.mixer != l.mixer || s.kv_from >= 0) return bad(at + "kv_from names a layer without latents of its own");
                    if (s.kv_rank != l.kv_rank || !same_rotation(s, l)) return bad(at + "kv_from names a layer with another latent or rotation");
                }
                if (l.dim <= 0 || l.q_rank <= 0 || l.kv_rank <= 0 || l.window < 0 || l.dim > 2048) return bad(at + "bad latent attention sizes");
                break;
            case NVL_MIXER_MAMBA2:
                if (l.state <= 0 || l.state > 2048 || l.groups <= 0 || l.heads % l.groups || l.conv_taps <= 0 || l.norm_groups <= 0 ||
                    (l.heads * l.vdim) % l.norm_groups) return bad(at + "bad Mamba-2 sizes");
                break;
            case NVL_MIXER_GLA:
                if (l.dim <= 0 || l.dim > 2048 || !(l.tau > 0.f) || l.decay_rank < 0) return bad(at + "bad gated linear attention sizes");
                break;
            case NVL_MIXER_CHANNEL_DELTA:
                if (l.dim <= 0 || l.dim > 2048 || l.kv_heads <= 0 || l.heads % l.kv_heads || l.conv_taps <= 0 || l.decay_rank < 0) return bad(at + "bad channel delta sizes");
                break;
            case NVL_MIXER_ATTENTION: {
                if (l.dim <= 0 || l.dim > 2048 || l.kv_heads <= 0 || l.heads % l.kv_heads || l.window < 0 || !(l.softcap >= 0.f)) return bad(at + "bad attention sizes");
                if (l.chunk < 0 || l.keep_first < 0 || (l.chunk && l.window) || (l.keep_first && !l.window) || l.rot_dim > l.dim || l.qk_norm < 0 || l.qk_norm > NVL_QK_NORM_ROW || l.sink < 0 || l.sink > NVL_SINK_LEARNED)
                    return bad(at + "bad key mask, rotation, query/key norm or sink");
                if (!l.ungated && (l.qk_norm || l.rot_dim || l.mixer2 || l.qkv_bias)) return bad(at + "normed, rotated or biased attention, and attention beside a second mixer, has no output gate");
                if (l.mixer2) {
                    if (l.mixer2 != NVL_MIXER_LIGHTNING || par) return bad(at + "the second mixer is not NVL_MIXER_LIGHTNING (or in a parallel block)");
                    if (l.heads2 <= 0 || l.heads2 > NVL_MAX_DECAYS || l.dim2 <= 0 || l.dim2 > 2048 || l.vdim2 <= 0 || l.vdim2 > 2048) return bad(at + "bad lightning attention sizes");
                    for (int h = 0; h < l.heads2; h++) if (!(l.decay[h] >= 0.0 && l.decay[h] <= 1.0)) return bad(at + "a decay is not between 0 and 1");
                }
                for (int j = 0; j < i && l.v_mix; j++)
                    if (layers[j].mixer == l.mixer && layers[j].v_mix && (layers[j].kv_heads != l.kv_heads || layers[j].vdim != l.vdim)) return bad(at + "mixes values of another shape");
                break;
            }
            default: return bad(at + "unknown mixer");
        }
        if (l.weights_of >= L || l.weights_of == i) return bad(at + "weights_of names no other layer");
    }
    std::vector<int> owner((size_t)L);
    for (int i = 0; i < L; i++) {
        int o = i, hops = 0;
        while (layers[o].weights_of >= 0) { o = layers[o].weights_of; if (++hops > L) return bad("weights_of goes round in a circle"); }
        owner[(size_t)i] = o;
        const nvl_layer_config &a = layers[i], &b = layers[o];
        if (a.mixer != b.mixer || a.heads != b.heads || a.dim != b.dim || a.vdim != b.vdim || a.q_rank != b.q_rank || a.kv_rank != b.kv_rank ||
            a.state != b.state || a.groups != b.groups || a.conv_taps != b.conv_taps || a.ffn_dim != b.ffn_dim || a.rot_dim != b.rot_dim ||
            a.kv_heads != b.kv_heads || a.qk_norm != b.qk_norm || a.sink != b.sink || a.qkv_bias != b.qkv_bias || a.ungated != b.ungated || a.out_scale2 != b.out_scale2 ||
            a.mixer2 != b.mixer2 || a.heads2 != b.heads2 || a.dim2 != b.dim2 || a.vdim2 != b.vdim2 || memcmp(a.decay, b.decay, sizeof a.decay) || a.gate_per_head != b.gate_per_head || a.experts != b.experts || a.expert_dim != b.expert_dim || a.v_mix != b.v_mix || a.ffn_act != b.ffn_act || (i != o && a.mixer == NVL_MIXER_LATENT_ATTENTION && (a.kv_from >= 0) != (b.kv_from >= 0)))
            return bad("layer " + std::to_string(i) + " does not have the shape of the layer whose tensors it uses");
    }
    if (opts.device < 0 || nvl_device_count() <= opts.device) return fail(nullptr, NVL_ERR_NO_DEVICE, "nvl_create_layers: no HIP device (this library has no CPU fallback)");
    nvl_model* m = new (std::nothrow) nvl_model();
    if (!m) return fail(nullptr, NVL_ERR_OOM, "nvl_create_layers: out of host memory");
    try {
        m->cfg = c; m->opts = opts; m->layered = true;
        m->cfg.attention_type = NVL_ATTN_GQA; m->cfg.use_moe = 0;
        m->f32 = opts.precision == NVL_PRECISION_F32;
        m->wsize = m->f32 ? 4 : 2;
        m->device = opts.device;
        NVL_HIP(hipSetDevice(m->device));
        NVL_HIP(hipStreamCreateWithFlags(&m->stream, hipStreamNonBlocking));
        NVL_HIP(hipEventCreate(&m->ev0));
        NVL_HIP(hipEventCreate(&m->ev1));
        m->Hn = c.hidden; m->H = (int)round_up(c.hidden, 64); m->V = c.vocab_size; m->Vpad = (int)round_up(m->V, 128); m->L = L;
        m->nH = m->nKV = 1; m->hd = 64; m->nH_full = m->nKV_full = 1;      // (unused by the layer stack)
        m->layers.resize((size_t)L);
        m->runs.resize((size_t)L); m->mixers.resize((size_t)L);
        if (m->opts.max_batch_tokens <= 0) m->opts.max_batch_tokens = std::min(c.max_seq_len, 4096);
        int64_t state = 0, cache = 0;
        const int bs = opts.kv_block_size > 0 ? opts.kv_block_size : (opts.kv_num_blocks > 0 ? 256 : 64);
        for (int i = 0; i < L; i++) {
            LayerRun& r = m->runs[(size_t)i];
            r.c = layers[i]; r.owner = owner[(size_t)i];
            r.Fp = (int)round_up(r.c.ffn_dim, 64);
            r.act = r.c.ffn_act ? r.c.ffn_act : c.activation_type;
            if (c.token_shift) { r.shift_off = state; state += m->H; }
            if (r.c.experts) {      // padded so that a wave of the decode down projection owns one expert, at most 16 of them a workgroup
                r.Ip = (int)round_up(r.c.expert_dim, 64);
                if (sum && r.c.ffn_dim && r.act == NVL_ACT_CLAMPED_GLU && r.c.expert_limit > 0.f && cdiv(r.Fp, r.Ip) <= SHARED_PARTS_MAX) r.shared_parts = cdiv(r.Fp, r.Ip);
                const int all = r.c.experts + r.shared_parts;
                r.Ep = (int)round_up(all, all <= 32 ? 2 : 16); r.moe_slices = r.Ep <= 32 ? 2 : r.Ep / 16;
            }
            if (r.c.mixer == NVL_MIXER_LATENT_ATTENTION || r.c.mixer == NVL_MIXER_ATTENTION) {
                const KeyMask mask{r.c.window, r.c.chunk, r.c.keep_first};
                size_t w = 0;
                while (w < m->masks.size() && !(m->masks[w] == mask)) w++;
                if (w == m->masks.size()) m->masks.push_back(mask);
                r.win = (int)w;
            }
            const int H = r.c.heads;
            if (r.c.mixer == NVL_MIXER_LATENT_ATTENTION) {
                r.vp = pad_head(r.c.vdim, 64);
                r.rotp = (int)round_up(r.c.rot_dim, 32);
                r.dp = r.rotp ? pad_rotated((int)round_up(r.c.dim, 32) + r.rotp, r.vp) : pad_head(r.c.dim, 64);
                r.dn = r.dp - r.rotp;
                r.src = r.c.kv_from >= 0 ? r.c.kv_from : i;
                r.qrp = (int)round_up(r.c.q_rank, 64); r.rp = (int)round_up(r.c.kv_rank, 64);
                if (r.rp > 256 && r.rp < 512) r.rp = r.rp <= 384 ? 384 : 512;       // (instances of the absorbed form)
                r.gate_off = r.qrp + (r.src == i ? r.rp + r.rotp : 0);
                r.n_in = r.gate_off + (r.c.gate_per_head ? H : H * r.vp); r.ko = (int)round_up((int64_t)H * r.vp, 64);
                if (r.src == i) { r.cache_off = cache; cache += (int64_t)bs * (r.rp + r.rotp); }
                else r.cache_off = m->runs[(size_t)r.src].cache_off;
            } else if (r.c.mixer == NVL_MIXER_ATTENTION) {
                const int G = r.c.kv_heads;
                r.dp = pad_head(r.c.dim, 64); r.vp = pad_head(r.c.vdim, 64);
                r.k_off = H * r.dp; r.v_off = r.k_off + G * r.dp; r.gate_off = r.v_off + G * r.vp; r.ffn_off = r.gate_off + (r.c.ungated ? 0 : H * r.vp);
                r.raw = r.c.qk_norm || r.c.rot_dim || r.c.mixer2;
                r.ffn_in = par && r.c.ffn_dim && r.act == NVL_ACT_RELU2;
                r.glu_in = par && r.c.experts && r.c.ffn_dim && r.act == NVL_ACT_SWIGLU && r.Fp <= GLU_IN_MAX;
                r.route_off = r.ffn_off + (r.ffn_in ? r.Fp : r.glu_in ? 2 * r.Fp : 0);
                r.n_in = r.route_off + (par ? r.c.experts : 0); r.ko = (int)round_up((int64_t)H * r.vp, 64);
                if (r.c.mixer2) {
                    const int qk = (int)round_up(r.c.heads2 * r.c.dim2, 4), v = (int)round_up(r.c.heads2 * r.c.vdim2, 4);
                    r.lq_off = r.ffn_off; r.lk_off = r.lq_off + qk; r.lv_off = r.lk_off + qk; r.lg_off = r.lv_off + v;
                    r.n_in = r.lg_off + r.c.heads2 * r.c.vdim2;
                    r.ko2 = (int)round_up((int64_t)r.c.heads2 * r.c.vdim2, 64);
                    r.state_off = state; state += round_up((int64_t)r.c.heads2 * r.c.dim2 * round_up(r.c.vdim2, 4), 64);
                }
                r.cache_off = cache; cache += (int64_t)bs * G * (r.dp + r.vp);
                if (r.c.v_mix) {
                    r.mix = m->lvf_ld ? 2 : 1;
                    m->lvf_ld = (int64_t)G * r.vp;
                }
            } else {
                const int DVp = (int)round_up(r.c.vdim, 4), DK = r.c.mixer == NVL_MIXER_MAMBA2 ? r.c.state : r.c.dim;
                r.ko = (int)round_up((int64_t)H * r.c.vdim, 64);
                r.state_off = state; state += round_up((int64_t)H * DK * DVp, 64);
                if (r.c.mixer == NVL_MIXER_MAMBA2) {
                    r.conv_dim = H * r.c.vdim + 2 * r.c.groups * r.c.state;
                    r.n_in = H * r.c.vdim + r.conv_dim + H;
                    r.ring_off = state; state += round_up((int64_t)r.c.conv_taps * r.conv_dim, 64);
                } else if (r.c.mixer == NVL_MIXER_CHANNEL_DELTA) {
                    r.conv_dim = 2 * r.c.kv_heads * r.c.dim + H * r.c.vdim;
                    r.ring_off = state; state += round_up((int64_t)r.c.conv_taps * r.conv_dim, 64);
                }       // (GLA, channel delta: n_in follows from the decay rank, layered_finalize)
            }
            r.kd = r.ko + r.ko2 + (par ? r.Fp : 0);
        }
        m->lat_block_stride = cache; m->rec_slot_stride = state;
        m->pool = 1; m->Tmax = bs; m->blocks_per_seq = cdiv(c.max_seq_len, bs);
        if (opts.kv_num_blocks > 0) m->num_blocks = opts.kv_num_blocks;
        else {      // what every slot can hold at once: its window and the tokens of the call that is running
            int64_t span = c.max_seq_len;
            int w = 0;
            bool windowed = true;
            for (const KeyMask& x : m->masks) { w = std::max(w, x.span() + (int)round_up(x.keep, bs)); windowed &= x.span() > 0; }
            if (windowed) span = std::min<int64_t>(span, (int64_t)w + m->opts.max_batch_tokens + 2 * bs);
            m->num_blocks = opts.max_seqs * cdiv(span, bs);
        }
        m->table_cap = opts.max_seqs * m->blocks_per_seq;
        *out = m;
        return NVL_OK;
    } catch (const HipError& e) {
        const std::string s = std::string("nvl_create_layers: HIP error: ") + hipGetErrorString(e.code);
        delete m;
        return fail(nullptr, NVL_ERR_HIP, s);
    } catch (const std::exception& e) {
        const std::string s = e.what();
        delete m;
        return fail(nullptr, NVL_ERR_INVALID, s);
    }
}

// ------------------------------------------------------------------------------------------
// tensors: staged on the device in the checkpoint's dtype, placed into the kernels' layouts by layered_finalize
// ------------------------------------------------------------------------------------------
void layered_shape(const nvl_model* m, int kind, int layer, int64_t& N, int64_t& K) {     // N = 0: the model has no such tensor; K = 1: a vector
    const int64_t W = m->Hn, W1 = m->cfg.norm_type == NVL_NORM_RMS_SCALAR ? 1 : W;
    N = 0; K = 1;
    switch (kind) {
        case NVL_T_TOK_EMB: case NVL_T_LM_HEAD: N = m->V; K = W; return;
        case NVL_T_FINAL_NORM_W: N = W1; return;
        case NVL_T_FINAL_NORM_B: if (m->cfg.norm_type == NVL_NORM_LAYER) N = W; return;
        case NVL_T_POS_EMB: if (m->cfg.position_type == NVL_POS_LEARNED) { N = -1; K = W; } return;
        case NVL_T_SIDE_EMB: if (m->cfg.side_dim) { N = m->V; K = (int64_t)m->L * m->cfg.side_dim; } return;
        default: if (is_global(kind)) return;
    }
    const LayerRun& r = m->runs[(size_t)layer];
    const nvl_layer_config& c = r.c;
    if (r.owner != layer) return;
    const bool sum = m->cfg.block_style == NVL_BLOCK_SUM_NORM, post = m->cfg.block_style == NVL_BLOCK_POST, par = m->cfg.block_style == NVL_BLOCK_PARALLEL, delta = c.mixer == NVL_MIXER_CHANNEL_DELTA;
    const bool att = c.mixer == NVL_MIXER_ATTENTION, lat = c.mixer == NVL_MIXER_LATENT_ATTENTION, mam = c.mixer == NVL_MIXER_MAMBA2, gla = c.mixer == NVL_MIXER_GLA;
    const int64_t hv = (int64_t)c.heads * c.vdim, hd = (int64_t)c.heads * c.dim;
    switch (kind) {
        case NVL_T_ATTN_NORM_W: if (!post && !sum) N = W1; return;
        case NVL_T_FFN_NORM_W: if (!post && !par && !sum) N = W1; return;
        case NVL_T_ATTN_NORM_B: if (m->cfg.norm_type == NVL_NORM_LAYER) N = W; return;
        case NVL_T_MIX_POST_NORM: case NVL_T_FFN_POST_NORM: if (!par) N = W1; return;
        case NVL_T_SHIFT: if (m->cfg.token_shift) N = W; return;
        case NVL_T_SIDE_GATE: if (m->cfg.side_dim) { N = m->cfg.side_dim; K = W; } return;
        case NVL_T_SIDE_PROJ: if (m->cfg.side_dim) { N = W; K = m->cfg.side_dim; } return;
        case NVL_T_SIDE_NORM: if (m->cfg.side_dim) N = W; return;
        case NVL_T_ROUTER: if (c.experts) { N = c.experts; K = W; } return;
        case NVL_T_ROUTER_BIAS: if (c.experts) N = c.experts; return;
        case NVL_T_MOE_IN: if (c.experts) { N = (int64_t)c.experts * 2 * c.expert_dim; K = W; } return;
        case NVL_T_MOE_OUT: if (c.experts) { N = c.experts * W; K = c.expert_dim; } return;
        case NVL_T_BIAS_R1: case NVL_T_BIAS_R2: if (att) N = c.heads; return;
        case NVL_T_V_MIX: if (att && c.v_mix) N = 1; return;
        case NVL_T_MIX_SCALE: case NVL_T_FFN_SCALE: if (post) N = W; return;
        case NVL_T_W1: N = (r.act == NVL_ACT_RELU2 ? 1 : 2) * (int64_t)c.ffn_dim; K = W; return;
        case NVL_T_W2: if (c.ffn_dim) { N = W; K = c.ffn_dim; } return;
        case NVL_T_WO: if (!mam) { N = W; K = hv; } return;
        case NVL_T_BQ: if (att && c.qkv_bias) N = hd; return;
        case NVL_T_BK: if (att && c.qkv_bias) N = (int64_t)c.kv_heads * c.dim; return;
        case NVL_T_BV: if (att && c.qkv_bias) N = (int64_t)c.kv_heads * c.vdim; return;
        case NVL_T_Q_NORM: if (c.qk_norm) N = c.qk_norm == NVL_QK_NORM_HEAD ? c.dim : hd; return;
        case NVL_T_K_NORM: if (c.qk_norm) N = c.qk_norm == NVL_QK_NORM_HEAD ? c.dim : (int64_t)c.kv_heads * c.dim; return;
        case NVL_T_SINK: if (c.sink == NVL_SINK_LEARNED) N = c.heads; return;
        case NVL_T_LIN_Q: case NVL_T_LIN_K: if (c.mixer2) { N = (int64_t)c.heads2 * c.dim2; K = W; } return;
        case NVL_T_LIN_V: case NVL_T_LIN_GATE: if (c.mixer2) { N = (int64_t)c.heads2 * c.vdim2; K = W; } return;
        case NVL_T_LIN_NORM: if (c.mixer2) N = (int64_t)c.heads2 * c.vdim2; return;
        case NVL_T_LIN_O: if (c.mixer2) { N = W; K = (int64_t)c.heads2 * c.vdim2; } return;
        case NVL_T_MIX_GATE: if (lat || gla || (att && !c.ungated)) { N = c.gate_per_head && lat ? c.heads : hv; K = W; } return;
        case NVL_T_LAT_DQ: if (lat) { N = c.q_rank; K = W; } return;
        case NVL_T_LAT_DQ_NORM: if (lat) N = c.q_rank; return;
        case NVL_T_LAT_UQ: if (lat) { N = hd + (int64_t)c.heads * c.rot_dim; K = c.q_rank; } return;
        case NVL_T_LAT_DKV: if (lat && r.src == layer) { N = c.kv_rank + c.rot_dim; K = W; } return;
        case NVL_T_LAT_DKV_NORM: if (lat && r.src == layer) N = c.kv_rank; return;
        case NVL_T_LAT_UK: if (lat) { N = hd; K = c.kv_rank; } return;
        case NVL_T_LAT_UV: if (lat) { N = hv; K = c.kv_rank; } return;
        case NVL_T_WQ: if (att) { N = hd; K = W; return; } [[fallthrough]];
        case NVL_T_WK: if (att) { N = (int64_t)c.kv_heads * c.dim; K = W; } else if (gla || delta) { N = delta ? (int64_t)c.kv_heads * c.dim : hd; K = W; } return;
        case NVL_T_WV: if (att) { N = (int64_t)c.kv_heads * c.vdim; K = W; } else if (gla || delta) { N = hv; K = W; } return;
        case NVL_T_DELTA_CONV: if (delta) N = (int64_t)r.conv_dim * c.conv_taps; return;
        case NVL_T_DELTA_BETA: if (delta) { N = c.heads; K = W; } return;
        case NVL_T_DELTA_G1: if (delta) { N = -1; K = W; } return;
        case NVL_T_DELTA_G2: if (delta) { N = hv; K = -1; } return;
        case NVL_T_GLA_NORM: if (gla || delta) N = c.vdim; return;
        case NVL_T_GLA_A1: if (gla || delta) { N = c.decay_rank ? c.decay_rank : -1; K = W; } return;       // -1: any
        case NVL_T_GLA_A2: if (gla || delta) { N = hd; K = c.decay_rank ? c.decay_rank : -1; } return;
        case NVL_T_GLA_A2_B: if (gla || delta) N = hd; return;
        case NVL_T_MAMBA_IN_PROJ: if (mam) { N = r.n_in; K = W; } return;
        case NVL_T_MAMBA_CONV_W: if (mam) N = (int64_t)r.conv_dim * c.conv_taps; return;
        case NVL_T_MAMBA_CONV_B: if (mam) N = r.conv_dim; return;
        case NVL_T_MAMBA_A_LOG: if (mam || delta) N = c.heads; return;
        case NVL_T_MAMBA_D: case NVL_T_MAMBA_DT_BIAS: if (mam) N = c.heads; return;
        case NVL_T_MAMBA_NORM: if (mam) N = hv; return;
        case NVL_T_MAMBA_OUT_PROJ: if (mam) { N = W; K = hv; } return;
        default: return;
    }
}
bool layered_1d(int kind) {
    if (is_1d(kind)) return true;
    return kind == NVL_T_MIX_POST_NORM || kind == NVL_T_FFN_POST_NORM || kind == NVL_T_LAT_DQ_NORM || kind == NVL_T_LAT_DKV_NORM ||
           kind == NVL_T_BIAS_R1 || kind == NVL_T_BIAS_R2 || kind == NVL_T_V_MIX || kind == NVL_T_ROUTER_BIAS || kind == NVL_T_SIDE_NORM ||
           kind == NVL_T_Q_NORM || kind == NVL_T_K_NORM || kind == NVL_T_SINK || kind == NVL_T_SHIFT || kind == NVL_T_LIN_NORM || kind == NVL_T_GLA_NORM || kind == NVL_T_GLA_A2_B || kind == NVL_T_MIX_SCALE || kind == NVL_T_FFN_SCALE || kind == NVL_T_DELTA_CONV;
}
int layered_upload(nvl_model* m, int kind, int layer, const void* data, int dtype, int64_t rows, int64_t cols, int layout) {
    int64_t N, K;
    layered_shape(m, kind, layer, N, K);
    char buf[256];
    if (N == 0) {
        snprintf(buf, sizeof buf, "nvl_upload_tensor: layer %d has no tensor of kind %d", layer, kind);
        return fail(m, NVL_ERR_INVALID, buf);
    }
    const bool vec = layered_1d(kind);
    if (vec) { rows *= cols > 0 ? cols : 1; cols = 1; }
    else if (layout != NVL_LAYOUT_OUT_IN && kind != NVL_T_TOK_EMB && kind != NVL_T_POS_EMB) return fail(m, NVL_ERR_INVALID, "nvl_upload_tensor: matrices of this model are given [out, in]");
    if (rows <= 0 || cols <= 0 || (N > 0 && rows != N) || (K > 0 && cols != K)) {
        snprintf(buf, sizeof buf, "tensor kind %d of layer %d: got [%lld,%lld], the model needs [%lld,%lld]", kind, layer, (long long)rows, (long long)cols, (long long)N, (long long)K);
        return fail(m, NVL_ERR_INVALID, buf);
    }
    DevTensor* t = tensor_slot(m, kind, layer);
    const size_t bytes = (size_t)(rows * cols) * (dtype == NVL_DTYPE_F32 ? 4 : 2);
    dfree(t->p);
    t->p = dmalloc_bytes((int64_t)bytes);
    NVL_HIP(hipMemcpyAsync(t->p, data, bytes, hipMemcpyDefault, m->stream));
    NVL_HIP(hipStreamSynchronize(m->stream));
    t->rows = rows; t->cols = cols; t->rows_pad = rows; t->raw_dtype = dtype;
    return NVL_OK;
}

void* lay_alloc(nvl_model* m, int64_t bytes) {      // zero-filled
    bytes = round_up(std::max<int64_t>(bytes, 16), 16);
    void* p = dmalloc_bytes(bytes);
    m->layered_allocs.push_back(p);
    NVL_HIP(hipMemsetAsync(p, 0, (size_t)bytes, m->stream));
    return p;
}
void* lay_matrix(nvl_model* m, int64_t N, int64_t Kd) {       // zero matrix of the weight dtype; rows padded to whole GEMM tiles
    const int64_t bytes = round_up(N, W_ROW_PAD) * Kd * (int64_t)m->wsize;
    m->stats.weight_bytes += (double)bytes;
    return lay_alloc(m, bytes);
}
float* lay_vector(nvl_model* m, const DevTensor& t, int64_t padded) {
    float* p = (float*)lay_alloc(m, padded * 4);
    const int64_t n = t.rows * t.cols;
    hipLaunchKernelGGL(convert_1d_kernel, dim3(cdiv(n, 256)), dim3(256), 0, m->stream, t.p, t.raw_dtype, p, n, (int64_t)0);
    NVL_HIP(hipGetLastError());
    m->stats.weight_bytes += (double)padded * 4;
    return p;
}
// (w + offset) * scale (scale: NULL or another staged vector), zero beyond the vector: what a norm multiplies by
__global__ void norm_weight_kernel(float* w, const void* scale, int scale_dtype, float offset, int64_t n) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i < n) w[i] = (w[i] + offset) * (scale ? ld_as_f32(scale, scale_dtype, i) : 1.0f);
}
// w[i] *= f; with `spread`, every w[i] <- w[0] * f
__global__ void scale_weight_kernel(float* w, float f, int64_t n, bool spread) {
    const float first = w[0];
    __syncthreads();
    for (int64_t i = threadIdx.x; i < n; i += blockDim.x) w[i] = (spread ? first : w[i]) * f;
}
void lay_scale(nvl_model* m, float* w, float f, int64_t n, bool spread = false) {
    hipLaunchKernelGGL(scale_weight_kernel, dim3(1), dim3(1024), 0, m->stream, w, f, n, spread);
    NVL_HIP(hipGetLastError());
}
float* lay_norm(nvl_model* m, const DevTensor& t, int64_t padded, const DevTensor* scale = nullptr) {
    float* p = lay_vector(m, t, padded);
    const bool sc = scale && scale->present(), one = m->cfg.norm_type == NVL_NORM_RMS_SCALAR;
    if (one) lay_scale(m, p, 1.0f, m->Hn, true);          // one weight for all coordinates
    if (m->cfg.norm_weight_offset != 0.f || sc) {
        const int64_t n = one ? m->Hn : t.rows * t.cols;
        hipLaunchKernelGGL(norm_weight_kernel, dim3(cdiv(n, 256)), dim3(256), 0, m->stream, p, sc ? (const void*)scale->p : nullptr, sc ? scale->raw_dtype : 0, m->cfg.norm_weight_offset, n);
        NVL_HIP(hipGetLastError());
    }
    return p;
}
// (cos, sin) of every position for a rotation; angles in double
f32x2* lay_rotation(nvl_model* m, const nvl_layer_config& c) {
    const int half = c.rot_dim / 2;
    std::vector<double> f((size_t)half);
    double mag = 1.0;
    for (int i = 0; i < half; i++) f[(size_t)i] = std::pow(c.rot_base, -2.0 * i / c.rot_dim);
    if (c.rot_high > 0.0) {        // Llama 3.1: waves longer than original / low are slowed down, those shorter than original / high are not, in between a blend
        for (double& v : f) {
            const double wave = 2.0 * M_PI / v, s = (c.rot_original / wave - c.rot_low) / (c.rot_high - c.rot_low);
            if (wave > c.rot_original / c.rot_low) v /= c.rot_factor;
            else if (!(wave < c.rot_original / c.rot_high)) v = (1.0 - s) * v / c.rot_factor + s * v;
        }
    } else if (c.rot_factor > 0.0) {      // YaRN: pairs that turn often over the original length keep their frequency, the others are slowed down
        auto place = [&](double turns) { return c.rot_dim * std::log(c.rot_original / (2.0 * M_PI * turns)) / (2.0 * std::log(c.rot_base)); };
        const double lo = std::max(std::floor(place(c.rot_fast)), 0.0), hi = std::min(std::ceil(place(c.rot_slow)), c.rot_dim - 1.0);
        for (int i = 0; i < half; i++) {
            const double ramp = std::min(std::max((i - lo) / std::max(hi - lo, 0.001), 0.0), 1.0);
            f[(size_t)i] = f[(size_t)i] / c.rot_factor * ramp + f[(size_t)i] * (1.0 - ramp);
        }
        mag = 0.1 * std::log(c.rot_factor) + 1.0;
    }
    std::vector<float> t((size_t)m->cfg.max_seq_len * half * 2);
    for (int p = 0; p < m->cfg.max_seq_len; p++)
        for (int i = 0; i < half; i++) {
            const double a = p * f[(size_t)i];
            t[((size_t)p * half + i) * 2] = (float)(std::cos(a) * mag);
            t[((size_t)p * half + i) * 2 + 1] = (float)(std::sin(a) * mag);
        }
    f32x2* d = (f32x2*)lay_alloc(m, (int64_t)t.size() * 4);
    NVL_HIP(hipMemcpyAsync(d, t.data(), t.size() * 4, hipMemcpyHostToDevice, m->stream));
    NVL_HIP(hipStreamSynchronize(m->stream));
    return d;
}
// rows [n0, n0 + N) of a staged matrix into dst: grouped row / column padding as place_2d_kernel
void lay_place(nvl_model* m, const DevTensor& t, void* dst, int64_t Kd, int64_t row0 = 0, int rg = 0, int rgp = 0, int cg = 0, int cgp = 0,
               int64_t n0 = 0, int64_t N = -1, bool trans = false, bool row_major = false, int64_t col0 = 0) {
    if (N < 0) N = t.rows;
    Place2D pl{N, t.cols, Kd, row0, rg ? rg : 1, rg ? rgp : 1, cg ? cg : 1, cg ? cgp : 1, col0};
    const dim3 grid((unsigned)std::min<int64_t>(cdiv(t.cols, 256), 64), (unsigned)std::min<int64_t>(N, 32768), (unsigned)cdiv(N, 32768));
    const int64_t src0 = n0 * t.cols;
    if (m->f32) {
        if (trans) hipLaunchKernelGGL((place_2d_kernel<float, false, true>), grid, dim3(256), 0, m->stream, t.p, t.raw_dtype, src0, (float*)dst, pl);
        else hipLaunchKernelGGL((place_2d_kernel<float, false, false>), grid, dim3(256), 0, m->stream, t.p, t.raw_dtype, src0, (float*)dst, pl);
    } else {
        if (row_major) hipLaunchKernelGGL((place_2d_kernel<bf16_t, false, false>), grid, dim3(256), 0, m->stream, t.p, t.raw_dtype, src0, (bf16_t*)dst, pl);
        else if (trans) hipLaunchKernelGGL((place_2d_kernel<bf16_t, true, true>), grid, dim3(256), 0, m->stream, t.p, t.raw_dtype, src0, (bf16_t*)dst, pl);
        else hipLaunchKernelGGL((place_2d_kernel<bf16_t, true, false>), grid, dim3(256), 0, m->stream, t.p, t.raw_dtype, src0, (bf16_t*)dst, pl);
    }
    NVL_HIP(hipGetLastError());
}

// absorbed latent attention: available to a layer?
bool lat_absorb_ok(const nvl_model* m, const LayerRun& r) { return !m->f32 && r.rp <= LAT_ABSORB_MAX_RP && (r.rotp <= 64 || r.rotp == 128); }

void layered_finalize(nvl_model* m) {
    auto need = [&](const DevTensor& t, const std::string& what) -> const DevTensor& {
        if (!t.present()) throw std::runtime_error("nvl_finalize: missing tensor: " + what);
        return t;
    };
    const int64_t H = m->H;
    need(m->g[NVL_T_TOK_EMB], "token embedding"); need(m->g[NVL_T_FINAL_NORM_W], "final norm");
    const bool sum = m->cfg.block_style == NVL_BLOCK_SUM_NORM, post = sum || m->cfg.block_style == NVL_BLOCK_POST;      // post: sublayers read the stream itself
    const bool par = m->cfg.block_style == NVL_BLOCK_PARALLEL, ln = m->cfg.norm_type == NVL_NORM_LAYER, learned = m->cfg.position_type == NVL_POS_LEARNED;
    m->final_norm = lay_norm(m, m->g[NVL_T_FINAL_NORM_W], H);
    if (ln) m->final_norm_b = lay_vector(m, need(m->g[NVL_T_FINAL_NORM_B], "final norm bias"), H);
    auto big = [&](int kind, const char* what) {      // [V][H]: the embedding table / LM head
        void* p = lay_matrix(m, m->V, H);
        lay_place(m, need(m->g[kind], what), p, H);
        return p;
    };
    void* emb = big(NVL_T_TOK_EMB, "token embedding");
    m->lm_head = m->g[NVL_T_LM_HEAD].present() && !m->cfg.tied_embedding ? big(NVL_T_LM_HEAD, "LM head") : emb;
    void* pos = nullptr;
    if (learned) {
        const DevTensor& t = need(m->g[NVL_T_POS_EMB], "position embedding");
        if (t.rows < m->cfg.max_seq_len) throw std::runtime_error("nvl_finalize: max_seq_len exceeds the learned positions");
        pos = lay_matrix(m, t.rows, H);
        lay_place(m, t, pos, H);
    }
    const int sd = m->cfg.side_dim, sd4 = (int)round_up(sd, 4);
    if (sd) {       // [V][layer][sd4], row-major
        const DevTensor& t = need(m->g[NVL_T_SIDE_EMB], "per-layer token embedding");
        m->side_ld = (int64_t)m->L * sd4; m->side_kp = (int)round_up(sd, 64);
        m->side_emb = lay_alloc(m, (int64_t)m->V * m->side_ld * (int64_t)m->wsize);
        lay_place(m, t, m->side_emb, m->side_ld, 0, 0, 0, sd, sd4, 0, -1, false, true);
    }
    NVL_HIP(hipStreamSynchronize(m->stream));
    for (int k = 0; k < NVL_T_COUNT; k++) if (is_global(k)) { dfree(m->g[k].p); m->g[k].p = nullptr; }
    m->g[NVL_T_TOK_EMB].p = emb; m->g[NVL_T_TOK_EMB].raw_dtype = -1;      // (the embedding kernels' view of it)
    m->g[NVL_T_POS_EMB].p = pos;

    int64_t ld_in = 0, q_cols = 0, cq_cols = 0, ko = 0, conv = 0, ocols = 0, Fmax = 0, abs_cols = 0, z_cols = 0, g_cols = 0, pa_cols = 0, pg_cols = 0;
    int64_t moe_k = 0, moe_e = 0, moe_kI = 0, moe_ep = 0, moe_all = 0, moe_sl = 0, grp_vp = 0, qg_cols = 0;
    for (int i = 0; i < m->L; i++) {
        LayerRun& r = m->runs[(size_t)i];
        const nvl_layer_config& c = r.c;
        MixerW& w = m->mixers[(size_t)i];
        LayerW& l = m->layers[(size_t)i];
        const std::string at = "layer " + std::to_string(i) + " ";
        if (r.owner == i) {
            auto T = [&](int kind, const char* what) -> const DevTensor& { return need(l.t[kind], at + what); };
            if (!post) w.norm1 = lay_norm(m, T(NVL_T_ATTN_NORM_W, "norm before the mixer"), H);
            if (ln) w.norm1_bias = lay_vector(m, T(NVL_T_ATTN_NORM_B, "bias of the norm before the mixer"), H);
            if (!par) w.norm1b = lay_norm(m, T(NVL_T_MIX_POST_NORM, "norm after the mixer"), H, &l.t[NVL_T_MIX_SCALE]);
            if (m->cfg.token_shift) w.shift = lay_vector(m, T(NVL_T_SHIFT, "token shift"), H);
            if (sum && (c.ffn_dim || c.experts)) w.norm2b = lay_norm(m, T(NVL_T_FFN_POST_NORM, "norm after the feed-forward"), H);
            if (c.ffn_dim) {
                if (!post && !par) w.norm2 = lay_norm(m, T(NVL_T_FFN_NORM_W, "norm before the feed-forward"), H);
                if (!par && !sum) w.norm2b = lay_norm(m, T(NVL_T_FFN_POST_NORM, "norm after the feed-forward"), H, &l.t[NVL_T_FFN_SCALE]);
                const DevTensor& w1 = T(NVL_T_W1, "feed-forward gate / up");
                const bool in_experts = r.shared_parts && !m->f32;        // (rows of the experts' matrix)
                if (!r.ffn_in && !r.glu_in && !in_experts) w.w1 = lay_matrix(m, (r.act == NVL_ACT_RELU2 ? 1 : 2) * r.Fp, H);
                if (r.ffn_in || r.glu_in || in_experts) {}      // (or rows of the fused input projection)
                else if (r.act == NVL_ACT_RELU2) lay_place(m, w1, w.w1, H);
                else if (m->f32) { lay_place(m, w1, w.w1, H, 0, 0, 0, 0, 0, 0, c.ffn_dim); lay_place(m, w1, w.w1, H, r.Fp, 0, 0, 0, 0, c.ffn_dim, c.ffn_dim); }
                else { lay_place(m, w1, w.w1, H, 0, 16, 32, 0, 0, 0, c.ffn_dim); lay_place(m, w1, w.w1, H, 16, 16, 32, 0, 0, c.ffn_dim, c.ffn_dim); }
                if (!par) {
                    w.w2 = lay_matrix(m, H, r.Fp);
                    lay_place(m, T(NVL_T_W2, "feed-forward down"), w.w2, r.Fp);
                }
            }
            if (c.experts) {
                const int64_t E = c.experts, I = c.expert_dim, Ip = r.Ip, Es = E + (m->f32 ? 0 : r.shared_parts);
                const DevTensor &up = T(NVL_T_MOE_IN, "experts' gate / up"), &down = T(NVL_T_MOE_OUT, "experts' down");
                // (a grouped launch reads whole column tiles of its expert's rows: the last expert's need rows behind them)
                w.moe_up = lay_matrix(m, (Es - 1) * 2 * Ip + round_up(2 * Ip, W_ROW_PAD), H);
                w.moe_down = lay_matrix(m, (E - 1) * H + round_up(H, W_ROW_PAD), Ip);
                if (!m->f32) w.moe_cat = lay_matrix(m, H, r.Ep * Ip);
                for (int64_t e = 0; e < E; e++) {
                    const int64_t row = e * 2 * Ip, from = e * 2 * I;
                    if (m->f32) { lay_place(m, up, w.moe_up, H, row, 0, 0, 0, 0, from, I); lay_place(m, up, w.moe_up, H, row + Ip, 0, 0, 0, 0, from + I, I); }
                    else { lay_place(m, up, w.moe_up, H, row, 16, 32, 0, 0, from, I); lay_place(m, up, w.moe_up, H, row + 16, 16, 32, 0, 0, from + I, I); }
                    lay_place(m, down, w.moe_down, Ip, e * H, 0, 0, 0, 0, e * m->Hn, m->Hn);
                    if (!m->f32) lay_place(m, down, w.moe_cat, r.Ep * Ip, 0, 0, 0, 0, 0, e * m->Hn, m->Hn, false, false, e * Ip);
                }
                if (Es > E) {        // the shared expert behind them: the same 16 + 16 rows, its columns of the down projection
                    const DevTensor& w1 = T(NVL_T_W1, "shared expert's gate / up");
                    lay_place(m, w1, w.moe_up, H, E * 2 * Ip, 16, 32, 0, 0, 0, c.ffn_dim);
                    lay_place(m, w1, w.moe_up, H, E * 2 * Ip + 16, 16, 32, 0, 0, c.ffn_dim, c.ffn_dim);
                    lay_place(m, T(NVL_T_W2, "shared expert's down"), w.moe_cat, r.Ep * Ip, 0, 0, 0, 0, 0, 0, -1, false, false, E * Ip);
                }
                if (!par) { w.router = lay_matrix(m, E, H); lay_place(m, T(NVL_T_ROUTER, "router"), w.router, H); }
                if (l.t[NVL_T_ROUTER_BIAS].present()) w.route_bias = lay_vector(m, l.t[NVL_T_ROUTER_BIAS], E);
            }
            if (sd) {
                w.side_gate = lay_matrix(m, sd, H); lay_place(m, T(NVL_T_SIDE_GATE, "token input gate"), w.side_gate, H);
                w.side_proj = lay_matrix(m, H, m->side_kp); lay_place(m, T(NVL_T_SIDE_PROJ, "token input projection"), w.side_proj, m->side_kp);
                w.side_norm = lay_vector(m, T(NVL_T_SIDE_NORM, "token input norm"), H);
            }
            if (c.mixer == NVL_MIXER_LATENT_ATTENTION) {
                w.in = lay_matrix(m, r.n_in, H);
                lay_place(m, T(NVL_T_LAT_DQ, "query down projection"), w.in, H);
                if (r.src == i) {
                    const DevTensor& dkv = T(NVL_T_LAT_DKV, "key/value down projection");
                    lay_place(m, dkv, w.in, H, r.qrp, 0, 0, 0, 0, 0, c.kv_rank);
                    if (c.rot_dim) lay_place(m, dkv, w.in, H, r.qrp + r.rp, 0, 0, 0, 0, c.kv_rank, c.rot_dim);
                    w.dkv_norm = lay_vector(m, T(NVL_T_LAT_DKV_NORM, "key/value latent norm"), r.rp);
                }
                const DevTensor& gate = T(NVL_T_MIX_GATE, "output gate");
                if (c.gate_per_head) lay_place(m, gate, w.in, H, r.gate_off);
                else lay_place(m, gate, w.in, H, r.gate_off, c.vdim, r.vp);
                w.dq_norm = lay_vector(m, T(NVL_T_LAT_DQ_NORM, "query latent norm"), r.qrp);
                w.uq = lay_matrix(m, (int64_t)c.heads * r.dp, r.qrp);
                const DevTensor& uq = T(NVL_T_LAT_UQ, "query up projection");
                if (!c.rot_dim) lay_place(m, uq, w.uq, r.qrp, 0, c.dim, r.dp);
                else for (int64_t h = 0; h < c.heads; h++) {
                    const int64_t from = h * (c.dim + c.rot_dim);
                    lay_place(m, uq, w.uq, r.qrp, h * r.dp, 0, 0, 0, 0, from, c.dim);
                    lay_place(m, uq, w.uq, r.qrp, h * r.dp + r.dn, 0, 0, 0, 0, from + c.dim, c.rot_dim);
                }
                const DevTensor& uk = T(NVL_T_LAT_UK, "key up projection");
                w.uk = lay_matrix(m, (int64_t)c.heads * r.dn, r.rp);
                lay_place(m, uk, w.uk, r.rp, 0, c.dim, r.dn);
                if (lat_absorb_ok(m, r)) {
                    w.ukt = lay_matrix(m, (int64_t)c.heads * r.rp, r.dn);
                    for (int h = 0; h < c.heads; h++)
                        lay_place(m, uk, (char*)w.ukt + (int64_t)h * r.rp * r.dn * (int64_t)m->wsize, r.dn, 0, 0, 0, 0, 0, (int64_t)h * c.dim, c.dim, true);
                }
                w.uv = lay_matrix(m, (int64_t)c.heads * r.vp, r.rp);
                lay_place(m, T(NVL_T_LAT_UV, "value up projection"), w.uv, r.rp, 0, c.vdim, r.vp);
                w.o = lay_matrix(m, H, r.kd);
                lay_place(m, T(NVL_T_WO, "output projection"), w.o, r.kd, 0, 0, 0, c.vdim, r.vp);
            } else if (c.mixer == NVL_MIXER_ATTENTION) {
                w.in = lay_matrix(m, r.n_in, H);
                lay_place(m, T(NVL_T_WQ, "query projection"), w.in, H, 0, c.dim, r.dp);
                lay_place(m, T(NVL_T_WK, "key projection"), w.in, H, r.k_off, c.dim, r.dp);
                lay_place(m, T(NVL_T_WV, "value projection"), w.in, H, r.v_off, c.vdim, r.vp);
                if (!c.ungated) lay_place(m, T(NVL_T_MIX_GATE, "output gate"), w.in, H, r.gate_off, c.vdim, r.vp);
                if (c.qkv_bias) {
                    w.in_bias = (float*)lay_alloc(m, round_up(r.n_in, W_ROW_PAD) * 4);
                    auto bias = [&](int kind, const char* what, int off, int d, int dp) {
                        const DevTensor& t = T(kind, what);
                        const Place2D pl{1, t.rows, round_up(r.n_in, W_ROW_PAD), 0, 1, 1, d, dp, off};
                        hipLaunchKernelGGL((place_2d_kernel<float, false, false>), dim3((unsigned)std::min<int64_t>(cdiv(t.rows, 256), 64), 1, 1), dim3(256), 0, m->stream, t.p, t.raw_dtype, 0, w.in_bias, pl);
                        NVL_HIP(hipGetLastError());
                    };
                    bias(NVL_T_BQ, "query bias", 0, c.dim, r.dp); bias(NVL_T_BK, "key bias", r.k_off, c.dim, r.dp); bias(NVL_T_BV, "value bias", r.v_off, c.vdim, r.vp);
                }
                if (c.qk_norm) { w.q_norm = lay_vector(m, T(NVL_T_Q_NORM, "query norm"), l.t[NVL_T_Q_NORM].rows); w.k_norm = lay_vector(m, T(NVL_T_K_NORM, "key norm"), l.t[NVL_T_K_NORM].rows); }
                if (c.sink == NVL_SINK_LEARNED) w.sink = lay_vector(m, T(NVL_T_SINK, "sinks"), c.heads);
                else if (c.sink) w.sink = (float*)lay_alloc(m, (int64_t)c.heads * 4);
                if (l.t[NVL_T_BIAS_R1].present()) {
                    w.r1 = lay_vector(m, l.t[NVL_T_BIAS_R1], c.heads);
                    w.r2 = lay_vector(m, T(NVL_T_BIAS_R2, "distance bias (r2)"), c.heads);
                    std::vector<float> v((size_t)c.heads * 2);
                    NVL_HIP(hipMemcpyAsync(v.data(), w.r1, (size_t)c.heads * 4, hipMemcpyDeviceToHost, m->stream));
                    NVL_HIP(hipMemcpyAsync(v.data() + c.heads, w.r2, (size_t)c.heads * 4, hipMemcpyDeviceToHost, m->stream));
                    NVL_HIP(hipStreamSynchronize(m->stream));
                    w.bias_lowers = std::all_of(v.begin(), v.end(), [](float x) { return x >= 0.f; });
                }
                if (c.v_mix) w.v_lambda = lay_vector(m, T(NVL_T_V_MIX, "value mixing"), 1);
                w.o = lay_matrix(m, H, r.kd);
                lay_place(m, T(NVL_T_WO, "output projection"), w.o, r.kd, 0, 0, 0, c.vdim, r.vp);
                if (c.mixer2) {
                    lay_place(m, T(NVL_T_LIN_Q, "lightning query projection"), w.in, H, r.lq_off); lay_place(m, T(NVL_T_LIN_K, "lightning key projection"), w.in, H, r.lk_off);
                    lay_place(m, T(NVL_T_LIN_V, "lightning value projection"), w.in, H, r.lv_off); lay_place(m, T(NVL_T_LIN_GATE, "lightning gate"), w.in, H, r.lg_off);
                    const int64_t hv = (int64_t)c.heads2 * c.vdim2;
                    w.lin_norm = lay_vector(m, T(NVL_T_LIN_NORM, "lightning norm"), hv);
                    lay_scale(m, w.lin_norm, c.out_scale2, hv);
                    lay_place(m, T(NVL_T_LIN_O, "lightning output projection"), w.o, r.kd, 0, 0, 0, 0, 0, 0, -1, false, false, r.ko);
                    std::vector<float> d((size_t)c.heads2 * 2);       // decays, then their logarithms (finite, and 2^-300 is zero)
                    for (int h = 0; h < c.heads2; h++) { d[(size_t)h] = (float)c.decay[h]; d[(size_t)(c.heads2 + h)] = (float)std::max(std::log2(c.decay[h]), -300.0); }
                    w.decay = (float*)lay_alloc(m, (int64_t)d.size() * 4); w.log2_decay = w.decay + c.heads2;
                    NVL_HIP(hipMemcpyAsync(w.decay, d.data(), d.size() * 4, hipMemcpyHostToDevice, m->stream));
                    NVL_HIP(hipStreamSynchronize(m->stream));
                }
            } else if (c.mixer == NVL_MIXER_MAMBA2) {
                w.in = lay_matrix(m, r.n_in, H);
                lay_place(m, T(NVL_T_MAMBA_IN_PROJ, "input projection"), w.in, H);
                w.conv_w = lay_vector(m, T(NVL_T_MAMBA_CONV_W, "convolution"), (int64_t)r.conv_dim * c.conv_taps);
                w.conv_b = lay_vector(m, T(NVL_T_MAMBA_CONV_B, "convolution bias"), r.conv_dim);
                w.a_log = lay_vector(m, T(NVL_T_MAMBA_A_LOG, "A_log"), c.heads);
                w.dskip = lay_vector(m, T(NVL_T_MAMBA_D, "D"), c.heads);
                w.dt_bias = lay_vector(m, T(NVL_T_MAMBA_DT_BIAS, "dt_bias"), c.heads);
                w.mix_norm = lay_vector(m, T(NVL_T_MAMBA_NORM, "inner norm"), (int64_t)c.heads * c.vdim);
                w.o = lay_matrix(m, H, r.kd);
                lay_place(m, T(NVL_T_MAMBA_OUT_PROJ, "output projection"), w.o, r.kd);
            } else if (c.mixer == NVL_MIXER_CHANNEL_DELTA) {
                const DevTensor &a1 = T(NVL_T_GLA_A1, "decay projection (a1)"), &a2 = T(NVL_T_GLA_A2, "decay projection (a2)");
                const DevTensor &g1 = T(NVL_T_DELTA_G1, "output gate (g1)"), &g2 = T(NVL_T_DELTA_G2, "output gate (g2)");
                if (a1.rows != a2.cols || g1.rows != g2.cols || a1.rows > 2048 || g1.rows > 2048)
                    throw std::runtime_error("nvl_finalize: " + at + "the low-rank projections do not fit (or a rank exceeds 2048)");
                w.rank = (int)a1.rows; w.grank = (int)g1.rows;
                w.a_rkp = (int)round_up(w.rank, 64); w.g_rkp = (int)round_up(w.grank, 64);
                const int64_t qk = (int64_t)c.kv_heads * c.dim, hd = (int64_t)c.heads * c.dim, hv = (int64_t)c.heads * c.vdim;
                r.a1_off = (int)round_up(r.conv_dim, 4); r.g1_off = r.a1_off + (int)round_up(w.rank, 4); r.b_off = r.g1_off + (int)round_up(w.grank, 4);
                r.n_in = r.b_off + c.heads;
                w.in = lay_matrix(m, r.n_in, H);
                lay_place(m, T(NVL_T_WQ, "query projection"), w.in, H);
                lay_place(m, T(NVL_T_WK, "key projection"), w.in, H, qk);
                lay_place(m, T(NVL_T_WV, "value projection"), w.in, H, 2 * qk);
                lay_place(m, a1, w.in, H, r.a1_off);
                lay_place(m, g1, w.in, H, r.g1_off);
                lay_place(m, T(NVL_T_DELTA_BETA, "step size projection"), w.in, H, r.b_off);
                w.conv_w = lay_vector(m, T(NVL_T_DELTA_CONV, "convolution"), (int64_t)r.conv_dim * c.conv_taps);
                w.conv_b = (float*)lay_alloc(m, (int64_t)r.conv_dim * 4);
                w.a_log = lay_vector(m, T(NVL_T_MAMBA_A_LOG, "A_log"), c.heads);
                w.dt_bias = lay_vector(m, T(NVL_T_GLA_A2_B, "decay bias"), hd);
                w.mix_norm = lay_vector(m, T(NVL_T_GLA_NORM, "head norm"), c.vdim);
                w.a2m = lay_matrix(m, hd, w.a_rkp); lay_place(m, a2, w.a2m, w.a_rkp);
                w.g2m = lay_matrix(m, hv, w.g_rkp); lay_place(m, g2, w.g2m, w.g_rkp);
                w.a2r = w.a2m; w.g2r = w.g2m;
                if (!m->f32) {
                    w.a2r = lay_matrix(m, hd, w.a_rkp); lay_place(m, a2, w.a2r, w.a_rkp, 0, 0, 0, 0, 0, 0, -1, false, true);
                    w.g2r = lay_matrix(m, hv, w.g_rkp); lay_place(m, g2, w.g2r, w.g_rkp, 0, 0, 0, 0, 0, 0, -1, false, true);
                }
                w.o = lay_matrix(m, H, r.kd);
                lay_place(m, T(NVL_T_WO, "output projection"), w.o, r.kd);
            } else {
                const DevTensor& a1 = T(NVL_T_GLA_A1, "decay projection (a1)");
                const DevTensor& a2 = T(NVL_T_GLA_A2, "decay projection (a2)");
                if (a1.rows != a2.cols || a1.rows > 512) throw std::runtime_error("nvl_finalize: " + at + "the two decay projections do not fit (or their rank exceeds 512)");
                w.rank = (int)a1.rows;
                const int64_t hd = (int64_t)c.heads * c.dim, hv = (int64_t)c.heads * c.vdim;
                w.in = lay_matrix(m, 2 * hd + 2 * hv + w.rank, H);
                lay_place(m, T(NVL_T_WQ, "query projection"), w.in, H);
                lay_place(m, T(NVL_T_WK, "key projection"), w.in, H, hd);
                lay_place(m, T(NVL_T_WV, "value projection"), w.in, H, 2 * hd);
                lay_place(m, T(NVL_T_MIX_GATE, "output gate"), w.in, H, 2 * hd + hv);
                lay_place(m, a1, w.in, H, 2 * hd + 2 * hv);
                w.a2 = lay_vector(m, a2, a2.rows * a2.cols);
                w.a2_b = lay_vector(m, T(NVL_T_GLA_A2_B, "decay bias"), hd);
                w.mix_norm = lay_vector(m, T(NVL_T_GLA_NORM, "head norm"), c.vdim);
                w.o = lay_matrix(m, H, r.kd);
                lay_place(m, T(NVL_T_WO, "output projection"), w.o, r.kd);
            }
            if (r.ffn_in) lay_place(m, T(NVL_T_W1, "feed-forward up"), w.in, H, r.ffn_off);
            if (r.glu_in) lay_place(m, T(NVL_T_W1, "feed-forward gate / up"), w.in, H, r.ffn_off, c.ffn_dim, r.Fp);
            if (c.experts && par) lay_place(m, T(NVL_T_ROUTER, "router"), w.in, H, r.route_off);
            if (par && c.ffn_dim) lay_place(m, T(NVL_T_W2, "feed-forward down"), w.o, r.kd, 0, 0, 0, 0, 0, 0, -1, false, false, r.ko);
            NVL_HIP(hipStreamSynchronize(m->stream));
            for (auto& t : l.t) { dfree(t.p); t.p = nullptr; }
        }
    }
    for (int i = 0; i < m->L; i++) {
        LayerRun& r = m->runs[(size_t)i];
        const nvl_layer_config& c = r.c;
        if (c.rot_dim) {
            for (int j = 0; j < i && !r.turn; j++)
                if (m->runs[(size_t)j].turn && same_rotation(m->runs[(size_t)j].c, c)) r.turn = m->runs[(size_t)j].turn;
            if (!r.turn) r.turn = lay_rotation(m, c);
        }
        if (c.mixer == NVL_MIXER_CHANNEL_DELTA) {      // (also the layers that use another layer's tensors)
            const LayerRun& o = m->runs[(size_t)r.owner];
            const MixerW& w = m->mixers[(size_t)r.owner];
            r.a1_off = o.a1_off; r.g1_off = o.g1_off; r.b_off = o.b_off; r.n_in = o.n_in;
            z_cols = std::max(z_cols, (int64_t)c.heads * c.dim); g_cols = std::max(g_cols, (int64_t)c.heads * c.vdim);
            pa_cols = std::max<int64_t>(pa_cols, w.a_rkp); pg_cols = std::max<int64_t>(pg_cols, w.g_rkp);
        }
        if (c.mixer == NVL_MIXER_GLA) r.n_in = 2 * c.heads * (c.dim + c.vdim) + m->mixers[(size_t)r.owner].rank;
        const bool qg = c.mixer == NVL_MIXER_ATTENTION && !m->f32 && !r.raw;           // (its projection goes to lqg, the cache and lmix; the router's columns stay)
        ld_in = std::max(ld_in, round_up(qg ? r.n_in - (r.ffn_in ? r.route_off : r.ffn_off) : r.n_in, 4));
        if (c.experts && !par) ld_in = std::max(ld_in, round_up(c.experts, 4));         // (the router's scores, once the mixer is done)
        if (qg || r.raw) qg_cols = std::max<int64_t>(qg_cols, (int64_t)c.heads * (r.dp + (c.ungated ? 0 : r.vp)));
        ko = std::max<int64_t>(ko, r.kd);
        Fmax = std::max<int64_t>(Fmax, r.Fp);
        if (c.experts) {
            const int64_t k = c.top_k;
            moe_k = std::max(moe_k, k); moe_e = std::max<int64_t>(moe_e, c.experts); moe_kI = std::max(moe_kI, k * r.Ip);
            moe_ep = std::max<int64_t>(moe_ep, r.Ep); moe_all = std::max(moe_all, (int64_t)r.Ep * r.Ip); moe_sl = std::max<int64_t>(moe_sl, r.moe_slices);
        }
        if (c.mixer == NVL_MIXER_LATENT_ATTENTION) {
            q_cols = std::max<int64_t>(q_cols, (int64_t)c.heads * r.dp);
            cq_cols = std::max<int64_t>(cq_cols, r.qrp);
            if (lat_absorb_ok(m, r)) abs_cols = std::max(abs_cols, round_up(c.heads, 16) * (r.rp + r.rotp));
        } else if (c.mixer == NVL_MIXER_ATTENTION) {
            grp_vp = std::max<int64_t>(grp_vp, r.vp);
            if (c.mixer2) ocols = std::max<int64_t>(ocols, (int64_t)c.heads2 * c.vdim2);
        } else {
            ocols = std::max<int64_t>(ocols, (int64_t)c.heads * c.vdim);
            conv = std::max<int64_t>(conv, r.conv_dim);
        }
    }
    m->F = (int)std::max<int64_t>(Fmax, 64);
    const int64_t Mmax = m->opts.max_batch_tokens, S = m->opts.max_seqs, Mp = round_up(Mmax, 64), ws = (int64_t)m->wsize;
    auto f32buf = [&](int64_t n) { return (float*)lay_alloc(m, n * 4); };
    m->lproj_ld = ld_in; m->lq_ld = q_cols; m->lo_ld = round_up(ocols, 4); m->lconv_ld = round_up(conv, 4);
    m->x = dmalloc<float>(Mmax * H);
    m->xn = dmalloc_bytes(Mp * H * ws);
    ld_in = std::max<int64_t>(ld_in, 4);
    const int64_t hbuf = std::max(Mp * m->F, (Mmax + 64) * moe_kI);      // (pairs, rounded up to whole tiles, x the experts' width)
    m->hbuf = dmalloc_bytes(hbuf * ws);
    m->xn_last = dmalloc_bytes(round_up(S, 64) * H * ws);
    NVL_HIP(hipMemsetAsync(m->xn, 0, (size_t)(Mp * H * ws), m->stream));
    NVL_HIP(hipMemsetAsync(m->hbuf, 0, (size_t)(hbuf * ws), m->stream));
    NVL_HIP(hipMemsetAsync(m->xn_last, 0, (size_t)(round_up(S, 64) * H * ws), m->stream));
    if (m->f32) m->h2 = dmalloc<float>(Mmax * std::max<int64_t>(2 * std::max<int64_t>(m->F, moe_kI), sd4));
    if (moe_k) {
        m->expert_ids = dmalloc<int32_t>(Mmax * moe_k); m->expert_w = dmalloc<float>(Mmax * moe_k);
        m->seg_start = dmalloc<int32_t>(moe_e + 1); m->moe_counts = dmalloc<int32_t>(moe_e); m->moe_cursor = dmalloc<int32_t>(moe_e);
        m->moe_tile_map = dmalloc<int32_t>(4 * (cdiv(Mmax * moe_k, 128) + moe_e)); m->moe_n_mtiles = dmalloc<int32_t>(4);
        m->perm_token = dmalloc<int32_t>(Mmax * moe_k); m->slot_of = dmalloc<int32_t>(Mmax * moe_k);
        m->moe_eo = dmalloc<float>(Mmax * moe_k * H);
        if (!m->f32) {
            m->moe_xg = dmalloc_bytes(round_up(Mmax * moe_k, 64) * H * 2);
            m->moe_gate = dmalloc<float>(64 * moe_ep);
            m->moe_hall = dmalloc_bytes(64 * moe_all * 2);
            NVL_HIP(hipMemsetAsync(m->moe_hall, 0, (size_t)(64 * moe_all * 2), m->stream));
            m->moe_part = dmalloc<float>(moe_sl * 64 * H);
        }
    }
    if (sd) m->lside = lay_alloc(m, Mp * m->side_kp * ws);
    if (qg_cols) m->lqg = lay_alloc(m, Mp * qg_cols * ws);
    if (m->lvf_ld) m->lvf = (float*)lay_alloc(m, Mmax * m->lvf_ld * 4);
    if (grp_vp && !m->f32 && grp_vp <= 256) {
        m->grp_cap = GROUPED_SPLIT_WGS;
        m->grp_part = (float*)lay_alloc(m, m->grp_cap * (grp_vp * 16 + 32) * 4);
        m->grp_cnt = (int32_t*)lay_alloc(m, m->grp_cap * 4);
    }
    m->lproj = f32buf(Mmax * ld_in);
    m->ly = f32buf(Mmax * H);
    if (q_cols) { m->lq = f32buf(Mmax * q_cols); m->lcq = lay_alloc(m, Mp * cq_cols * ws); }
    m->lmix = lay_alloc(m, Mp * ko * ws);
    if (ocols) m->lo = f32buf(Mmax * m->lo_ld);
    if (z_cols) {
        m->lz_ld = round_up(z_cols, 4); m->lg_ld = round_up(g_cols, 4);
        m->lz = f32buf(Mmax * m->lz_ld); m->lg = f32buf(Mmax * m->lg_ld);
        m->lpa = lay_alloc(m, Mp * pa_cols * ws); m->lpg = lay_alloc(m, Mp * pg_cols * ws);
    }
    if (conv) m->lconv = f32buf(Mmax * m->lconv_ld);
    if (m->lat_block_stride) m->lat_cache = lay_alloc(m, m->lat_block_stride * m->num_blocks * ws);
    if (m->rec_slot_stride) m->rec_state = f32buf(m->rec_slot_stride * S);
    if (m->cfg.token_shift) {
        m->lshift = f32buf((int64_t)m->L * S * H);
        std::vector<int64_t> off;
        for (const LayerRun& r : m->runs) off.push_back(r.shift_off);
        m->shift_offs = (int64_t*)lay_alloc(m, (int64_t)off.size() * 8);
        NVL_HIP(hipMemcpyAsync(m->shift_offs, off.data(), off.size() * 8, hipMemcpyHostToDevice, m->stream));
        NVL_HIP(hipStreamSynchronize(m->stream));
    }
    if (abs_cols) {     // tokens on the absorbed form, and their partial results: splits x tokens <= max(tokens, LAT_PART)
        m->lat_abs_cap = (int)std::max<int64_t>(std::min(Mmax, S * LAT_ABSORB_MAX), 512);
        m->lat_qa = (bf16_t*)lay_alloc(m, (int64_t)m->lat_abs_cap * abs_cols * 2);
        m->lat_part_o = f32buf((int64_t)m->lat_abs_cap * abs_cols);
        m->lat_part_ml = f32buf((int64_t)m->lat_abs_cap * abs_cols);
    }
    m->logit_rows = S;
    m->logits = dmalloc<float>(S * (int64_t)m->Vpad);
    m->argmax_dev = dmalloc<int32_t>(std::max<int64_t>(S, Mmax));
    m->argmax_pval = dmalloc<float>(std::max<int64_t>(S, Mmax) * cdiv(m->V, ARGMAX_CHUNK));
    m->argmax_pidx = dmalloc<int32_t>(std::max<int64_t>(S, Mmax) * cdiv(m->V, ARGMAX_CHUNK));
    m->sk_rows = (int)std::min<int64_t>(std::max<int64_t>(Mmax, 64), SK_TILE_MAX_M);
    if (!m->f32) m->sk_part = dmalloc<float>((int64_t)std::max(m->sk_max_slices, SK_TILE_MAX_SLICES) * m->sk_rows * H);
    m->key_rows.assign(m->masks.size(), 0); m->key_max.assign(m->masks.size(), 0);
    init_slots(m);
    init_meta(m);
    NVL_HIP(hipStreamSynchronize(m->stream));
}

void layered_free(nvl_model* m) {
    if (!m->layered) return;
    for (void* p : m->layered_allocs) dfree(p);
    dfree(m->key_c); dfree(m->key_r); dfree(m->key_k); dfree(m->key_v); dfree(m->rec_z); dfree(m->rec_decay); dfree(m->delta_ws);
    if (m->finalized) m->g[NVL_T_TOK_EMB].p = m->g[NVL_T_POS_EMB].p = nullptr;
    m->lm_head = nullptr;
}

// ------------------------------------------------------------------------------------------
// the batch being enqueued
// ------------------------------------------------------------------------------------------
// Which tokens take the absorbed attention, and where every other sequence's keys sit in the key workspace.  hm: host metadata with
// the sequences filled in; `steps` one-token passes will run on it (the positions advance on the device).
void layered_meta(nvl_model* m, const Meta& hm, int n_seqs, int steps) {
    bool absorb = !m->masks.empty();
    for (const LayerRun& r : m->runs) if (r.c.mixer == NVL_MIXER_LATENT_ATTENTION) absorb &= lat_absorb_ok(m, r);
    m->n_abs = 0; m->meta_dynamic = false;
    m->min_len = hm.seq_len[0];
    for (size_t w = 0; w < m->masks.size(); w++) { m->key_rows[w] = 0; m->key_max[w] = 0; }
    const int64_t S = m->opts.max_seqs;
    m->win_pairs.assign(m->masks.size(), {0.0, 0.0}); m->win_keys.assign(m->masks.size(), {0.0, 0.0});
    for (int i = 0; i < n_seqs; i++) {
        const int n = hm.seq_len[i], pos = hm.seq_pos[i];
        for (size_t w = 0; w < m->masks.size(); w++) {       // visible (query, key) pairs, keys read: [several new tokens]
            const KeyMask& k = m->masks[w];
            if (k.chunk > 0) {                                // a first part of a chunk, whole chunks, a last part
                auto upto = [&](double p) { const double c = std::floor(p / k.chunk), x = p - c * k.chunk; return c * k.chunk * (k.chunk + 1.0) / 2 + x * (x + 1) / 2; };
                m->win_pairs[w][n > 1] += upto(pos + n) - upto(pos);
                m->win_keys[w][n > 1] += pos + n - k.lo(pos);
                continue;
            }
            m->win_pairs[w][n > 1] += (double)n * std::min<double>(k.keep, std::max(0, pos - k.window)); m->win_keys[w][n > 1] += std::min<double>(k.keep, std::max(0, pos - k.window));      // (kept tokens behind the window, nearly)
            const double W = k.window > 0 ? k.window : 1e18, full = std::min<double>(n, std::max(0.0, pos + n - W));      // tokens whose window is full
            const double part = n - full;                       // the others are the first ones: they see pos + 1 .. pos + part keys
            m->win_pairs[w][n > 1] += full * std::min(W, 1e17) * (full > 0) + part * pos + part * (part + 1) / 2;
            m->win_keys[w][n > 1] += std::min<double>(pos + n, W + n - 1);
        }
        m->min_len = std::min(m->min_len, n);
        const bool abs = absorb && n <= LAT_ABSORB_MAX;
        if (abs) for (int j = 0; j < n; j++) { hm.abs_tok[m->n_abs] = hm.seq_tok_start[i] + j; hm.abs_seq[m->n_abs] = i; m->n_abs++; }
        for (size_t w = 0; w < m->masks.size(); w++) {
            if (abs) { hm.kbase[(int64_t)w * S + i] = -1; continue; }
            int64_t nk = (int64_t)pos + n - latent_key0(pos, m->masks[w].window);
            if (steps > 1) {
                nk = (int64_t)pos + n + steps;
                if (m->masks[w].window > 0) nk = std::min<int64_t>(nk, m->masks[w].window + n + 31);
            }
            hm.kbase[(int64_t)w * S + i] = (int32_t)m->key_rows[w];
            m->key_rows[w] += round_up(nk, 32);
            m->key_max[w] = std::max<int>(m->key_max[w], (int)nk);
            m->meta_dynamic = true;
        }
    }
}

// keys a launch has to cover in the absorbed form, as a power of two of 64-key tiles (a captured pass serves every context up to it)
int layered_kt_log2(const nvl_model* m) {
    int64_t ctx = m->ctx_hint > 0 ? m->ctx_hint : m->cfg.max_seq_len;
    bool windowed = true;
    int w = 0;
    for (const KeyMask& x : m->masks) { windowed &= x.span() > 0; w = std::max(w, x.span() + (x.keep ? 64 : 0)); }
    if (windowed && !m->masks.empty()) ctx = std::min<int64_t>(ctx, w);
    int b = 0;
    while ((64ll << b) < ctx) b++;
    return b;
}
int layered_decode_key(const nvl_model* m) { return layered_kt_log2(m); }

// a sublayer's last projection: fp32 [M][H] in m->ly, or K-split partial sums in m->sk_part (the sandwich norm adds them up)
struct SubOut { const float* y; int slices; int64_t stride; };
// the norm that follows: rms(x) * w, with b a layer norm, or (w NULL, raw) x as it is
struct NextNorm { const float *w, *b; bool raw; };
// experts' results that join the stream beside a sublayer's: K slices, or rows of pairs to be gathered and weighted
struct ExpertOut { const float* y = nullptr; int slices = 0; int64_t stride = 0; const int32_t* slot_of = nullptr; const float* gate_w = nullptr; };
// token shift of the next mixer's input: its weights, the rows kept in the slots (one token per sequence: done by the same launch)
struct ShiftOut { const float* mu = nullptr; float* state = nullptr; const Meta* md = nullptr; };

// x += rms(y) * w_post (w_post NULL: x += y + experts; NVL_BLOCK_SUM_NORM: x = rms(stream_scale x + y + experts) * w_post) and / or
// xn = next(x) (elem.h SandwichArgs)
void sandwich(nvl_model* m, SubOut y, const float* w_post, NextNorm next, void* xn, int rows, const int32_t* rows_idx = nullptr, ExpertOut ex = {}, ShiftOut sh = {}) {
    KScope ks(m, KC_OTHER, 0, KS_SANDWICH, (double)rows * m->Hn * ((y.y ? 8.0 + 4.0 * (std::max(y.slices, 1) + ex.slices) : 4.0) + (next.w || next.raw ? (double)m->wsize : 0.0)));
    SandwichArgs a{};
    a.x = m->x; a.y = y.y; a.slices = y.slices; a.slice_stride = y.stride; a.w_post = w_post; a.w_next = next.w; a.b_next = next.b; a.rows_idx = rows_idx;
    a.rows = rows; a.H = m->H; a.width = m->Hn; a.eps = m->cfg.norm_eps; a.raw_next = next.raw;
    a.y2 = ex.y; a.slices2 = ex.slices; a.stride2 = ex.stride; a.slot_of = ex.slot_of; a.gate_w = ex.gate_w;
    if (m->cfg.block_style == NVL_BLOCK_SUM_NORM && w_post) a.sum_scale = m->cfg.stream_scale;
    if (sh.mu) { a.shift = sh.mu; a.before = sh.state; a.before_stride = m->rec_slot_stride; a.seq_slot = sh.md->seq_slot; a.seq_pos = sh.md->seq_pos; }
    const bool ext = (y.y && !w_post) || next.b || a.sum_scale != 0.f || sh.mu;
    if (!m->f32 && rows > 512 && !sh.mu && m->H <= 4096 && y.slices <= 1) {
        const size_t lds = (size_t)16 * m->H * 2;
#define NVL_SW16E(CH, EXT)                                                                                                  \
        do {                                                                                                                \
            NVL_LDS_ATTR((sandwich_tile16_kernel<CH, EXT>), 160 * 1024);                                                    \
            hipLaunchKernelGGL((sandwich_tile16_kernel<CH, EXT>), dim3(cdiv(rows, 16)), dim3(1024), lds, m->stream, a, (bf16_t*)xn); \
        } while (0)
#define NVL_SW16(CH) do { if (ext) NVL_SW16E(CH, true); else NVL_SW16E(CH, false); } while (0)
        if (m->H <= 1024) NVL_SW16(4); else if (m->H <= 2048) NVL_SW16(8); else NVL_SW16(16);
#undef NVL_SW16
#undef NVL_SW16E
    } else {
#define NVL_SWR(CH)                                                                                                          \
        do {                                                                                                                \
            if (m->f32 && ext) hipLaunchKernelGGL((sandwich_row_kernel<float, CH, true>), dim3(rows), dim3(256), 0, m->stream, a, (float*)xn); \
            else if (m->f32) hipLaunchKernelGGL((sandwich_row_kernel<float, CH>), dim3(rows), dim3(256), 0, m->stream, a, (float*)xn); \
            else if (ext) hipLaunchKernelGGL((sandwich_row_kernel<bf16_t, CH, true>), dim3(rows), dim3(256), 0, m->stream, a, (bf16_t*)xn); \
            else hipLaunchKernelGGL((sandwich_row_kernel<bf16_t, CH>), dim3(rows), dim3(256), 0, m->stream, a, (bf16_t*)xn);      \
        } while (0)
        if (m->H <= 1024) NVL_SWR(1); else if (m->H <= 2048) NVL_SWR(2); else if (m->H <= 4096) NVL_SWR(4); else NVL_SWR(20);
#undef NVL_SWR
    }
    NVL_HIP(hipGetLastError());
}

SubOut sub_out(nvl_model* m, int site, const void* A, const void* W, int M, int K) {
    const int N = m->H;
    int slices = 1;
    if (!m->f32 && M <= 64) {
        const int nblocks = N / 16;
        while (slices < m->sk_max_slices && nblocks * slices < 256 && (K >> 5) / (slices * 2) >= 8) slices *= 2;
    } else if (!m->f32 && M <= 512 && M <= m->sk_rows && N % 128 == 0 && g_force_tile == 0) {
        const int tiles = cdiv(M, 128) * (N / 128);
        while (slices < SK_TILE_MAX_SLICES && tiles * slices < 512 && K / (slices * 2) >= 512) slices *= 2;
        if (tiles * slices < 64) slices = 1;
    }
    m->site = site;
    GemmArgs a = mk(A, K, W, m->ly, N, nullptr, 1.f, M, N, K);
    if (slices > 1) {
        a.C = m->x; a.sk_part = m->sk_part; a.sk_slices = slices;      // (EPI_RESID with slices: plain stores into sk_part, x is not touched)
        gemm(m, EPI_RESID, true, a);
        return {m->sk_part, slices, (int64_t)M * N};
    }
    gemm(m, EPI_STORE, true, a);
    return {m->ly, 1, 0};
}

void grow(nvl_model* m, float*& p, int64_t& have, int64_t want) {
    if (want <= have) return;
    clear_graphs(m);
    dfree(p);
    p = dmalloc<float>(want);
    have = want;
}

// ------------------------------------------------------------------------------------------
// mixers: read the normed operand m->xn, leave the mixer's output before its last projection in m->lmix
// ------------------------------------------------------------------------------------------
void in_proj(nvl_model* m, const LayerRun& r, const MixerW& w, int M) {
    m->site = KS_MIX_IN;
    gemm(m, EPI_STORE, true, mk(m->xn, m->H, w.in, m->lproj, (int)m->lproj_ld, w.in_bias, 1.f, M, r.n_in, m->H));
}

void mix_latent(nvl_model* m, const LayerRun& r, const MixerW& w, const Meta& md, int n_seqs, int M, int max_len) {
    const nvl_layer_config& c = r.c;
    const int H = c.heads;
    const double ws = (double)m->wsize;
    in_proj(m, r, w, M);
    LatentArgs a{};
    a.H = H; a.dim = c.dim; a.dn = r.dn; a.dp = r.dp; a.rot = c.rot_dim; a.rotp = r.rotp; a.turn = r.turn;
    a.own = m->mixers[(size_t)r.owner].dkv_norm != nullptr; a.gate_off = r.gate_off; a.gate_head = c.gate_per_head; a.vp = r.vp; a.qrank = c.q_rank; a.qrp = r.qrp; a.kvrank = c.kv_rank; a.rp = r.rp;
    a.window = c.window; a.scale = c.scale; a.eps = m->cfg.norm_eps;
    a.proj = m->lproj; a.proj_ld = m->lproj_ld; a.cq_norm = w.dq_norm; a.c_norm = w.dkv_norm; a.cq = m->lcq;
    a.cache = (char*)m->lat_cache + r.cache_off * (int64_t)m->wsize; a.block_stride = m->lat_block_stride; a.bs = m->Tmax;
    a.blk_table = md.blk_table; a.tok_pos = md.tok_pos; a.tok_tbl = md.tok_tbl; a.seq_tok_start = md.seq_tok_start; a.seq_len = md.seq_len;
    a.seq_pos = md.seq_pos; a.tbl_stride = m->blocks_per_seq;
    a.q = m->lq; a.q_ld = (int64_t)H * r.dp;
    a.kbase = md.kbase + (int64_t)r.win * m->opts.max_seqs;
    a.out = m->lmix; a.out_ld = r.kd;
    {
        KScope ks(m, KC_OTHER, 0, KS_LAT_NORM, (double)M * (c.q_rank + (a.own ? c.kv_rank + c.rot_dim : 0)) * (4.0 + ws));
        if (m->f32) hipLaunchKernelGGL((latent_norm_kernel<float>), dim3(M), dim3(256), 0, m->stream, a);
        else hipLaunchKernelGGL((latent_norm_kernel<bf16_t>), dim3(M), dim3(256), 0, m->stream, a);
        NVL_HIP(hipGetLastError());
    }
    m->site = KS_LAT_UQ;
    gemm(m, EPI_STORE, true, mk(m->lcq, r.qrp, w.uq, m->lq, H * r.dp, nullptr, 1.f, M, H * r.dp, r.qrp));
    a.turn_q = c.rot_dim && c.rot_dim % 16 == 0;
    if (c.rot_dim && !a.turn_q) {
        KScope ks(m, KC_OTHER, 0, KS_ROPE, 8.0 * M * H * c.rot_dim);
        hipLaunchKernelGGL(latent_turn_q_kernel, dim3(M, H), dim3(64), 0, m->stream, a);
        NVL_HIP(hipGetLastError());
    }
    const int64_t rows = m->key_rows[(size_t)r.win];
    if (rows > 0) {                       // sequences on the expanded form
        if (rows > m->key_rows_cap) {
            int64_t kc = 0, kr = 0, kk = 0, kv = 0;
            for (const LayerRun& q : m->runs) if (q.c.mixer == NVL_MIXER_LATENT_ATTENTION) {
                kc = std::max<int64_t>(kc, q.rp); kr = std::max<int64_t>(kr, q.rotp); kk = std::max<int64_t>(kk, (int64_t)q.c.heads * q.dn); kv = std::max<int64_t>(kv, (int64_t)q.c.heads * q.vp);
            }
            clear_graphs(m);
            dfree(m->key_c); dfree(m->key_r); dfree(m->key_k); dfree(m->key_v);
            m->key_c = m->key_r = m->key_k = m->key_v = nullptr; m->key_rows_cap = 0; m->key_src = -1;
            const int64_t cap = round_up(rows + rows / 4, 256) + 256, wsz = (int64_t)m->wsize;     // (+ whole GEMM tiles beyond the last row)
            m->key_c = dmalloc_bytes(cap * kc * wsz); m->key_r = dmalloc_bytes(std::max<int64_t>(cap * kr * wsz, 16)); m->key_k = dmalloc_bytes(cap * kk * wsz); m->key_v = dmalloc_bytes(cap * kv * wsz);
            NVL_HIP(hipMemsetAsync(m->key_c, 0, (size_t)(cap * kc * wsz), m->stream));
            NVL_HIP(hipMemsetAsync(m->key_k, 0, (size_t)(cap * kk * wsz), m->stream));
            NVL_HIP(hipMemsetAsync(m->key_v, 0, (size_t)(cap * kv * wsz), m->stream));
            m->key_rows_cap = cap - 256;
        }
        a.cg = m->key_c; a.kr = m->key_r; a.kx = m->key_k; a.vx = m->key_v; a.rows_pad = rows;
        if (m->key_src != r.src || m->key_win != r.win) {       // (else: the layer before this one read the same latents)
            m->key_src = r.src; m->key_win = r.win;
            KScope ks(m, KC_OTHER, 0, KS_LAT_GATHER, 2.0 * (double)rows * (c.kv_rank + c.rot_dim) * ws);
            const dim3 grid(cdiv(m->key_max[(size_t)r.win], 32), n_seqs);
            if (m->f32) hipLaunchKernelGGL((latent_gather_kernel<float>), grid, dim3(256), 0, m->stream, a);
            else hipLaunchKernelGGL((latent_gather_kernel<bf16_t>), grid, dim3(256), 0, m->stream, a);
            NVL_HIP(hipGetLastError());
        }
        m->site = KS_LAT_KV;
        gemm(m, EPI_STORE, m->f32, mk(m->key_c, r.rp, w.uk, m->key_k, H * r.dn, nullptr, 1.f, (int)rows, H * r.dn, r.rp));
        m->site = KS_LAT_KV;
        if (m->f32) gemm(m, EPI_STORE, true, mk(m->key_c, r.rp, w.uv, m->key_v, H * r.vp, nullptr, 1.f, (int)rows, H * r.vp, r.rp));
        else gemm(m, EPI_STORE, false, mk(w.uv, r.rp, m->key_c, m->key_v, (int)rows, nullptr, 1.f, H * r.vp, (int)rows, r.rp));     // V^T = W_uv c^T
        {
            // visible (query, key) pairs are at most tokens x min(window, keys)
            const double pairs = (double)(M - m->n_abs) * (c.window > 0 ? std::min<double>(c.window, m->key_max[(size_t)r.win]) : 0.5 * m->key_max[(size_t)r.win]);
            KScope ks(m, KC_ATTN, 2.0 * pairs * H * (c.dim + c.rot_dim + c.vdim), KS_ATTN,
                      ((double)rows * (H * (c.dim + c.vdim) + c.rot_dim)) * ws + (double)M * H * (4.0 * (c.dim + c.rot_dim) + (c.gate_per_head ? 4.0 : 4.0 * c.vdim) + ws * c.vdim));
            if (m->f32 || r.dp > 256 || r.vp > 256 || c.scale == 0.f) {
                const dim3 grid(max_len, H, n_seqs);
                const size_t lds = (size_t)(r.dp + r.vp) * 4;
                if (m->f32) hipLaunchKernelGGL((latent_plain_kernel<float>), grid, dim3(256), lds, m->stream, a);
                else hipLaunchKernelGGL((latent_plain_kernel<bf16_t>), grid, dim3(256), lds, m->stream, a);
            } else {
                latent_prefill_launch(m->stream, a, n_seqs, max_len);
            }
            NVL_HIP(hipGetLastError());
        }
    }
    if (m->n_abs > 0) {
        const int n = m->n_abs, ht = cdiv(H, 16);
        a.abs_tok = md.abs_tok; a.abs_seq = md.abs_seq; a.n_abs = n; a.ukt = (const bf16_t*)w.ukt; a.uv = (const bf16_t*)w.uv;
        a.qa = m->lat_qa; a.Hp = ht * 16; a.part_o = m->lat_part_o; a.part_ml = m->lat_part_ml;
        const int tiles = 1 << layered_kt_log2(m);
        int split = 1;
        while (split < LAT_SPLITS && ht * n * split < 256 && split * 2 <= tiles && (split * 2) * n <= m->lat_abs_cap) split *= 2;
        a.n_split = split;
        {
            KScope ks(m, KC_OTHER, 2.0 * n * H * (double)c.dim * c.kv_rank, KS_LAT_ABSORB, (double)H * c.dim * c.kv_rank * 2.0 + (double)n * H * (4.0 * (c.dim + c.rot_dim) + 2.0 * (c.kv_rank + c.rot_dim)));
            hipLaunchKernelGGL(latent_absorb_q_kernel, dim3(H, r.rp / 64 + (c.rot_dim > 0), cdiv(n, 16)), dim3(256), 0, m->stream, a);
            NVL_HIP(hipGetLastError());
        }
        {
            const double keys = m->kv_tok > 0 && c.window > 0 ? std::min(m->kv_tok, (double)n * c.window) : (m->kv_tok > 0 ? m->kv_tok : (double)n * std::max(1, c.window));
            KScope ks(m, KC_ATTN, keys * H * (4.0 * c.kv_rank + 2.0 * c.rot_dim), KS_ATTN, keys * (c.kv_rank + c.rot_dim) * 2.0 + (double)n * H * c.kv_rank * (2.0 + 4.0 * split));
            const dim3 grid(ht, n, split);
            latent_decode_launch(m->stream, a, grid);
            NVL_HIP(hipGetLastError());
        }
        {
            KScope ks(m, KC_OTHER, 2.0 * n * H * (double)c.vdim * c.kv_rank, KS_LAT_UV, (double)H * c.vdim * c.kv_rank * 2.0 + (double)n * H * (4.0 * split * c.kv_rank + 6.0 * c.vdim));
            hipLaunchKernelGGL(latent_uv_kernel, dim3(H, cdiv(r.vp, 256), cdiv(n, 16)), dim3(1024), (size_t)16 * r.rp * 2, m->stream, a);
            NVL_HIP(hipGetLastError());
        }
    }
}

// the recurrence of a layer over the batch; fused: one token (or a few) per sequence, everything between the projections in one launch
template <bool CH>
void linrec(nvl_model* m, LinRecArgs a, int n_seqs, int M, int max_len, bool fused, int site) {
    const double elems = (double)a.H * a.DK * a.DVp;
    const double bytes = (double)M * a.H * (2.0 * a.DK / a.kdiv + 2.0 * a.DV) * 4.0 + 2.0 * n_seqs * elems * 4.0;
    KScope ks(m, KC_OTHER, 4.0 * (double)M * a.H * a.DK * a.DV, site, bytes);
    a.len_lo = 1; a.len_hi = 1 << 30;
    if (fused) {
        linrec_step_launch(m->stream, a, n_seqs, CH, true, m->f32);
        return;
    }
    const int nk = a.DK <= 32 ? 2 : (a.DK <= 64 ? 4 : (a.DK <= 128 ? 8 : 16)), nw = a.DV <= 64 ? 4 : 8;
    const bool chunks = a.DK <= 256 && (!CH || linrec_chunk_lds_bytes<16, 8, true>(a.rank) <= 160 * 1024 || nk < 16);
    const bool steps = !chunks || m->min_len <= REC_STEP_MAX;
    if (steps) {
        a.len_hi = chunks ? REC_STEP_MAX : 1 << 30;
        linrec_step_launch(m->stream, a, n_seqs, CH, false, m->f32);
    }
    if (!chunks || max_len <= REC_STEP_MAX) return;
    a.len_lo = REC_STEP_MAX + 1; a.len_hi = 1 << 30;
    a.vec4 = a.DK % 4 == 0 && a.DV % 4 == 0 && a.ld % 4 == 0 && (((uintptr_t)a.q | (uintptr_t)a.k | (uintptr_t)a.v) & 15) == 0;
    a.n_slices = cdiv(a.DV, nw * 16);
    // few (head, sequence, slice) workgroups and a long prompt: pieces of the prompt in parallel (MODE 1, prefix, MODE 2)
    const int wgs = a.H * n_seqs * a.n_slices;
    a.super = 0; a.n_super = 1;
    if (wgs < 256 && max_len >= 512) {
        const int want = std::max(2, 512 / wgs);
        a.super = (int)round_up(std::max(128, cdiv(max_len, want)), 32);
        a.n_super = cdiv(max_len, a.super);
    }
    const bool par = a.n_super > 1;
    if (par) {
        grow(m, m->rec_z, m->rec_z_floats, (int64_t)n_seqs * a.n_super * a.H * a.DK * a.DVp);
        grow(m, m->rec_decay, m->rec_decay_floats, (int64_t)n_seqs * a.n_super * a.H * (CH ? a.DK : 1));
        a.z = m->rec_z; a.zdecay = m->rec_decay;
    }
    linrec_chunk_launch(m->stream, a, n_seqs, CH, nk, nw, par);
    NVL_HIP(hipGetLastError());
}

template <typename ActT, bool GATE_FIRST>
void gated_norm_launch(nvl_model* m, GatedNormArgs a, int col) {
    const bool v4 = a.part % 4 == 0 && a.y_ld % 4 == 0 && a.gate_ld % 4 == 0 && (((uintptr_t)a.y | (uintptr_t)a.gate) & 15) == 0;
    const bool wide = a.part > 1024;
    a.lanes = 4;
    while (a.lanes < 64 && a.lanes * (v4 ? 4 : 1) < a.part) a.lanes *= 2;
    const dim3 grid(wide ? a.rows * a.parts : cdiv((int64_t)a.rows * a.parts, 256 / a.lanes));
    ActT* out = (ActT*)m->lmix + (sizeof(ActT) == 2 ? (int64_t)(col >> 5) * 512 : col);      // (the operand's column blocks are 32 wide: a shift by columns is a shift of the base)
    if (wide && v4) hipLaunchKernelGGL((gated_norm_kernel<ActT, GATE_FIRST, true, true>), grid, dim3(256), 0, m->stream, a, out);
    else if (wide) hipLaunchKernelGGL((gated_norm_kernel<ActT, GATE_FIRST, true, false>), grid, dim3(256), 0, m->stream, a, out);
    else if (v4) hipLaunchKernelGGL((gated_norm_kernel<ActT, GATE_FIRST, false, true>), grid, dim3(256), 0, m->stream, a, out);
    else hipLaunchKernelGGL((gated_norm_kernel<ActT, GATE_FIRST, false, false>), grid, dim3(256), 0, m->stream, a, out);
}
template <bool GATE_FIRST>
void gated_norm(nvl_model* m, const GatedNormArgs& a, int site, int col = 0) {
    KScope ks(m, KC_OTHER, 0, site, (double)a.rows * a.parts * a.part * (8.0 + (double)m->wsize));
    if (m->f32) gated_norm_launch<float, GATE_FIRST>(m, a, col);
    else gated_norm_launch<bf16_t, GATE_FIRST>(m, a, col);
    NVL_HIP(hipGetLastError());
}

LinRecArgs linrec_args(nvl_model* m, const LayerRun& r, const Meta& md) {
    LinRecArgs a{};
    a.H = r.c.heads; a.DV = r.c.vdim; a.DVp = (int)round_up(r.c.vdim, 4);
    a.o = m->lo; a.o_ld = m->lo_ld;
    a.state = m->rec_state + r.state_off; a.slot_stride = m->rec_slot_stride;
    a.seq_tok_start = md.seq_tok_start; a.seq_len = md.seq_len; a.seq_pos = md.seq_pos; a.seq_slot = md.seq_slot;
    a.eps = m->cfg.norm_eps; a.out = m->lmix; a.out_ld = r.kd;
    return a;
}

// causal convolution + silu of the batch's raw rows into m->lconv, then the newest rows into the slots' rings
void conv_launch(nvl_model* m, const LayerRun& r, const MixerW& w, const Meta& md, float* ring, const float* raw, int n_seqs, int M) {
    ConvArgs v{};
    v.raw = raw; v.raw_ld = m->lproj_ld; v.w = w.conv_w; v.b = w.conv_b; v.taps = r.c.conv_taps; v.channels = r.conv_dim;
    v.out = m->lconv; v.out_ld = m->lconv_ld; v.ring = ring; v.ring_slot_stride = m->rec_slot_stride;
    v.tok_seq = md.tok_seq; v.tok_pos = md.tok_pos; v.seq_tok_start = md.seq_tok_start; v.seq_len = md.seq_len; v.seq_pos = md.seq_pos; v.seq_slot = md.seq_slot;
    const bool v4 = r.conv_dim % 4 == 0 && v.raw_ld % 4 == 0 && ((uintptr_t)v.raw & 15) == 0;
    const dim3 cgrid(cdiv(M, CONV_TOKENS), cdiv(r.conv_dim, 1024));
    if (v4 && v.taps == 4) hipLaunchKernelGGL((conv_silu_kernel<4>), cgrid, dim3(256), 0, m->stream, v, M);
    else if (v4 && v.taps == 3) hipLaunchKernelGGL((conv_silu_kernel<3>), cgrid, dim3(256), 0, m->stream, v, M);
    else if (v4 && v.taps == 2) hipLaunchKernelGGL((conv_silu_kernel<2>), cgrid, dim3(256), 0, m->stream, v, M);
    else hipLaunchKernelGGL((conv_silu_kernel<0>), cgrid, dim3(256), 0, m->stream, v, M);
    hipLaunchKernelGGL(conv_ring_kernel, dim3(n_seqs, cdiv(r.conv_dim, 256)), dim3(256), 0, m->stream, v);
    NVL_HIP(hipGetLastError());
}

void mix_mamba2(nvl_model* m, const LayerRun& r, const MixerW& w, const Meta& md, int n_seqs, int M, int max_len) {
    const nvl_layer_config& c = r.c;
    const int inner = c.heads * c.vdim, GN = c.groups * c.state;
    in_proj(m, r, w, M);
    LinRecArgs a = linrec_args(m, r, md);
    a.DK = c.state; a.kdiv = c.heads / c.groups; a.q_scale = 1.f;
    a.dt = m->lproj + inner + r.conv_dim; a.dt_ld = m->lproj_ld; a.dt_bias = w.dt_bias; a.a_log = w.a_log; a.Dskip = w.dskip;
    float* ring = m->rec_state + r.ring_off;
    const bool fused = max_len == 1;
    if (fused) {
        a.raw = m->lproj + inner; a.raw_ld = m->lproj_ld; a.conv_w = w.conv_w; a.conv_b = w.conv_b; a.taps = c.conv_taps; a.conv_dim = r.conv_dim;
        a.ring = ring; a.ring_slot_stride = m->rec_slot_stride;
    } else {
        KScope ks(m, KC_OTHER, 0, KS_MAMBA_CONV, (double)M * r.conv_dim * 8.0);
        conv_launch(m, r, w, md, ring, m->lproj + inner, n_seqs, M);
        a.v = m->lconv; a.k = m->lconv + inner; a.q = m->lconv + inner + GN; a.ld = m->lconv_ld;
    }
    linrec<false>(m, a, n_seqs, M, max_len, fused, KS_MAMBA_SCAN);
    GatedNormArgs g{m->lo, m->lo_ld, m->lproj, m->lproj_ld, w.mix_norm, M, c.norm_groups, inner / c.norm_groups, m->cfg.norm_eps, r.kd, 0, 0};
    gated_norm<true>(m, g, KS_MAMBA_GATE);
}

void mix_gla(nvl_model* m, const LayerRun& r, const MixerW& w, const Meta& md, int n_seqs, int M, int max_len) {
    const nvl_layer_config& c = r.c;
    const int64_t hd = (int64_t)c.heads * c.dim, hv = (int64_t)c.heads * c.vdim;
    in_proj(m, r, w, M);
    LinRecArgs a = linrec_args(m, r, md);
    a.DK = c.dim; a.kdiv = 1; a.q_scale = 1.0f / sqrtf((float)c.dim);
    a.q = m->lproj; a.k = m->lproj + hd; a.v = m->lproj + 2 * hd; a.ld = m->lproj_ld;
    a.gate = m->lproj + 2 * hd + hv; a.gate_ld = m->lproj_ld; a.norm_w = w.mix_norm;
    a.a1 = m->lproj + 2 * hd + 2 * hv; a.a1_ld = m->lproj_ld; a.rank = w.rank; a.a2 = w.a2; a.a2_b = w.a2_b; a.inv_tau = 1.0f / c.tau;
    const bool fused = max_len <= REC_STEP_MAX;
    linrec<true>(m, a, n_seqs, M, max_len, fused, KS_GLA_SCAN);
    if (fused) return;
    GatedNormArgs g{m->lo, m->lo_ld, a.gate, m->lproj_ld, w.mix_norm, M, c.heads, c.vdim, m->cfg.norm_eps, r.kd, 0, 0};
    gated_norm<false>(m, g, KS_GLA_GATE);
}

void mix_delta(nvl_model* m, const LayerRun& r, const MixerW& w, const Meta& md, int n_seqs, int M, int max_len) {
    const nvl_layer_config& c = r.c;
    const int64_t qk = (int64_t)c.kv_heads * c.dim, hd = (int64_t)c.heads * c.dim, hv = (int64_t)c.heads * c.vdim;
    in_proj(m, r, w, M);
    DeltaArgs a{};
    a.H = c.heads; a.G = c.kv_heads; a.DK = c.dim; a.DV = c.vdim; a.DVp = (int)round_up(c.vdim, 4);
    a.q_scale = 1.0f / sqrtf((float)c.dim);
    a.a_log = w.a_log; a.dt_bias = w.dt_bias;
    a.beta = m->lproj + r.b_off; a.beta_ld = m->lproj_ld;
    a.o = m->lo; a.o_ld = m->lo_ld;
    a.state = m->rec_state + r.state_off; a.slot_stride = m->rec_slot_stride;
    a.seq_tok_start = md.seq_tok_start; a.seq_len = md.seq_len; a.seq_pos = md.seq_pos; a.seq_slot = md.seq_slot;
    a.len_lo = 1; a.len_hi = 1 << 30;
    float* ring = m->rec_state + r.ring_off;
    const double elems = (double)a.H * a.DK * a.DVp;
    if (max_len == 1) {       // everything between the projections in one launch
        a.raw = m->lproj; a.raw_ld = m->lproj_ld; a.conv_w = w.conv_w; a.taps = c.conv_taps; a.channels = r.conv_dim;
        a.ring = ring; a.ring_slot_stride = m->rec_slot_stride;
        a.a1 = m->lproj + r.a1_off; a.g1 = m->lproj + r.g1_off; a.lr_ld = m->lproj_ld;
        a.a_rank = w.rank; a.g_rank = w.grank; a.a_rkp = w.a_rkp; a.g_rkp = w.g_rkp; a.a2 = w.a2r; a.g2 = w.g2r;
        a.norm_w = w.mix_norm; a.eps = m->cfg.norm_eps; a.out = m->lmix; a.out_ld = r.kd;
        KScope ks(m, KC_OTHER, 6.0 * M * elems, KS_DELTA_SCAN, 2.0 * n_seqs * elems * 4.0 + (double)M * (r.conv_dim * 4.0 * (c.conv_taps + 1) + hv * (double)m->wsize) +
                                                                   ((double)hd * w.rank + (double)hv * w.grank) * (double)m->wsize);
        delta_step_launch(m->stream, a, n_seqs, true, m->f32);
        return;
    }
    {
        KScope ks(m, KC_OTHER, 0, KS_DELTA_CONV, (double)M * r.conv_dim * 8.0);
        conv_launch(m, r, w, md, ring, m->lproj, n_seqs, M);
    }
    {
        KScope ks(m, KC_OTHER, 0, KS_DELTA_PACK, (double)M * (w.rank + w.grank) * (4.0 + (double)m->wsize));
        const PackArgs p{m->lproj + r.a1_off, m->lproj_ld, w.rank, w.a_rkp, w.grank, w.g_rkp, r.g1_off - r.a1_off, m->lpa, m->lpg};
        if (m->f32) hipLaunchKernelGGL((pack_rows_kernel<float>), dim3(M), dim3(64), 0, m->stream, p);
        else hipLaunchKernelGGL((pack_rows_kernel<bf16_t>), dim3(M), dim3(64), 0, m->stream, p);
        NVL_HIP(hipGetLastError());
    }
    m->site = KS_DELTA_RANK;
    gemm(m, EPI_STORE, true, mk(m->lpa, w.a_rkp, w.a2m, m->lz, (int)m->lz_ld, nullptr, 1.f, M, (int)hd, w.a_rkp));
    m->site = KS_DELTA_RANK;
    gemm(m, EPI_STORE, true, mk(m->lpg, w.g_rkp, w.g2m, m->lg, (int)m->lg_ld, nullptr, 1.f, M, (int)hv, w.g_rkp));
    a.q = m->lconv; a.k = m->lconv + qk; a.v = m->lconv + 2 * qk; a.ld = m->lconv_ld;
    a.z = m->lz; a.z_ld = m->lz_ld;
    const double io = (double)M * (2.0 * qk + hd + 2.0 * hv) * 4.0;
    const bool chunks = c.dim <= 256;
    if (!chunks || m->min_len <= REC_STEP_MAX) {
        a.len_hi = chunks ? REC_STEP_MAX : 1 << 30;
        KScope ks(m, KC_OTHER, chunks ? 0.0 : 6.0 * M * elems, KS_DELTA_SCAN, chunks ? 0.0 : io + 2.0 * n_seqs * elems * 4.0);
        delta_step_launch(m->stream, a, n_seqs, false, m->f32);
    }
    if (chunks && max_len > REC_STEP_MAX) {
        a.len_lo = REC_STEP_MAX + 1; a.len_hi = 1 << 30;
        a.vec4 = c.dim % 4 == 0 && qk % 4 == 0 && a.ld % 4 == 0;
        a.vec4v = c.vdim % 4 == 0 && 2 * qk % 4 == 0 && a.ld % 4 == 0 && a.o_ld % 4 == 0;
        const int nk = c.dim <= 32 ? 2 : (c.dim <= 64 ? 4 : (c.dim <= 128 ? 8 : 16));
        grow(m, m->delta_ws, m->delta_ws_cap, (int64_t)(m->opts.max_batch_tokens / DELTA_C + m->opts.max_seqs + 1) * c.heads * delta_ws_floats(nk * 16));
        a.ws = m->delta_ws;
        const dim3 pgrid(c.heads, n_seqs, cdiv(max_len, DELTA_C));
        const double scratch = (double)M * c.heads * (3.0 * nk * 16 + 2.0 * c.vdim) * 4.0;
        {
            KScope ks(m, KC_OTHER, 0, KS_DELTA_PREP, io + scratch);
            delta_prep_launch(m->stream, a, pgrid, nk);
            NVL_HIP(hipGetLastError());
        }
        {
            KScope ks(m, KC_OTHER, 6.0 * M * elems, KS_DELTA_SCAN, scratch + 2.0 * n_seqs * elems * 4.0);
            delta_scan_launch(m->stream, a, n_seqs, nk);
            NVL_HIP(hipGetLastError());
        }
    }
    GatedNormArgs g{m->lo, m->lo_ld, m->lg, m->lg_ld, w.mix_norm, M, c.heads, c.vdim, m->cfg.norm_eps, r.kd, 0, 1};
    gated_norm<false>(m, g, KS_DELTA_GATE);
}

void tap_layer(nvl_model* m, int li, int M);

// ---- lightning attention beside another mixer: columns of the joint input projection -> m->lmix columns [ko, ko + ko2) ----
void mix_lightning(nvl_model* m, const LayerRun& r, const MixerW& w, const Meta& md, int n_seqs, int M, int max_len) {
    const nvl_layer_config& c = r.c;
    LinRecArgs a = linrec_args(m, r, md);
    a.H = c.heads2; a.DK = c.dim2; a.DV = c.vdim2; a.DVp = (int)round_up(c.vdim2, 4); a.kdiv = 1; a.q_scale = 1.f;
    a.q = m->lproj + r.lq_off; a.k = m->lproj + r.lk_off; a.v = m->lproj + r.lv_off; a.ld = m->lproj_ld;
    a.decay = w.decay; a.log2_decay = w.log2_decay;
    linrec<false>(m, a, n_seqs, M, max_len, false, KS_LIN_SCAN);
    GatedNormArgs g{m->lo, m->lo_ld, m->lproj + r.lg_off, m->lproj_ld, w.lin_norm, M, 1, c.heads2 * c.vdim2, m->cfg.norm_eps, r.kd, 0, 1};
    gated_norm<false>(m, g, KS_LIN_GATE, r.ko);
}

// ---- grouped-query attention: m->xn -> m->lmix columns [0, ko) ----
void mix_grouped(nvl_model* m, const LayerRun& r, const MixerW& w, const Meta& md, int n_seqs, int M, int max_len) {
    const nvl_layer_config& c = r.c;
    GroupedArgs a{};
    a.H = c.heads; a.G = c.kv_heads; a.group = c.heads / c.kv_heads; a.dim = c.dim; a.dp = r.dp; a.vdim = c.vdim; a.vp = r.vp;
    a.mask = m->masks[(size_t)r.win]; a.scale = c.scale; a.softcap = c.softcap; a.r1 = w.r1; a.r2 = w.r2; a.sink = w.sink; a.out_scale = c.out_scale != 0.f ? c.out_scale : 1.f;
    a.mix = r.mix; a.lambda = w.v_lambda; a.vfirst = m->lvf; a.vfirst_ld = m->lvf_ld;
    a.cache = (char*)m->lat_cache + r.cache_off * (int64_t)m->wsize; a.block_stride = m->lat_block_stride; a.bs = m->Tmax;
    a.blk_table = md.blk_table; a.seq_tok_start = md.seq_tok_start; a.seq_len = md.seq_len; a.seq_pos = md.seq_pos; a.tbl_stride = m->blocks_per_seq;
    a.out = m->lmix; a.out_ld = r.kd;
    const double ws = (double)m->wsize;
    if (m->f32) {
        in_proj(m, r, w, M);
        a.q = m->lproj; a.q_ld = m->lproj_ld; a.gate_col = c.ungated ? -1 : r.gate_off;
        a.proj = m->lproj; a.proj_ld = m->lproj_ld; a.k_off = r.raw ? -1 : r.k_off; a.v_off = r.v_off;
        if (c.mixer2) {
            KScope ks(m, KC_OTHER);
            hipLaunchKernelGGL(silu_cols_kernel, dim3(M), dim3(256), 0, m->stream, m->lproj, m->lproj_ld, r.lq_off, r.lg_off - r.lq_off);
            NVL_HIP(hipGetLastError());
        }
        KScope ks(m, KC_OTHER, 0, KS_KV_PLACE, (double)M * a.G * (c.dim + c.vdim) * (4.0 + ws) + (r.mix ? (double)M * a.G * c.vdim * 4.0 : 0.0));
        hipLaunchKernelGGL(grouped_place_kernel, dim3(cdiv(max_len + 31, 32), n_seqs, a.G), dim3(256), 0, m->stream, a);
        NVL_HIP(hipGetLastError());
    } else {
        a.q = m->lqg; a.q_ld = (int64_t)a.H * (r.dp + (c.ungated ? 0 : r.vp)); a.gate_col = c.ungated ? -1 : a.H * r.dp;
        GemmArgs g = mk(m->xn, m->H, w.in, m->lqg, (int)a.q_ld, w.in_bias, 1.f, M, r.n_in, m->H);
        g.grp = GroupedEpi{r.k_off, r.v_off, r.gate_off, r.raw ? 1 << 30 : r.ffn_off, r.raw ? 1 << 30 : r.ffn_in ? r.route_off : r.ffn_off, md.tok_pos, md.tok_tbl, md.blk_table, (bf16_t*)a.cache, a.block_stride, a.bs, a.G, r.dp, r.vp,
                           r.mix, w.v_lambda, m->lvf, m->lvf_ld, (bf16_t*)m->lmix + (r.ko >> 5) * 512, r.kd, m->lproj, m->lproj_ld,
                           m->lproj, m->lproj_ld, r.ffn_off, c.mixer2 ? r.lg_off : 0};
        m->site = KS_MIX_IN;
        gemm(m, r.raw ? EPI_GROUPED_RAW : EPI_GROUPED, false, g);
    }
    if (c.mixer2) mix_lightning(m, r, w, md, n_seqs, M, max_len);
    if (r.raw) {          // norms and rotation of the fp32 queries and keys
        a.proj = m->lproj; a.proj_ld = m->lproj_ld; a.qk_koff = r.k_off; a.qk_norm = c.qk_norm; a.q_norm = w.q_norm; a.k_norm = w.k_norm; a.eps = m->cfg.norm_eps;
        a.rot = c.rot_dim; a.turn = r.turn; a.tok_pos = md.tok_pos; a.tok_tbl = md.tok_tbl; a.rows = M;
        a.q = a.q_out = m->lqg; a.q_ld = (int64_t)a.H * r.dp;
        KScope ks(m, KC_OTHER, 0, KS_QK_TURN, (double)M * (a.H + a.G) * c.dim * (4.0 + ws));
        grouped_qk_launch(m->stream, a, m->f32);
        NVL_HIP(hipGetLastError());
    }
    const bool plain = m->f32 || r.dp > 256 || r.vp > 256;
    const int ctx = m->ctx_hint > 0 ? m->ctx_hint : m->cfg.max_seq_len;
    int tiles = cdiv(ctx, 64) + 1;                              // most key tiles a 256-row workgroup walks
    const int span = a.mask.span();
    if (span > 0) tiles = std::min(tiles, (span + cdiv(256, a.group) + 1) / 64 + 3 + cdiv(a.mask.keep, 64));
    const size_t ring = (size_t)3 * round_up(4 * (r.dp >> 5) + 2 * (r.vp >> 4), 8) * 1024;
    size_t lds = ring + (size_t)tiles * 8;
    // the distance biases of a workgroup's rows as a table in LDS, where they leave as many workgroups per CU as the ring does
    const size_t tab = lds + (size_t)grouped_tab_span(std::min(ctx, span > 0 ? span : ctx)) * a.group * 4;
    if (w.r1 && !a.mask.keep && tab <= (size_t)(r.dp <= 64 && r.vp <= 64 ? 80 : 160) * 1024) { a.table = tiles; lds = tab; }
    a.short_rows = GROUPED_SHORT_ROWS;
    if ((r.dp == 256 && r.vp == 256) || lds > 160 * 1024) a.short_rows = 1 << 30;      // (three slots would not fit LDS)
    const bool any_short = m->min_len * a.group <= a.short_rows, any_long = max_len * a.group > a.short_rows;
    auto scope = [&](int several) {
        const double pairs = m->win_pairs[(size_t)r.win][(size_t)several], keys = m->win_keys[(size_t)r.win][(size_t)several];
        return KScope(m, KC_ATTN, 2.0 * pairs * a.H * (c.dim + c.vdim), KS_ATTN, (keys * a.G * (c.dim + c.vdim) + (double)M * a.H * (c.dim + 2.0 * c.vdim)) * ws);
    };
    if (plain) {
        KScope ks = scope(max_len > 1);
        const dim3 grid(max_len, a.H, n_seqs);
        const size_t sm = (size_t)(r.dp + r.vp) * 4;
        if (m->f32) hipLaunchKernelGGL((grouped_plain_kernel<float>), grid, dim3(256), sm, m->stream, a);
        else hipLaunchKernelGGL((grouped_plain_kernel<bf16_t>), grid, dim3(256), sm, m->stream, a);
        NVL_HIP(hipGetLastError());
        return;
    }
    const int dt = r.vp >> 4;
    if (any_long) {
        KScope scp = scope(1);
        const dim3 grid(a.G, n_seqs, cdiv((int64_t)max_len * a.group, 256));
        grouped_prefill_launch(m->stream, a, grid, lds, a.table && w.bias_lowers && c.softcap > 0.f && c.softcap <= GROUPED_FAST_CAP);
        NVL_HIP(hipGetLastError());
    }
    if (any_short) {
        KScope scp = scope(any_long ? 0 : max_len > 1);
        const int64_t wgs = (int64_t)a.G * cdiv(std::min<int64_t>((int64_t)max_len * a.group, a.short_rows), 16);
        // Key tiles are split over workgroups once a wave would walk more than two: a split costs a round trip to memory and back (one
        // sequence of 2048 tokens with a window of 1024: 13.1 us unsplit, 13.7 in four; without a window, 3900 tokens: 27.8 -> 16.6 us)
        const int key_tiles = 1 << layered_kt_log2(m), nw = dt <= 8 ? 8 : 4;
        int z = 1;
        while (z < GROUPED_SPLITS && wgs * n_seqs * z * 2 <= 256 && z * 2 * 2 * nw <= key_tiles) z *= 2;
        if (g_grouped_split) z = (int)std::min<int64_t>(g_grouped_split, std::max<int64_t>(1, m->grp_cap / (wgs * n_seqs)));
        a.part = m->grp_part; a.part_cnt = m->grp_cnt;
        const dim3 grid((unsigned)wgs, n_seqs, z);
        grouped_short_launch(m->stream, a, grid);
        NVL_HIP(hipGetLastError());
    }
}

// ---- feed-forward of a parallel block: m->xn -> m->lmix columns [ko, kd); the experts' results for the join ----
ExpertOut parallel_ffn(nvl_model* m, const LayerRun& r, const MixerW& w, int M) {
    const nvl_layer_config& c = r.c;
    if (r.ffn_in && m->f32) {       // (bf16: the input projection's epilogue has written them)
        const int64_t n = (int64_t)M * r.Fp;
        KScope ks(m, KC_OTHER);
        hipLaunchKernelGGL((relu2_kernel<float>), dim3(cdiv(n, 256)), dim3(256), 0, m->stream, m->lproj + r.ffn_off, m->lproj_ld, (float*)m->lmix, (int64_t)M, r.Fp, (int64_t)r.kd, r.ko);
        NVL_HIP(hipGetLastError());
    } else if (c.ffn_dim && !r.ffn_in && !r.glu_in) {
        m->site = KS_FFN_UP;
        const bool relu2 = r.act == NVL_ACT_RELU2;
        const int N = relu2 ? r.Fp : 2 * r.Fp;
        if (m->f32) {
            gemm(m, EPI_STORE, true, mk(m->xn, m->H, w.w1, m->h2, N, nullptr, 1.f, M, N, m->H));
            const int64_t n = (int64_t)M * r.Fp;
            KScope ks(m, KC_OTHER);
            if (relu2) hipLaunchKernelGGL((relu2_kernel<float>), dim3(cdiv(n, 256)), dim3(256), 0, m->stream, m->h2, (int64_t)N, (float*)m->lmix, (int64_t)M, r.Fp, (int64_t)r.kd, r.ko);
            else hipLaunchKernelGGL((swiglu_kernel<float>), dim3(cdiv(n, 256)), dim3(256), 0, m->stream, m->h2, (float*)m->lmix, (int64_t)M, r.Fp, (int64_t)r.kd, r.ko);
            NVL_HIP(hipGetLastError());
        } else      // (the operand's column blocks are 32 wide: a shift by ko columns is a shift of the base)
            gemm(m, relu2 ? EPI_RELU2 : EPI_SWIGLU, false, mk(m->xn, m->H, w.w1, (bf16_t*)m->lmix + (r.ko >> 5) * 512, r.kd, nullptr, 1.f, M, N, m->H));
    }
    if (!c.experts) return {};
    const int E = c.experts, k = c.top_k, pairs = M * k;
    // decode: all experts as one projection each way with the routing weights as a mask (gemm.h GemmArgs::moe_gate)
    const bool dense = !m->f32 && M <= 64 && r.Ip <= 2048;
    const float* tail = m->lproj + (m->f32 ? r.ffn_off : 0);          // [a small shared expert's gate | up |] router logits
    GroupRouteArgs ra{m->f32 ? m->lproj + r.route_off : tail + (r.glu_in ? 2 * r.Fp : 0), m->lproj_ld, w.route_bias, M, E, k, c.expert_groups, c.groups_kept, m->expert_ids, m->expert_w, dense ? m->moe_gate : nullptr, r.Ep,
                      tail, r.Fp, m->lmix, r.kd, r.ko};
    {
        KScope ks(m, KC_OTHER, 0, KS_MOE_ROUTER, (double)M * ((E + 2.0 * k) * 4.0 + (r.glu_in ? c.ffn_dim * (8.0 + (double)m->wsize) : 0.0)));
        const dim3 grid(cdiv(M, 4), 1 + (r.glu_in ? cdiv(r.Fp, 256) : 0));
        if (m->f32) hipLaunchKernelGGL((moe_route_grouped_kernel<float>), grid, dim3(256), 0, m->stream, ra);
        else hipLaunchKernelGGL((moe_route_grouped_kernel<bf16_t>), grid, dim3(256), 0, m->stream, ra);
        NVL_HIP(hipGetLastError());
    }
    const double touch = (double)std::min(E, pairs);
    if (dense) {
        GemmArgs u = mk(m->xn, m->H, w.moe_up, m->moe_hall, r.Ep * r.Ip, nullptr, 1.f, M, E * 2 * r.Ip, m->H);
        u.moe_gate = m->moe_gate; u.moe_E = r.Ep; u.moe_I = r.Ip;
        m->site = KS_MOE_UP; m->site_bytes = (touch * 2 * c.expert_dim * m->Hn + (double)M * m->Hn + (double)pairs * c.expert_dim) * (double)m->wsize;
        gemm(m, EPI_SWIGLU, false, u, 4.0 * pairs * c.expert_dim * m->Hn);
        GemmArgs d = mk(m->moe_hall, r.Ep * r.Ip, w.moe_cat, m->x, m->H, nullptr, 1.f, M, m->H, r.Ep * r.Ip);      // (K slices: plain stores into moe_part)
        d.moe_gate = m->moe_gate; d.moe_E = r.Ep; d.moe_I = r.Ip; d.sk_part = m->moe_part; d.sk_slices = r.moe_slices;
        m->site = KS_MOE_DOWN; m->site_bytes = (touch * m->Hn * c.expert_dim + (double)pairs * c.expert_dim) * (double)m->wsize + (double)r.moe_slices * M * m->Hn * 4.0;
        gemm(m, EPI_RESID, true, d, 2.0 * pairs * m->Hn * c.expert_dim);
        return {m->moe_part, r.moe_slices, (int64_t)M * m->H, nullptr, nullptr};
    }
    const bool pp = moe_pp_ok(m, r.Ip, false);
    const int BM = pp ? 256 : ((!m->f32 && g_moe_bm == 256) ? 256 : 128);
    moe_sort(m, E, k, M, BM);
    moe_expert_gemms(m, MoeW{E, k, r.Ip, w.moe_up, w.moe_down}, M, BM, pp, false);
    return {m->moe_eo, k, 0, m->slot_of, m->expert_w};
}

// ---- gate and up of a gated feed-forward, m->xn -> m->hbuf (fp32 mode: W [gate rows | up rows], the activation in a launch of its own) ----
void glu_up(nvl_model* m, const void* W, int M, int Fp, int act, float limit) {
    m->site = KS_FFN_UP;
    if (m->f32) {
        gemm(m, EPI_STORE, true, mk(m->xn, m->H, W, m->h2, 2 * Fp, nullptr, 1.f, M, 2 * Fp, m->H));
        const int64_t n = (int64_t)M * Fp;
        KScope ks(m, KC_OTHER);
        if (act == NVL_ACT_CLAMPED_GLU) hipLaunchKernelGGL((clamp_glu_kernel<float>), dim3(cdiv(n, 256)), dim3(256), 0, m->stream, m->h2, (float*)m->hbuf, (int64_t)M, Fp, limit, CLAMPED_GLU_SLOPE);
        else if (act == NVL_ACT_REGLU) hipLaunchKernelGGL((reglu_kernel<float>), dim3(cdiv(n, 256)), dim3(256), 0, m->stream, m->h2, (float*)m->hbuf, (int64_t)M, Fp);
        else hipLaunchKernelGGL((swiglu_kernel<float, true>), dim3(cdiv(n, 256)), dim3(256), 0, m->stream, m->h2, (float*)m->hbuf, (int64_t)M, Fp, (int64_t)Fp, 0);
        NVL_HIP(hipGetLastError());
        return;
    }
    GemmArgs up = mk(m->xn, m->H, W, m->hbuf, Fp, nullptr, 1.f, M, 2 * Fp, m->H);
    up.glu_limit = limit; up.glu_slope = CLAMPED_GLU_SLOPE;
    gemm(m, act == NVL_ACT_CLAMPED_GLU ? EPI_CLAMP_GLU : act == NVL_ACT_REGLU ? EPI_REGLU : EPI_GEGLU, false, up);
}
// ---- experts that read m->xn by themselves, and their shared expert: returns what is added, the rest of it in `ex` ----
SubOut expert_ffn(nvl_model* m, const LayerRun& r, const MixerW& w, int M, ExpertOut& ex) {
    const nvl_layer_config& c = r.c;
    const int E = c.experts, k = c.top_k, pairs = M * k;
    const bool dense = !m->f32 && M <= 64 && r.Ip <= 2048;          // decode: masked projections over all experts (gemm.h GemmArgs::moe_gate)
    const int parts = dense ? r.shared_parts : 0;
    SubOut y{nullptr, 1, 0};
    auto shared = [&] {
        const void* W = r.shared_parts && !m->f32 ? (const void*)((const char*)w.moe_up + (int64_t)E * 2 * r.Ip * m->H * (int64_t)m->wsize) : w.w1;
        glu_up(m, W, M, r.Fp, r.act, c.ffn_limit);
        y = sub_out(m, KS_FFN_DOWN, m->hbuf, w.w2, M, r.Fp);
    };
    if (dense && E <= 64 && c.route_softmax) {
        GemmArgs a = mk(m->xn, m->H, w.router, nullptr, E, w.route_bias, 1.f, M, E, m->H);
        KScope ks(m, KC_OTHER, 2.0 * M * E * m->Hn, KS_MOE_ROUTER, ((double)E * m->Hn + (double)M * m->Hn) * (double)m->wsize + (double)M * E * 4.0);
        hipLaunchKernelGGL(moe_router_gate_kernel, dim3(cdiv(M, 16)), dim3(1024), 0, m->stream, a, k, m->moe_gate, (float*)nullptr, 0, r.Ep, parts);
        NVL_HIP(hipGetLastError());
    } else {
        m->site = KS_MOE_ROUTER;
        gemm(m, EPI_STORE, true, mk(m->xn, m->H, w.router, m->lproj, (int)m->lproj_ld, nullptr, 1.f, M, E, m->H));
        GroupRouteArgs ra{};
        ra.logits = m->lproj; ra.ld = m->lproj_ld; ra.correction = w.route_bias; ra.rows = M; ra.E = E; ra.top = k; ra.groups = c.expert_groups; ra.keep = c.groups_kept;
        ra.ids = m->expert_ids; ra.w = m->expert_w; ra.gate = dense ? m->moe_gate : nullptr; ra.gate_ld = r.Ep; ra.softmax = c.route_softmax; ra.n_always = parts;
        KScope ks(m, KC_OTHER, 0, KS_MOE_ROUTER, (double)M * (E + 2.0 * k) * 4.0);
        hipLaunchKernelGGL((moe_route_grouped_kernel<float>), dim3(cdiv(M, 4)), dim3(256), 0, m->stream, ra);
        NVL_HIP(hipGetLastError());
    }
    if (dense) {
        const double touch = (double)std::min(E, pairs) * c.expert_dim + (parts ? c.ffn_dim : 0), work = (double)pairs * c.expert_dim + (parts ? (double)M * c.ffn_dim : 0.0);
        GemmArgs u = mk(m->xn, m->H, w.moe_up, m->moe_hall, r.Ep * r.Ip, nullptr, 1.f, M, (E + parts) * 2 * r.Ip, m->H);
        u.moe_gate = m->moe_gate; u.moe_E = r.Ep; u.moe_I = r.Ip;
        u.glu_limit = c.expert_limit; u.glu_limit2 = c.ffn_limit; u.glu_from2 = E * r.Ip; u.glu_slope = CLAMPED_GLU_SLOPE;
        m->site = KS_MOE_UP; m->site_bytes = (2 * touch * m->Hn + (double)M * m->Hn + work) * (double)m->wsize;
        gemm(m, c.expert_limit > 0.f ? EPI_CLAMP_GLU : EPI_SWIGLU, false, u, 4.0 * work * m->Hn);
        GemmArgs d = mk(m->moe_hall, r.Ep * r.Ip, w.moe_cat, m->x, m->H, nullptr, 1.f, M, m->H, r.Ep * r.Ip);      // (K slices: plain stores into moe_part)
        d.moe_gate = m->moe_gate; d.moe_E = r.Ep; d.moe_I = r.Ip; d.sk_part = m->moe_part; d.sk_slices = r.moe_slices;
        m->site = KS_MOE_DOWN; m->site_bytes = (touch * m->Hn + work) * (double)m->wsize + (double)r.moe_slices * M * m->Hn * 4.0;
        gemm(m, EPI_RESID, true, d, 2.0 * work * m->Hn);
        if (!c.ffn_dim || parts) return {m->moe_part, r.moe_slices, (int64_t)M * m->H};
        ex = {m->moe_part, r.moe_slices, (int64_t)M * m->H, nullptr, nullptr};
        shared();
        return y;
    }
    const bool pp = moe_pp_ok(m, r.Ip, false);
    const int BM = pp ? 256 : ((!m->f32 && g_moe_bm == 256) ? 256 : 128);
    moe_sort(m, E, k, M, BM);
    moe_expert_gemms(m, MoeW{E, k, r.Ip, w.moe_up, w.moe_down, c.expert_limit}, M, BM, pp, false);
    ex = {m->moe_eo, k, 0, m->slot_of, m->expert_w};
    if (c.ffn_dim) shared();
    else {               // nothing but the experts joins
        y = {m->ly, 1, 0};
        hipLaunchKernelGGL(fill_i32_kernel, dim3(cdiv((int64_t)M * m->H, 256)), dim3(256), 0, m->stream, (int32_t*)m->ly, 0, M * m->H);
        NVL_HIP(hipGetLastError());
    }
    return y;
}

// ---- per-layer token input: x (as m->xn) -> m->ly or its K slices ----
SubOut side_input(nvl_model* m, const MixerW& w, const Meta& md, int li, int M) {
    const int sd = m->cfg.side_dim, kp = m->side_kp;
    const int64_t col = (int64_t)li * round_up(sd, 4);
    const int sd4 = (int)round_up(sd, 4);
    m->site = KS_SIDE_GATE;
    if (m->f32) {
        gemm(m, EPI_STORE, true, mk(m->xn, m->H, w.side_gate, m->h2, sd4, nullptr, 1.f, M, sd, m->H));
        KScope ks(m, KC_OTHER);
        hipLaunchKernelGGL((gelu_token_kernel<float, float>), dim3(M), dim3(256), 0, m->stream, m->h2, (int64_t)sd4, 1, (int64_t)0, (const float*)m->side_emb + col, m->side_ld, md.tokens, (float*)m->lside, (int64_t)kp, sd);
        NVL_HIP(hipGetLastError());
    } else {
        GemmArgs a = mk(m->xn, m->H, w.side_gate, m->lside, kp, nullptr, 1.f, M, sd, m->H);
        // a few hundred rows: the narrow projection has too few tiles for the chip; split along K, the activation in a launch of its own
        int slices = 1;
        const int tiles = cdiv(M, 128) * cdiv(sd, 128);
        if (M > 512 && M <= m->sk_rows && sd4 <= m->H) while (slices < SK_TILE_MAX_SLICES && tiles * slices < 256 && m->H / (slices * 2) >= 256) slices *= 2;
        if (slices > 1) {
            a.C = m->x; a.N = sd4; a.sk_part = m->sk_part; a.sk_slices = slices;      // (x is not touched)
            gemm(m, EPI_RESID, true, a);
            KScope ks(m, KC_OTHER, 0, KS_SIDE_GATE, (double)M * sd * (4.0 * slices + 4.0));
            hipLaunchKernelGGL((gelu_token_kernel<bf16_t, bf16_t>), dim3(M), dim3(256), 0, m->stream, m->sk_part, (int64_t)sd4, slices, (int64_t)M * sd4, (const bf16_t*)m->side_emb + col, m->side_ld, md.tokens, (bf16_t*)m->lside, (int64_t)kp, sd);
            NVL_HIP(hipGetLastError());
        } else {
            a.tok_ids = md.tokens; a.tok_table = (const bf16_t*)m->side_emb + col; a.tok_ld = m->side_ld;
            gemm(m, EPI_GELU_TOK, false, a);
        }
    }
    return sub_out(m, KS_SIDE_PROJ, m->lside, w.side_proj, M, kp);
}

// The layers of one pass.  have_xn: m->xn already holds the first norm (decode seam).  all_rows: the logits of every row are wanted,
// in order: the last sandwich norm then leaves the final norm of every row in m->xn; returns whether it did.
bool layered_stack(nvl_model* m, const Meta& md, int n_seqs, int M, int max_len, bool have_xn, bool all_rows) {
    auto W = [&](int li) -> const MixerW& { return m->mixers[(size_t)m->runs[(size_t)li].owner]; };
    const bool sum = m->cfg.block_style == NVL_BLOCK_SUM_NORM, post = sum || m->cfg.block_style == NVL_BLOCK_POST;        // post: sublayers read x itself
    const bool shift = m->cfg.token_shift != 0, ones = max_len == 1;       // ones: token shift in the launch that makes x, else in one of its own
    const bool par = m->cfg.block_style == NVL_BLOCK_PARALLEL;
    m->key_src = m->key_win = -1;
    auto shift_out = [&](int li) { return shift && ones && li < m->L ? ShiftOut{W(li).shift, m->rec_state + m->runs[(size_t)li].shift_off, &md} : ShiftOut{}; };
    auto shift_rows = [&](int li) {          // x -> m->xn, the shifted input of layer li's mixer
        ShiftArgs a{m->x, W(li).shift, m->lshift + (int64_t)li * m->opts.max_seqs * m->H, m->rec_state + m->runs[(size_t)li].shift_off, m->rec_slot_stride,
                    md.tok_seq, md.tok_pos, md.seq_tok_start, md.seq_len, md.seq_pos, md.seq_slot, M, m->H};
        KScope ks(m, KC_OTHER, 0, KS_SHIFT, (double)M * m->Hn * (4.0 + (double)m->wsize));
        if (m->f32) hipLaunchKernelGGL((token_shift_kernel<float>), dim3(M), dim3(256), 0, m->stream, a, (float*)m->xn);
        else hipLaunchKernelGGL((token_shift_kernel<bf16_t>), dim3(cdiv(M, 16)), dim3(std::min(1024, m->H * 2)), 0, m->stream, a, (bf16_t*)m->xn);
        NVL_HIP(hipGetLastError());
    };
    if (shift && !ones) {
        KScope ks(m, KC_OTHER, 0, KS_SHIFT);
        hipLaunchKernelGGL(shift_copy_kernel, dim3(n_seqs, m->L), dim3(256), 0, m->stream, m->rec_state, m->rec_slot_stride, m->shift_offs, md.seq_slot, m->lshift, m->opts.max_seqs, m->H);
        NVL_HIP(hipGetLastError());
    }
    if (!have_xn && shift && !ones) shift_rows(0);
    else if (!have_xn) sandwich(m, SubOut{}, nullptr, {W(0).norm1, W(0).norm1_bias, post}, m->xn, M, nullptr, {}, shift_out(0));
    for (int li = 0; li < m->L; li++) {
        const LayerRun& r = m->runs[(size_t)li];
        const MixerW& w = W(li);
        NextNorm after{nullptr, nullptr, post};                    // the norm that follows this layer
        if (li + 1 < m->L) { after.w = W(li + 1).norm1; after.b = W(li + 1).norm1_bias; }
        else if (all_rows) { after.w = m->final_norm; after.b = m->final_norm_b; }
        switch (r.c.mixer) {
            case NVL_MIXER_LATENT_ATTENTION: mix_latent(m, r, w, md, n_seqs, M, max_len); break;
            case NVL_MIXER_MAMBA2: mix_mamba2(m, r, w, md, n_seqs, M, max_len); break;
            case NVL_MIXER_CHANNEL_DELTA: mix_delta(m, r, w, md, n_seqs, M, max_len); break;
            case NVL_MIXER_ATTENTION: mix_grouped(m, r, w, md, n_seqs, M, max_len); break;
            default: mix_gla(m, r, w, md, n_seqs, M, max_len);
        }
        if (par) {
            const ExpertOut ex = parallel_ffn(m, r, w, M);
            const SubOut y = sub_out(m, KS_OPROJ, m->lmix, w.o, M, r.kd);
            if (m->cfg.side_dim) {
                sandwich(m, y, nullptr, {nullptr, nullptr, true}, m->xn, M, nullptr, ex);
                sandwich(m, side_input(m, w, md, li, M), w.side_norm, after, m->xn, M);
            } else sandwich(m, y, nullptr, after, m->xn, M, nullptr, ex);
            tap_layer(m, li, M);
            continue;
        }
        SubOut y = sub_out(m, KS_OPROJ, m->lmix, w.o, M, r.kd);
        if (sum || shift) {
            const bool apart = shift && !ones && li + 1 < m->L, ff = r.c.ffn_dim || r.c.experts;      // apart: the next mixer's input comes from shift_rows
            const NextNorm own{nullptr, nullptr, true}, close = apart ? NextNorm{nullptr, nullptr, false} : after;
            sandwich(m, y, w.norm1b, ff ? own : close, m->xn, M, nullptr, {}, ff ? ShiftOut{} : shift_out(li + 1));
            if (ff) {
                ExpertOut ex;
                if (r.c.experts) y = expert_ffn(m, r, w, M, ex);
                else { glu_up(m, w.w1, M, r.Fp, r.act, r.c.ffn_limit); y = sub_out(m, KS_FFN_DOWN, m->hbuf, w.w2, M, r.Fp); }
                sandwich(m, y, w.norm2b, close, m->xn, M, nullptr, ex, shift_out(li + 1));
            }
            if (apart) shift_rows(li + 1);
            tap_layer(m, li, M);
            continue;
        }
        sandwich(m, y, w.norm1b, r.c.ffn_dim ? NextNorm{w.norm2, nullptr, post} : after, m->xn, M);
        if (r.c.ffn_dim) {
            glu_up(m, w.w1, M, r.Fp, m->cfg.activation_type, r.c.ffn_limit);
            y = sub_out(m, KS_FFN_DOWN, m->hbuf, w.w2, M, r.Fp);
            sandwich(m, y, w.norm2b, after, m->xn, M);
        }
        tap_layer(m, li, M);
    }
    return all_rows;
}

}  // namespace
