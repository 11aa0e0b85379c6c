// linrec.h — gated linear recurrences with a matrix state per head, in fp32 throughout:
//     S_t = diag(alpha_t) S_{t-1} + k_t v_t^T        S [DK][DV], alpha_t in (0, 1]
//     o_t = S_t^T q_t
// Three designs of the family run on the same kernels:
//   per-channel decay (gated linear attention): alpha = sigmoid(z)^(1/tau), z = A2 (A1 h) + b per key channel;
//   one decay per head (Mamba-2, state-space duality): q = C, k = dt B, v = x, alpha = exp(-exp(A_log) dt), o += D x; a group
//     of heads shares q and k;
//   one fixed decay per head (lightning attention): alpha given, dt = 1, D = 0.
//
//   linrec_step_kernel   token by token, the state streamed once per token (decode; the convolution of a Mamba-2 decode token,
//                        and GLA's head norm + output gate, are fused in)
//   linrec_chunk_kernel  32 tokens per step on v_mfma_f32_16x16x4_f32 (prefill).  With b_t = the inclusive sum of log alpha
//                        inside the chunk and S_in the state that enters it:
//                            o_t   = (q_t e^{b_t}) S_in + sum_{s<=t} A[t][s] v_s,   A[t][s] = sum_c q_t[c] k_s[c] e^{b_t[c] - b_s[c]}
//                            S_out = diag(e^{b_end}) S_in + sum_s (k_s e^{b_end - b_s}) v_s^T
//                        Every exponent that is evaluated is <= 0: a per-channel decay cannot be split into e^{b_t} e^{-b_s}
//                        (the second factor overflows for strong decays), so the 16 x 16 diagonal blocks of A are summed pair by
//                        pair and the block below the diagonal takes the boundary between the two halves as its reference.
//                        The products stay in fp32 (no bf16 operands): state, decays and what they scale are 32-bit quantities.
//
// Sequences: token t0 .. t0 + n of the batch belong to sequence `seq`; its state lives in slot seq_slot[seq]; a sequence whose
// first token of this call has position 0 starts from a zero state whatever the slot holds.
#pragma once
#include "common.h"

namespace nvl {

struct LinRecArgs {
    int H, DK, DV, DVp, kdiv;          // DVp: row pitch of the state (DV padded to 4); kdiv: heads that share one q / k vector
    const float *q, *k, *v;            // head 0's first column; row pitch ld
    int64_t ld;
    float q_scale;
    // one decay per head
    const float* dt; int64_t dt_ld;    // raw step sizes (before bias and softplus), one column per head
    const float *dt_bias, *a_log, *Dskip;
    const float *decay, *log2_decay;   // not NULL: fixed decays instead, and their base-2 logarithms
    // a decay per key channel
    const float* a1; int64_t a1_ld;    // [token][rank]
    int rank;
    const float *a2, *a2_b;            // [H * DK][rank], [H * DK]
    float inv_tau;
    float* o; int64_t o_ld;            // [token][H * DV]
    float* state; int64_t slot_stride; // slot s: state + s * slot_stride, [H][DK][DVp]
    const int32_t *seq_tok_start, *seq_len, *seq_pos, *seq_slot;
    int vec4;                          // q, k and v rows may be read 16 bytes at a time
    int len_lo, len_hi;                // sequences with len_lo <= tokens of this call <= len_hi are served, the others skipped
    // chunk-parallel prefill: `super` tokens per workgroup, scratch [seq][n_super][H][DK * DVp] and decays [..][H][DK or 1]
    float *z, *zdecay; int super, n_super, n_slices;
    // fused decode epilogue of a per-channel recurrence: out = rms(o) * norm_w * silu(gate)
    const float* gate; int64_t gate_ld; const float* norm_w; float eps; void* out; int64_t out_ld;
    // fused convolution of a one-token Mamba-2 step: raw [x | B | C] columns, a ring of the last `taps` raw rows per slot
    const float* raw; int64_t raw_ld;
    const float *conv_w, *conv_b; int taps, conv_dim;
    float* ring; int64_t ring_slot_stride;
};

__device__ __forceinline__ float lr_silu(float x) { return x / (1.0f + expf(-x)); }
__device__ __forceinline__ float lr_sigmoid(float x) { return 1.0f / (1.0f + expf(-x)); }
__device__ __forceinline__ float lr_softplus(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }

// ------------------------------------------------------------------------------------------
// token by token.  grid (H, sequences), 512 threads: tv threads side by side on a state row (4 columns each), 512 / tv rows at
// a time.  KIND bit 0: per-channel decay; bit 1: fused (conv in front of / norm + gate behind the recurrence).
// ------------------------------------------------------------------------------------------
constexpr int LR_STEP_THREADS = 512;
static inline int linrec_step_lds_bytes(int DK, int DVp) {
    int tv = 1;
    while (tv < DVp / 4) tv <<= 1;
    return 4 * (3 * ((DK + 3) & ~3) + DVp + LR_STEP_THREADS / tv * DVp);
}
template <int KIND, int LR_STEP_ROWS, typename ActT>      // LR_STEP_ROWS: state rows a thread keeps in registers
__global__ __launch_bounds__(LR_STEP_THREADS, LR_STEP_ROWS <= 8 ? 4 : 2) void linrec_step_kernel(LinRecArgs p) {
    constexpr bool CH = KIND & 1, FUSED = KIND & 2;
    constexpr int NT = LR_STEP_THREADS;
    const int h = blockIdx.x, seq = blockIdx.y, tid = threadIdx.x;
    const int n = p.seq_len[seq];
    if (n < p.len_lo || n > p.len_hi) return;
    extern __shared__ __attribute__((aligned(16))) float lr_sm[];
    const int DK4 = (p.DK + 3) & ~3;
    float* sq = lr_sm;                   // [DK]
    float* sk = sq + DK4;                // [DK]
    float* sa = sk + DK4;                // [DK]   decay (CH)
    float* sv = sa + DK4;                // [DVp]
    float* red = sv + p.DVp;             // [waves or groups of rows][DVp]
    __shared__ float s_red[NT / 64], s_sc[2];
    const int nv4 = p.DVp >> 2;
    int tv = 1;
    while (tv < nv4) tv <<= 1;           // host: nv4 <= NT
    const int rg = tid / tv, tc = tid - rg * tv, RG = NT / tv;
    const int NRED = tv >= 64 ? RG : NT / 64;
    const bool live = tc < nv4;
    const int t0 = p.seq_tok_start[seq], pos0 = p.seq_pos[seq], slot = p.seq_slot[seq];
    float* st = p.state + (int64_t)slot * p.slot_stride + (int64_t)h * p.DK * p.DVp;
    int so = rg * p.DVp + 4 * tc;        // this thread's place in a pass of RG rows
    const int pass = RG * p.DVp;
    const int g = h / p.kdiv;
    f32x4 s[LR_STEP_ROWS];               // the first LR_STEP_ROWS rows of this thread, fetched before anything else is known
#pragma unroll
    for (int i = 0; i < LR_STEP_ROWS; i++) {
        const int row = rg + i * RG;
        const bool ok = live && row < p.DK;                     // (no branches around s: it stays in registers)
        const f32x4 x = *(const f32x4*)(st + (ok ? i * pass + so : 0));
#pragma unroll
        for (int r = 0; r < 4; r++) s[i][r] = ok && pos0 > 0 ? x[r] : 0.f;
    }
    asm volatile("" : "+v"(so));            // (or the addresses of these loads are kept in registers for the stores)
    for (int i = tid; i < p.DVp; i += NT) sv[i] = 0.f;
    __syncthreads();
    for (int it = 0; it < n; it++) {
        const int64_t t = t0 + it;
        if constexpr (!CH) {
            if (p.decay) {
                if (tid == 0) { s_sc[0] = 1.0f; s_sc[1] = p.decay[h]; }
            } else if (tid == 0) {
                const float d = lr_softplus(p.dt[t * p.dt_ld + h] + p.dt_bias[h]);
                s_sc[0] = d;
                s_sc[1] = expf(-expf(p.a_log[h]) * d);
            }
        }
        if constexpr (!CH && FUSED) {
            // causal convolution + silu of this head's channels (n == 1): x of the head, B and C of its group
            const int inner = p.H * p.DV, GN = (p.H / p.kdiv) * p.DK;
            const float* rw = p.raw + t * p.raw_ld;
            float* ring = p.ring + (int64_t)slot * p.ring_slot_stride;
            for (int i = tid; i < p.DV + 2 * p.DK; i += NT) {
                const int c = i < p.DV ? h * p.DV + i : (i < p.DV + p.DK ? inner + g * p.DK + i - p.DV : inner + GN + g * p.DK + i - p.DV - p.DK);
                const float cur = rw[c];
                float acc = p.conv_b[c];
                for (int b = p.taps - 1; b >= 1; b--)
                    if (pos0 - b >= 0) acc = fmaf(ring[(int64_t)((pos0 - b) % p.taps) * p.conv_dim + c], p.conv_w[(int64_t)c * p.taps + p.taps - 1 - b], acc);
                acc = fmaf(cur, p.conv_w[(int64_t)c * p.taps + p.taps - 1], acc);
                ring[(int64_t)(pos0 % p.taps) * p.conv_dim + c] = cur;      // (heads of a group write the same values; nobody reads this row now)
                const float y = lr_silu(acc);
                if (i < p.DV) sv[i] = y;
                else if (i < p.DV + p.DK) sk[i - p.DV] = y;
                else sq[i - p.DV - p.DK] = y;
            }
        } else {
            for (int i = tid; i < p.DK; i += NT) {
                sq[i] = p.q[t * p.ld + (int64_t)g * p.DK + i] * p.q_scale;
                sk[i] = p.k[t * p.ld + (int64_t)g * p.DK + i];
                if constexpr (CH) {
                    float z = p.a2_b[h * p.DK + i];
                    const float* w = p.a2 + (int64_t)(h * p.DK + i) * p.rank;
                    const float* a = p.a1 + t * p.a1_ld;
                    for (int j = 0; j < p.rank; j++) z = fmaf(w[j], a[j], z);
                    sa[i] = expf(-lr_softplus(-z) * p.inv_tau);
                }
            }
            for (int i = tid; i < p.DV; i += NT) sv[i] = p.v[t * p.ld + (int64_t)h * p.DV + i];
        }
        __syncthreads();
        f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
        {
            const f32x4 v = *(const f32x4*)(sv + (live ? 4 * tc : 0));
            const float ksc = CH ? 1.f : s_sc[0], al0 = CH ? 1.f : s_sc[1];
#pragma unroll
            for (int i = 0; i < LR_STEP_ROWS; i++) {
                const int row = rg + i * RG;
                const bool ok = live && row < p.DK;
                const int rr = ok ? row : 0;
                const float al = CH ? sa[rr] : al0, kk = ok ? sk[rr] * ksc : 0.f, qq = ok ? sq[rr] : 0.f;
#pragma unroll
                for (int r = 0; r < 4; r++) { s[i][r] = fmaf(al, s[i][r], kk * v[r]); acc[r] = fmaf(qq, s[i][r], acc[r]); }
                if (ok && it == n - 1) *(f32x4*)(st + i * pass + so) = s[i];
            }
#pragma unroll 1
            for (int row = rg + LR_STEP_ROWS * RG; live && row < p.DK; row += RG) {     // (a state larger than the registers: streamed)
                f32x4 w = f32x4{0.f, 0.f, 0.f, 0.f};
                if (pos0 + it > 0) w = *(const f32x4*)(st + (int64_t)row * p.DVp + 4 * tc);
                const float al = CH ? sa[row] : al0, kk = sk[row] * ksc, qq = sq[row];
#pragma unroll
                for (int r = 0; r < 4; r++) { w[r] = fmaf(al, w[r], kk * v[r]); acc[r] = fmaf(qq, w[r], acc[r]); }
                *(f32x4*)(st + (int64_t)row * p.DVp + 4 * tc) = w;
            }
        }
        // row groups of one wave first (tv < 64: 64 / tv of them side by side), then over the waves through LDS
        for (int o = tv; o < 64; o <<= 1)
#pragma unroll
            for (int r = 0; r < 4; r++) acc[r] += __shfl_xor(acc[r], o, 64);
        if (live && (tv >= 64 || (tid & 63) < tv)) *(f32x4*)(red + (int64_t)(tv >= 64 ? rg : tid >> 6) * p.DVp + 4 * tc) = acc;
        __syncthreads();
        // sum over the row groups; one column per thread (DV <= 4 * NT: up to four columns)
        float ov[4], ss = 0.f;
#pragma unroll
        for (int c = 0; c < 4; c++) {
            const int i = tid + c * NT;
            ov[c] = 0.f;
            if (i < p.DV) {
                float a = 0.f;
#pragma unroll 4
                for (int r = 0; r < NRED; r++) a += red[(int64_t)r * p.DVp + i];
                if (!CH && p.Dskip) a = fmaf(p.Dskip[h], sv[i], a);
                ov[c] = a;
                ss = fmaf(a, a, ss);
                if (!(CH && FUSED)) p.o[t * p.o_ld + (int64_t)h * p.DV + i] = a;
            }
        }
        if constexpr (CH && FUSED) {
            ss = wave_sum(ss);
            if ((tid & 63) == 0) s_red[tid >> 6] = ss;
            __syncthreads();
            float tot = 0.f;
#pragma unroll
            for (int i = 0; i < NT / 64; i++) tot += s_red[i];
            const float inv = 1.0f / sqrtf(tot / (float)p.DV + p.eps);
#pragma unroll
            for (int c = 0; c < 4; c++) {
                const int i = tid + c * NT;
                if (i < p.DV) {
                    const float gt = p.gate[t * p.gate_ld + (int64_t)h * p.DV + i];
                    ActIO<ActT>::st((ActT*)p.out + act_index<ActT>(t, (int64_t)h * p.DV + i, p.out_ld), ov[c] * inv * p.norm_w[i] * lr_silu(gt));
                }
            }
        }
        __syncthreads();
    }
}

// ------------------------------------------------------------------------------------------
// 32 tokens at a time on the fp32 matrix cores.  One workgroup of NW waves per (head, sequence, slice of 16 NW value columns);
// wave w owns the 16 columns 16 w .. of the slice and keeps their DK x 16 state in accumulators: the accumulator layout (lane =
// column, four rows 4 (lane / 16) + r) IS the B operand of the product with q, so the state never goes through LDS.
// MFMA k order: operand element i of lane group g stands for k = 16 n + 4 g + i on both sides.
//   MODE 0: walk all chunks of the sequence; MODE 1: the contribution of `super` tokens from a zero state, and their total decay;
//   MODE 2: the outputs of `super` tokens from the state the prefix kernel left for them.
// ------------------------------------------------------------------------------------------
template <int NK, int NW, bool CH>
constexpr int linrec_chunk_lds_bytes(int rank) {
    return 4 * (32 * (NK * 16 + 4) * (CH ? 3 : 2) + 32 * (NW * 16 + 4) + 32 * 36 + (CH ? (NW * 64 / (NK * 16) < 16 ? NW * 64 / (NK * 16) : 16) * NK * 16 : 96) + (CH ? 32 * rank : 0));
}
__device__ __forceinline__ f32x4 mfma_f32(float a, float b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }
__device__ __forceinline__ float ex2(float x) { return __builtin_amdgcn_exp2f(x); }

template <int NK, int NW, bool CH, int MODE>
__global__ __launch_bounds__(NW * 64, NK > 8 ? 1 : (NW == 8 ? 4 : 3)) void linrec_chunk_kernel(LinRecArgs p) {
    constexpr int C = 32, DKP = NK * 16, LQ = DKP + 4, DVS = NW * 16, LV = DVS + 4, LA = C + 4, NT = NW * 64;
    constexpr float LOG2E = 1.4426950408889634f;
    const int h = blockIdx.x, seq = blockIdx.y;
    const int slice = blockIdx.z % p.n_slices, sup = blockIdx.z / p.n_slices;
    const int n = p.seq_len[seq];
    if (n < p.len_lo || n > p.len_hi) return;
    const int c_first = MODE == 0 ? 0 : sup * p.super, c_end = MODE == 0 ? n : min(n, c_first + p.super);
    if (c_first >= n) return;                                    // (uniform: before any barrier)
    extern __shared__ __attribute__((aligned(16))) float lr_sm[];
    float* qs = lr_sm;                                           // [C][LQ]
    float* ks = qs + C * LQ;                                     // [C][LQ]
    float* bs = ks + C * LQ;                                     // CH: [C][LQ] inclusive sums of log2 alpha
    float* vs = bs + (CH ? C * LQ : 0);                          // [C][LV]
    float* As = vs + C * LV;                                     // [C][LA]
    float* aux = As + C * LA;                                    // CH: [groups][DKP] partial sums; else b[32] | dt[32] | w[32]
    constexpr int NG = NT / DKP < 16 ? NT / DKP : 16, TPG = C / NG;      // CH: groups of threads that share the tokens of a channel
    float* a1s = aux + (CH ? NG * DKP : 96);                     // CH: [C][rank]
    const int tid = threadIdx.x, lane = tid & 63;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int fr = lane & 15, fg = lane >> 4;
    const int t0 = p.seq_tok_start[seq], g = h / p.kdiv;
    const int v0 = slice * DVS, vcol = v0 + 16 * wave + fr;
    const bool fresh = p.seq_pos[seq] == 0;
    float* st = p.state + (int64_t)p.seq_slot[seq] * p.slot_stride + (int64_t)h * p.DK * p.DVp;
    float* zs = MODE != 0 ? p.z + (((int64_t)seq * p.n_super + sup) * p.H + h) * ((int64_t)p.DK * p.DVp) : nullptr;
    const bool vlive = vcol < p.DVp;
    const int so = 4 * fg * p.DVp + vcol;                        // this lane's place in a 16-row block of the state
    f32x4 S[NK];
#pragma unroll
    for (int i = 0; i < NK; i++)
#pragma unroll
        for (int r = 0; r < 4; r++) {
            const int row = 16 * i + 4 * fg + r;
            S[i][r] = 0.f;
            if (MODE != 1 && row < p.DK && vlive && (MODE == 2 || !fresh)) S[i][r] = ((MODE == 2 ? zs : st) + (16 * i + r) * p.DVp)[so];
        }
    for (int i = tid; i < C * LA; i += NT) As[i] = 0.f;          // (the blocks above the diagonal stay zero)
    float btot = 0.f;                                            // MODE 1: log2 of the decay over all chunks (one channel per thread)
    const float A = CH ? 0.f : (p.decay ? p.log2_decay[h] : -expf(p.a_log[h])), Dh = CH || !p.Dskip ? 0.f : p.Dskip[h];
    // the next chunk's rows are fetched into registers while the current one is worked on
    constexpr int RQ = NT / (DKP / 4), RV = NT / (DVS / 4), NQ = (C + RQ - 1) / RQ, NV = (C + RV - 1) / RV, NA1 = 2;      // rows per pass, passes
    const int tq = tid / (DKP / 4), dq = tid % (DKP / 4) * 4, tv_ = tid / (DVS / 4), dv_ = tid % (DVS / 4) * 4;
    f32x4 rq[NQ], rk[NQ], rv[NV];
    float ra[NA1], rdt = 0.f;
    const int ld = (int)p.ld;
    auto ld4 = [&](const float* src, int off, int d, int lim) {
        f32x4 x = f32x4{0.f, 0.f, 0.f, 0.f};
        if (p.vec4) { if (d < lim) x = *(const f32x4*)(src + off); }
        else {
#pragma unroll
            for (int r = 0; r < 4; r++) if (d + r < lim) x[r] = src[off + r];
        }
        return x;
    };
    auto fetch = [&](int c0) {
        const int nv = min(C, c_end - c0);
        const int64_t tb = (int64_t)t0 + c0;
        const float *qb = p.q + tb * ld + (int64_t)g * p.DK, *kb = p.k + tb * ld + (int64_t)g * p.DK, *vb = p.v + tb * ld + (int64_t)h * p.DV + v0;
#pragma unroll
        for (int i = 0; i < NQ; i++) {
            const bool ok = tq + i * RQ < nv;
            const int off = (tq + i * RQ) * ld + dq;
            if (MODE != 1) rq[i] = ok ? ld4(qb, off, dq, p.DK) : f32x4{0.f, 0.f, 0.f, 0.f};
            rk[i] = ok ? ld4(kb, off, dq, p.DK) : f32x4{0.f, 0.f, 0.f, 0.f};
        }
#pragma unroll
        for (int i = 0; i < NV; i++)
            rv[i] = tv_ + i * RV < nv ? ld4(vb, (tv_ + i * RV) * ld + dv_, v0 + dv_, p.DV) : f32x4{0.f, 0.f, 0.f, 0.f};
        if constexpr (CH) {
#pragma unroll
            for (int i = 0; i < NA1; i++) {
                const int e = tid + i * NT, t = e / p.rank;
                ra[i] = t < nv ? p.a1[(tb + t) * p.a1_ld + (e - t * p.rank)] : 0.f;      // (t < nv <= 32: inside the chunk)
            }
        } else if (!p.decay && tid < nv) rdt = p.dt[(tb + tid) * p.dt_ld + h];
    };
    fetch(c_first);

    for (int c0 = c_first; c0 < c_end; c0 += C) {
        const int nv = min(C, c_end - c0);
        const int64_t tb = (int64_t)t0 + c0;
        __syncthreads();                                         // the previous chunk's readers are done
#pragma unroll
        for (int i = 0; i < NQ; i++)
            if (tq + i * RQ < C) {
                if (MODE != 1) *(f32x4*)(qs + (tq + i * RQ) * LQ + dq) = rq[i] * p.q_scale;
                *(f32x4*)(ks + (tq + i * RQ) * LQ + dq) = rk[i];
            }
#pragma unroll
        for (int i = 0; i < NV; i++) if (tv_ + i * RV < C) *(f32x4*)(vs + (tv_ + i * RV) * LV + dv_) = rv[i];
        const float dt_raw = rdt;
        if constexpr (CH) {
#pragma unroll
            for (int i = 0; i < NA1; i++) { const int e = tid + i * NT; if (e < C * p.rank) a1s[e] = ra[i]; }
            for (int e = tid + NA1 * NT; e < C * p.rank; e += NT) {
                const int t = e / p.rank;
                a1s[e] = t < nv ? p.a1[(tb + t) * p.a1_ld + (e - t * p.rank)] : 0.f;
            }
        }
        if (c0 + C < c_end) fetch(c0 + C);
        if constexpr (CH) {
            __syncthreads();
            const int d = tid % DKP, grp = tid / DKP;
            float pre[TPG];
            if (grp < NG) {
#pragma unroll
                for (int j = 0; j < TPG; j++) pre[j] = 0.f;
                if (d < p.DK) {
                    const float bias = p.a2_b[h * p.DK + d];
                    const float* w = p.a2 + (int64_t)(h * p.DK + d) * p.rank;
#pragma unroll
                    for (int j = 0; j < TPG; j++) pre[j] = bias;
#pragma unroll 2
                    for (int e = 0; e < p.rank; e++) {
                        const float we = w[e];
#pragma unroll
                        for (int j = 0; j < TPG; j++) pre[j] = fmaf(we, a1s[(grp * TPG + j) * p.rank + e], pre[j]);
                    }
#pragma unroll
                    for (int j = 0; j < TPG; j++) pre[j] = grp * TPG + j < nv ? -lr_softplus(-pre[j]) * p.inv_tau * LOG2E : 0.f;
#pragma unroll
                    for (int j = 1; j < TPG; j++) pre[j] += pre[j - 1];
                }
                aux[grp * DKP + d] = pre[TPG - 1];
            }
            __syncthreads();
            if (grp < NG) {
                float off = 0.f;
                for (int j = 0; j < grp; j++) off += aux[j * DKP + d];
#pragma unroll
                for (int j = 0; j < TPG; j++) bs[(grp * TPG + j) * LQ + d] = off + pre[j];
            }
        } else if (wave == 0 && lane < 32) {
            const float dt = lane < nv ? (p.decay ? 1.0f : lr_softplus(dt_raw + p.dt_bias[h])) : 0.f;
            float s = p.decay ? A * dt : A * dt * LOG2E;
#pragma unroll
            for (int o = 1; o < 32; o <<= 1) { const float v = __shfl_up(s, o, 32); if (lane >= o) s += v; }
            aux[lane] = s; aux[32 + lane] = dt;
            aux[64 + lane] = ex2(__shfl(s, 31, 32) - s) * dt;
        }
        __syncthreads();
        // ---- A[t][s], s <= t ----
        if constexpr (MODE != 1) {
            if constexpr (CH) {
                for (int pid = tid; pid < 272; pid += NT) {      // the two 16 x 16 diagonal blocks, pair by pair
                    const int half = pid >= 136, x = pid - 136 * half;
                    int t = (int)((sqrtf(8.f * (float)x + 1.f) - 1.f) * 0.5f);
                    if ((t + 1) * (t + 2) / 2 <= x) t++;
                    if (t * (t + 1) / 2 > x) t--;
                    const int s = x - t * (t + 1) / 2;
                    const int tr = (16 * half + t) * LQ, sr = (16 * half + s) * LQ;
                    f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 2
                    for (int d = 0; d < DKP; d += 4) {
                        const f32x4 q4 = *(const f32x4*)(qs + tr + d), k4 = *(const f32x4*)(ks + sr + d);
                        const f32x4 bt = *(const f32x4*)(bs + tr + d), b2 = *(const f32x4*)(bs + sr + d);
#pragma unroll
                        for (int r = 0; r < 4; r++) acc[r] = fmaf(q4[r] * ex2(bt[r] - b2[r]), k4[r], acc[r]);
                    }
                    As[(16 * half + t) * LA + 16 * half + s] = (acc[0] + acc[1]) + (acc[2] + acc[3]);
                }
                if (wave == NW - 1) {                            // tokens 16..31 against 0..15, token 15's sums as the reference
                    f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 2
                    for (int i = 0; i < NK; i++) {
                        const int c = 16 * i + 4 * fg;
                        const f32x4 ref = *(const f32x4*)(bs + 15 * LQ + c);
                        f32x4 a = *(const f32x4*)(qs + (16 + fr) * LQ + c), b = *(const f32x4*)(ks + fr * LQ + c);
                        const f32x4 ba = *(const f32x4*)(bs + (16 + fr) * LQ + c), bb = *(const f32x4*)(bs + fr * LQ + c);
#pragma unroll
                        for (int r = 0; r < 4; r++) acc = mfma_f32(a[r] * ex2(ba[r] - ref[r]), b[r] * ex2(ref[r] - bb[r]), acc);
                    }
#pragma unroll
                    for (int r = 0; r < 4; r++) As[(16 + 4 * fg + r) * LA + fr] = acc[r];
                }
            } else if (wave < 3) {
                const int tt = wave > 0, sb = wave == 2;
                f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 2
                for (int i = 0; i < NK; i++) {
                    const f32x4 a = *(const f32x4*)(qs + (16 * tt + fr) * LQ + 16 * i + 4 * fg), b = *(const f32x4*)(ks + (16 * sb + fr) * LQ + 16 * i + 4 * fg);
#pragma unroll
                    for (int r = 0; r < 4; r++) acc = mfma_f32(a[r], b[r], acc);
                }
                const int s = 16 * sb + fr;
#pragma unroll
                for (int r = 0; r < 4; r++) {
                    const int t = 16 * tt + 4 * fg + r;
                    As[t * LA + s] = s <= t ? acc[r] * (ex2(aux[t] - aux[s]) * aux[32 + s]) : 0.f;
                }
            }
            __syncthreads();
        }
        if constexpr (CH) {                                      // q e^{b}, k e^{b_end - b} in place
#pragma unroll 4
            for (int i = tid; i < C * DKP; i += NT) {
                const int t = i / DKP, d = i % DKP;
                const float b = bs[t * LQ + d];
                if (MODE != 1) qs[t * LQ + d] *= ex2(b);
                ks[t * LQ + d] *= ex2(bs[31 * LQ + d] - b);
            }
            __syncthreads();
        }
        float vf[2][4];
#pragma unroll
        for (int sb = 0; sb < 2; sb++)
#pragma unroll
            for (int r = 0; r < 4; r++) vf[sb][r] = vs[(16 * sb + 4 * fg + r) * LV + 16 * wave + fr];
        if constexpr (MODE != 1) {
            float* ob = p.o + tb * p.o_ld + (int64_t)h * p.DV;
            const int old = (int)p.o_ld;
#pragma unroll
            for (int tt = 0; tt < 2; tt++) {
                f32x4 y = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int i = 0; i < NK; i++) {
                    const f32x4 a = *(const f32x4*)(qs + (16 * tt + fr) * LQ + 16 * i + 4 * fg);
#pragma unroll
                    for (int r = 0; r < 4; r++) y = mfma_f32(a[r], S[i][r], y);
                }
                if constexpr (!CH) {
#pragma unroll
                    for (int r = 0; r < 4; r++) y[r] *= ex2(aux[16 * tt + 4 * fg + r]);
                }
#pragma unroll
                for (int sb = 0; sb <= tt; sb++) {
                    const f32x4 a = *(const f32x4*)(As + (16 * tt + fr) * LA + 16 * sb + 4 * fg);
#pragma unroll
                    for (int r = 0; r < 4; r++) y = mfma_f32(a[r], vf[sb][r], y);
                }
#pragma unroll
                for (int r = 0; r < 4; r++) {
                    const int t = 16 * tt + 4 * fg + r;
                    if (t < nv && vcol < p.DV) ob[t * old + vcol] = CH ? y[r] : fmaf(Dh, vf[tt][r], y[r]);
                }
            }
        }
        if (MODE != 2 || c0 + C < c_end) {                       // (MODE 2: nobody reads the state after the last chunk)
            if constexpr (!CH) {
#pragma unroll
                for (int sb = 0; sb < 2; sb++)
#pragma unroll
                    for (int r = 0; r < 4; r++) vf[sb][r] *= aux[64 + 16 * sb + 4 * fg + r];
                const float e = ex2(aux[31]);
#pragma unroll
                for (int i = 0; i < NK; i++) S[i] *= e;
            }
#pragma unroll
            for (int i = 0; i < NK; i++) {
                if constexpr (CH) {
                    const f32x4 b = *(const f32x4*)(bs + 31 * LQ + 16 * i + 4 * fg);
#pragma unroll
                    for (int r = 0; r < 4; r++) S[i][r] *= ex2(b[r]);
                }
#pragma unroll
                for (int sb = 0; sb < 2; sb++)
#pragma unroll
                    for (int r = 0; r < 4; r++) S[i] = mfma_f32(ks[(16 * sb + 4 * fg + r) * LQ + 16 * i + fr], vf[sb][r], S[i]);
            }
            if (MODE == 1 && tid < (CH ? DKP : 1)) btot += CH ? bs[31 * LQ + tid] : aux[31];
        }
    }
    if (MODE == 2) return;
    float* dst = MODE == 1 ? zs : st;
    int so_end = so;
    asm volatile("" : "+v"(so_end));                          // (or the addresses of the first loads are kept in registers all along)
#pragma unroll
    for (int i = 0; i < NK; i++)
#pragma unroll
        for (int r = 0; r < 4; r++) {
            const int row = 16 * i + 4 * fg + r;
            if (row < p.DK && vlive) (dst + (16 * i + r) * p.DVp)[so_end] = S[i][r];
        }
    if (MODE == 1 && slice == 0) {
        if (CH) { if (tid < p.DK) p.zdecay[(((int64_t)seq * p.n_super + sup) * p.H + h) * p.DK + tid] = ex2(btot); }
        else if (tid == 0) p.zdecay[((int64_t)seq * p.n_super + sup) * p.H + h] = ex2(btot);
    }
}

// MODE 1 -> MODE 2: S_{c+1} = decay_c S_c + Z_c over the `super`-token pieces of a sequence; leaves the state that enters piece c in
// the piece's scratch slot and the final state in the sequence's slot.  grid (H, sequences, state elements / 1024).
template <bool CH>
__global__ __launch_bounds__(256) void linrec_prefix_kernel(LinRecArgs p) {
    const int h = blockIdx.x, seq = blockIdx.y;
    const int elems = p.DK * p.DVp, e = (blockIdx.z * 256 + threadIdx.x) * 4;
    const int n = p.seq_len[seq];
    if (e >= elems || n < p.len_lo || n > p.len_hi) return;
    const int nc = (n + p.super - 1) / p.super, row = e / p.DVp;
    float* st = p.state + (int64_t)p.seq_slot[seq] * p.slot_stride + (int64_t)h * elems + e;
    f32x4 run = p.seq_pos[seq] == 0 ? f32x4{0.f, 0.f, 0.f, 0.f} : *(const f32x4*)st;
    for (int c = 0; c < nc; c++) {
        const int64_t at = ((int64_t)seq * p.n_super + c) * p.H + h;
        float* zp = p.z + at * elems + e;
        const f32x4 z = *(const f32x4*)zp;
        const float d = CH ? p.zdecay[at * p.DK + row] : p.zdecay[at];
        *(f32x4*)zp = run;
        run = d * run + z;
    }
    *(f32x4*)st = run;
}

// ------------------------------------------------------------------------------------------
// Causal convolution per channel + bias + silu over a batch whose raw rows [x | B | C] sit in `raw`; positions before this call come
// from the slot's ring (row = position mod taps).  conv_ring_kernel then records the newest rows (its own
// launch: a ring row may still be read by a token of the same call).
// ------------------------------------------------------------------------------------------
struct ConvArgs {
    const float* raw; int64_t raw_ld;
    const float *w, *b; int taps, channels;
    float* out; int64_t out_ld;
    float* ring; int64_t ring_slot_stride;
    const int32_t *tok_seq, *tok_pos, *seq_tok_start, *seq_len, *seq_pos, *seq_slot;
};
constexpr int CONV_TOKENS = 8;       // tokens per workgroup: the rows they share are fetched once
__device__ __forceinline__ float conv_at(const ConvArgs& p, const float* ring, int t, int pos, int first, int c) {
    float acc = p.b[c];
    for (int b = p.taps - 1; b >= 0; b--) {
        if (pos - b < 0) continue;
        const float v = pos - b >= first ? p.raw[(int64_t)(t - b) * p.raw_ld + c] : ring[(int64_t)((pos - b) % p.taps) * p.channels + c];
        acc = fmaf(v, p.w[(int64_t)c * p.taps + p.taps - 1 - b], acc);
    }
    return lr_silu(acc);
}
// grid (ceil(tokens / 8), ceil(channels / 1024)), 4 channels per thread.  TAPS > 0 (channel count, row pitch and base multiples of 4):
// a tile that lies inside one sequence runs from registers.
template <int TAPS>
__global__ __launch_bounds__(256) void conv_silu_kernel(ConvArgs p, int n_tok) {
    const int c = (blockIdx.y * 256 + threadIdx.x) * 4;
    if (c >= p.channels) return;
    const int t0 = blockIdx.x * CONV_TOKENS, t1 = min(n_tok, t0 + CONV_TOKENS);
    if constexpr (TAPS > 0) {
        const int seq = p.tok_seq[t0], first = p.seq_pos[seq];
        if (p.tok_seq[t1 - 1] == seq) {
            const int pos0 = p.tok_pos[t0] - (TAPS - 1);             // position of r[0]
            const float* x = p.raw + (int64_t)t0 * p.raw_ld + c;
            const float* ring = p.ring + (int64_t)p.seq_slot[seq] * p.ring_slot_stride + c;
            f32x4 r[CONV_TOKENS + TAPS - 1], w[TAPS];
#pragma unroll
            for (int i = 0; i < CONV_TOKENS + TAPS - 1; i++) {
                r[i] = f32x4{0.f, 0.f, 0.f, 0.f};
                if (i < TAPS - 1 && pos0 + i < first) {              // (uniform) before this call: zeros before the sequence, else the ring
                    if (pos0 + i >= 0) r[i] = *(const f32x4*)(ring + (int64_t)((pos0 + i) % TAPS) * p.channels);
                } else if (t0 + i - (TAPS - 1) < t1) {
                    r[i] = *(const f32x4*)(x + (int64_t)(i - (TAPS - 1)) * p.raw_ld);
                }
            }
#pragma unroll
            for (int k = 0; k < TAPS; k++)
#pragma unroll
                for (int e = 0; e < 4; e++) w[k][e] = p.w[(int64_t)(c + e) * TAPS + k];
            const f32x4 bias = *(const f32x4*)(p.b + c);
#pragma unroll
            for (int i = 0; i < CONV_TOKENS; i++) {
                f32x4 a = bias;
#pragma unroll
                for (int k = 0; k < TAPS; k++)
#pragma unroll
                    for (int e = 0; e < 4; e++) a[e] = fmaf(r[i + k][e], w[k][e], a[e]);
#pragma unroll
                for (int e = 0; e < 4; e++) a[e] = lr_silu(a[e]);
                if (t0 + i < t1) *(f32x4*)(p.out + (int64_t)(t0 + i) * p.out_ld + c) = a;
            }
            return;
        }
    }
    for (int t = t0; t < t1; t++) {                                  // (tiles that span sequences)
        const int seq = p.tok_seq[t], pos = p.tok_pos[t], first = p.seq_pos[seq];
        const float* ring = p.ring + (int64_t)p.seq_slot[seq] * p.ring_slot_stride;
#pragma unroll
        for (int e = 0; e < 4; e++) if (c + e < p.channels) p.out[(int64_t)t * p.out_ld + c + e] = conv_at(p, ring, t, pos, first, c + e);
    }
}
static __global__ __launch_bounds__(256) void conv_ring_kernel(ConvArgs p) {      // grid (sequences, ceil(channels / 256))
    const int seq = blockIdx.x, n = p.seq_len[seq], c = blockIdx.y * 256 + threadIdx.x;
    if (c >= p.channels) return;
    float* ring = p.ring + (int64_t)p.seq_slot[seq] * p.ring_slot_stride;
    for (int i = max(0, n - p.taps); i < n; i++)
        ring[(int64_t)((p.seq_pos[seq] + i) % p.taps) * p.channels + c] = p.raw[(int64_t)(p.seq_tok_start[seq] + i) * p.raw_ld + c];
}

// ------------------------------------------------------------------------------------------
// RMS norm over equal parts of a row with a silu gate, written as the next projection's operand.
//   GATE_FIRST (Mamba-2):  u = y * silu(gate); out = rms(u) * w[column of the row]
//   else                :  out = rms(y) * w[column of the part] * silu(gate) (GLA), or * sigmoid(gate) with `sig` (delta rule)
// V4: parts, row pitches and bases are multiples of 4 columns.  `lanes` (a power of two <= 64) lanes share a part, or one 256-thread
// workgroup each when the parts are long (WIDE): grid ceil(tokens * parts / (256 / lanes)).
// ------------------------------------------------------------------------------------------
struct GatedNormArgs {
    const float* y; int64_t y_ld;
    const float* gate; int64_t gate_ld;
    const float* w;
    int rows, parts, part;     // part = columns per part
    float eps;
    int64_t out_ld;
    int lanes;
    int sig;
};
template <typename ActT, bool GATE_FIRST, bool WIDE, bool V4>
__global__ __launch_bounds__(256) void gated_norm_kernel(GatedNormArgs p, ActT* __restrict__ out) {
    __shared__ float red[4];
    constexpr int E = V4 ? 4 : 1, KEEP = V4 ? 4 : 8;
    const int nt = WIDE ? 256 : p.lanes, l = threadIdx.x & (nt - 1);
    const int id = WIDE ? blockIdx.x : blockIdx.x * (256 / nt) + threadIdx.x / nt;
    const bool ok = id < p.rows * p.parts;
    const int64_t t = ok ? id / p.parts : 0;
    const int c0 = ok ? (id % p.parts) * p.part : 0, part = ok ? p.part : 0;
    const float* y = p.y + t * p.y_ld + c0;
    const float* g = p.gate + t * p.gate_ld + c0;
    struct Vec { float v[E]; };
    auto ld = [&](const float* a, int c) {
        Vec r;
        if constexpr (V4) { const f32x4 x = *(const f32x4*)(a + c); for (int e = 0; e < 4; e++) r.v[e] = x[e]; }
        else r.v[0] = a[c];
        return r;
    };
    auto load = [&](int c) {
        Vec u = ld(y, c);
        if (GATE_FIRST) {
            const Vec s = ld(g, c);
#pragma unroll
            for (int e = 0; e < E; e++) u.v[e] *= lr_silu(s.v[e]);
        }
        return u;
    };
    Vec u[KEEP];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < KEEP; i++) {
        const int c = (l + i * nt) * E;
#pragma unroll
        for (int e = 0; e < E; e++) u[i].v[e] = 0.f;
        if (c < part) u[i] = load(c);
#pragma unroll
        for (int e = 0; e < E; e++) ss = fmaf(u[i].v[e], u[i].v[e], ss);
    }
    for (int c = (l + KEEP * nt) * E; c < part; c += nt * E) {
        const Vec x = load(c);
#pragma unroll
        for (int e = 0; e < E; e++) ss = fmaf(x.v[e], x.v[e], ss);
    }
    if (WIDE) {
        ss = wave_sum(ss);
        if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = ss;
        __syncthreads();
        ss = red[0] + red[1] + red[2] + red[3];
    } else {
        for (int o = 1; o < nt; o <<= 1) ss += __shfl_xor(ss, o, 64);
    }
    const float inv = 1.0f / sqrtf(ss / (float)p.part + p.eps);
    auto put = [&](int c, Vec x) {
        const Vec w = ld(p.w, GATE_FIRST ? c0 + c : c);
#pragma unroll
        for (int e = 0; e < E; e++) x.v[e] *= inv * w.v[e];
        if (!GATE_FIRST) {
            const Vec s = ld(g, c);
#pragma unroll
            for (int e = 0; e < E; e++) x.v[e] *= p.sig ? lr_sigmoid(s.v[e]) : lr_silu(s.v[e]);
        }
        if constexpr (V4) act_store4<ActT>(out, t, c0 + c, p.out_ld, f32x4{x.v[0], x.v[1], x.v[2], x.v[3]});
        else ActIO<ActT>::st(out + act_index<ActT>(t, c0 + c, p.out_ld), x.v[0]);
    };
#pragma unroll
    for (int i = 0; i < KEEP; i++) { const int c = (l + i * nt) * E; if (c < part) put(c, u[i]); }
    for (int c = (l + KEEP * nt) * E; c < part; c += nt * E) put(c, load(c));
}

// launches (linrec_inst.hip).  ch: a decay per key channel; nk, nw: template arguments of the chunk kernel; par: pieces in parallel
void linrec_step_launch(hipStream_t st, const LinRecArgs& p, int n_seqs, bool ch, bool fused, bool f32);
void linrec_chunk_launch(hipStream_t st, const LinRecArgs& p, int n_seqs, bool ch, int nk, int nw, bool par);

}  // namespace nvl
