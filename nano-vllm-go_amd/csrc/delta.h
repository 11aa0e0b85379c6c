// delta.h — gated delta rule with a decay per key channel, in fp32 throughout.  Per head, S [DK][DV]:
//     S <- diag(a_t) S,  u_t = beta_t (v_t - S^T k_t),  S <- S + k_t u_t^T,  o_t = S^T q_t
// q and k are unit vectors (q also times q_scale); a_t = exp(-exp(A_log) softplus(z_t + bias)), z_t a projection; a group of heads
// shares q and k, decays and values are a head's own.
//
//   delta_step_kernel   token by token, the state streamed once per token (decode).  FUSED (one token per sequence): the short
//                       convolutions, the low-rank decay and gate projections, the head norm and the output gate in the same launch.
//   delta_prep_kernel   32 tokens of one head, independent of the state that enters them (prefill, all chunks at once).
//   delta_scan_kernel   carries the state through the chunks of a sequence: three products per chunk.
//
// Chunk form.  With b_t = the inclusive sum of log a inside the chunk and S_in the state that enters it:
//     u_t = beta_t (v_t - (k_t e^{b_t})^T S_in - sum_{s<t} M[t][s] u_s),      M[t][s] = sum_c k_t[c] k_s[c] e^{b_t[c] - b_s[c]}
//     o_t = (q_t e^{b_t})^T S_in + sum_{s<=t} A[t][s] u_s,                    A[t][s] = sum_c q_t[c] k_s[c] e^{b_t[c] - b_s[c]}
//     S_out = diag(e^{b_end}) S_in + sum_s (k_s e^{b_end - b_s}) u_s^T
// With T = (I + diag(beta) M)^-1 diag(beta):  U = U0 - W S_in,  U0 = T V,  W = T (K e^b);  O = O0 + Q' S_in,  O0 = (A T) V,
// Q' = Q e^b - (A T) (K e^b).  prep leaves -W, Q', (K e^{b_end - b})^T and e^{b_end} in scratch, U0 in the place of v and O0 in the place of o.
// Every exponent that is evaluated is <= 0: a decay per channel cannot be split into e^{b_t} e^{-b_s}, so the two 16 x 16 diagonal
// blocks of A and M are summed pair by pair, and the block below the diagonal takes token 15's sums as its reference.  T is built
// block by block from exact inverses: the powers of M that a series would need can be far larger than T itself.
// Products are v_mfma_f32_16x16x4_f32: operand element i of lane group g stands for k = 16 n + 4 g + i on both sides, so that an
// accumulator (lane = column, rows 4 g + r) is the B operand of the next product as it stands.
#pragma once
#include "common.h"
#include "linrec.h"

namespace nvl {

constexpr float DELTA_UNIT_EPS = 1e-6f;

struct DeltaArgs {
    int H, G, DK, DV, DVp;             // G: heads of q and k; DVp: row pitch of the state (DV padded to 4)
    const float *q, *k; float* v;      // after convolution and silu; row pitch ld; v: prep leaves U0 there
    int64_t ld;
    float q_scale;
    const float* z; int64_t z_ld;      // [token][H * DK] decay projections before the bias
    const float *a_log, *dt_bias;      // [H], [H * DK]
    const float* beta; int64_t beta_ld;        // raw step sizes (before sigmoid), one column per head
    float* o; int64_t o_ld;            // [token][H * DV]
    float* state; int64_t slot_stride; // slot s: state + s * slot_stride, [H][DK][DVp]
    const int32_t *seq_tok_start, *seq_len, *seq_pos, *seq_slot;
    int vec4, vec4v;                   // q, k / v, o rows may be accessed 16 bytes at a time
    int len_lo, len_hi;                // sequences with len_lo <= tokens of this call <= len_hi are served, the others skipped
    float* ws;                         // chunk c of sequence i is (seq_tok_start / 32 + i + c); per chunk and head delta_ws_floats
    // FUSED step: raw [q | k | v] columns before the convolution, a ring of the last `taps` raw rows per slot
    const float* raw; int64_t raw_ld; const float* conv_w; int taps, channels; float* ring; int64_t ring_slot_stride;
    const float *a1, *g1; int64_t lr_ld; int a_rank, g_rank, a_rkp, g_rkp;       // [token][rank]; ranks padded
    const void *a2, *g2;               // [H * DK][a_rkp], [H * DV][g_rkp], row-major
    const float* norm_w; float eps; void* out; int64_t out_ld;
};

constexpr int DELTA_C = 32;            // tokens per chunk
static inline __host__ __device__ int64_t delta_ws_floats(int dkp) { return (int64_t)dkp * (3 * DELTA_C + 1); }     // -W | Q' | K^T | e^{b_end}
__device__ __forceinline__ int64_t delta_chunk(const DeltaArgs& p, int seq, int c) { return p.seq_tok_start[seq] / DELTA_C + seq + c; }

// log(1 + e^x) from the hardware's base-2 exponential and logarithm; what 1 + y rounds away is added back
__device__ __forceinline__ float delta_softplus(float x) {
    const float y = ex2(-1.4426950408889634f * fabsf(x)), u = 1.0f + y;
    return fmaxf(x, 0.f) + fmaf(0.6931471805599453f, __builtin_amdgcn_logf(u), (y - (u - 1.0f)) * __builtin_amdgcn_rcpf(u));
}

// ------------------------------------------------------------------------------------------
// prep: grid (heads, sequences, chunks), 8 waves
// ------------------------------------------------------------------------------------------
template <int NK> constexpr int delta_prep_lds_bytes() { return 4 * (3 * DELTA_C * (NK * 16 + 4) + 2 * DELTA_C * 36 + DELTA_C + 512); }

template <int NK>
__global__ __launch_bounds__(512, NK > 8 ? 2 : 4) void delta_prep_kernel(DeltaArgs p) {
    constexpr int C = DELTA_C, DKP = NK * 16, LQ = DKP + 4, LA = 36, NT = 512, NW = NT / 64;
    constexpr float LOG2E = 1.4426950408889634f;
    const int h = blockIdx.x, seq = blockIdx.y, c0 = blockIdx.z * C;
    const int n = p.seq_len[seq];
    if (n < p.len_lo || n > p.len_hi || c0 >= n) return;         // (uniform: before any barrier)
    extern __shared__ __attribute__((aligned(16))) float dl_sm[];
    float* qs = dl_sm;                   // [C][LQ]  q, later q e^b
    float* ks = qs + C * LQ;             // [C][LQ]  k, later k e^b
    float* bs = ks + C * LQ;             // [C][LQ]  inclusive sums of log2 a
    float* As = bs + C * LQ;             // [C][LA]  A, later A T
    float* Ms = As + C * LA;             // [C][LA]  M, later X = (I + diag(beta) M)^-1
    float* be = Ms + C * LA;             // [C]
    float* aux = be + C;                 // [512]
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int fr = lane & 15, fg = lane >> 4;
    const int nv = min(C, n - c0);
    const int64_t tb = (int64_t)p.seq_tok_start[seq] + c0;
    const int g = h / (p.H / p.G);
    // every load of the chunk first: q and k (DKP / 4 lanes hold a row), z (a channel per thread, NG groups share the tokens) and the
    // first value channels of this wave
    constexpr int LR = DKP / 4, R = NT / LR, NQ = (C + R - 1) / R, NG = NT / DKP, TPG = C / NG;
    const int qt = tid / LR, qd = tid % LR * 4, zd = tid % DKP, grp = tid / DKP, nvb = (p.DV + 15) >> 4;
    f32x4 q4[NQ], k4[NQ], v4[2];
    float pre[TPG];
    auto ld4 = [&](const float* src) {
        f32x4 x = f32x4{0.f, 0.f, 0.f, 0.f};
        if (p.vec4) { if (qd < p.DK) x = *(const f32x4*)(src + qd); }
        else {
#pragma unroll
            for (int r = 0; r < 4; r++) if (qd + r < p.DK) x[r] = src[qd + r];
        }
        return x;
    };
    auto ldv = [&](int i, f32x4 (&v)[2]) {       // 16 value channels as the A operand of a transposed product
        const int c = 16 * i + fr;
        const float* vb = p.v + tb * p.ld + (int64_t)h * p.DV + min(c, p.DV - 1);
#pragma unroll
        for (int sb = 0; sb < 2; sb++)
#pragma unroll
            for (int r = 0; r < 4; r++) {
                const int t = 16 * sb + 4 * fg + r;
                const float x = vb[min(t, nv - 1) * p.ld];
                v[sb][r] = c < p.DV && t < nv ? x : 0.f;
            }
    };
#pragma unroll
    for (int i = 0; i < NQ; i++) {
        const int t = qt + i * R;
        q4[i] = k4[i] = f32x4{0.f, 0.f, 0.f, 0.f};
        if (t < nv) { q4[i] = ld4(p.q + (tb + t) * p.ld + (int64_t)g * p.DK); k4[i] = ld4(p.k + (tb + t) * p.ld + (int64_t)g * p.DK); }
    }
#pragma unroll
    for (int j = 0; j < TPG; j++) pre[j] = p.z[(tb + min(grp * TPG + j, nv - 1)) * p.z_ld + (int64_t)h * p.DK + min(zd, p.DK - 1)];
    if (wave < nvb) ldv(wave, v4);
#pragma unroll
    for (int i = 0; i < NQ; i++) {               // unit vectors
        const f32x4 q = q4[i], k = k4[i];
        float sq = (q[0] * q[0] + q[1] * q[1]) + (q[2] * q[2] + q[3] * q[3]), sk = (k[0] * k[0] + k[1] * k[1]) + (k[2] * k[2] + k[3] * k[3]);
#pragma unroll
        for (int o = 1; o < LR; o <<= 1) { sq += __shfl_xor(sq, o, 64); sk += __shfl_xor(sk, o, 64); }
        if (C % R && qt + i * R >= C) continue;
        *(f32x4*)(qs + (qt + i * R) * LQ + qd) = q * (p.q_scale / sqrtf(sq + DELTA_UNIT_EPS));
        *(f32x4*)(ks + (qt + i * R) * LQ + qd) = k * (1.0f / sqrtf(sk + DELTA_UNIT_EPS));
    }
    {   // decays
        const float A = -expf(p.a_log[h]) * LOG2E, bias = zd < p.DK ? p.dt_bias[h * p.DK + zd] : 0.f;
#pragma unroll
        for (int j = 0; j < TPG; j++) pre[j] = zd < p.DK && grp * TPG + j < nv ? A * delta_softplus(pre[j] + bias) : 0.f;
#pragma unroll
        for (int j = 1; j < TPG; j++) pre[j] += pre[j - 1];
        aux[grp * DKP + zd] = pre[TPG - 1];
        if (tid < C) be[tid] = tid < nv ? lr_sigmoid(p.beta[(tb + tid) * p.beta_ld + h]) : 0.f;
        __syncthreads();
        float off = 0.f;
        for (int j = 0; j < grp; j++) off += aux[j * DKP + zd];
#pragma unroll
        for (int j = 0; j < TPG; j++) bs[(grp * TPG + j) * LQ + zd] = off + pre[j];
    }
    for (int i = tid; i < 2 * C * LA; i += NT) As[i] = 0.f;      // (what lies above the diagonals stays zero)
    __syncthreads();
    // ---- A (s <= t) and M (s < t): 240 pairs of the two diagonal blocks, two threads each; the other 32 threads take A's diagonal ----
    if (tid < 480) {
        const int pr = tid >> 1, half = pr >= 120, x = pr - 120 * half;
        int t = (int)((sqrtf(8.f * (float)x + 1.f) - 1.f) * 0.5f);
        if ((t + 1) * (t + 2) / 2 <= x) t++;
        if (t * (t + 1) / 2 > x) t--;
        const int s = x - t * (t + 1) / 2, tr = (16 * half + t + 1) * LQ, sr = (16 * half + s) * LQ;
        f32x4 aq = f32x4{0.f, 0.f, 0.f, 0.f}, ak = aq;
#pragma unroll 2
        for (int d = 4 * (tid & 1); d < DKP; d += 8) {
            const f32x4 q4 = *(const f32x4*)(qs + tr + d), k4 = *(const f32x4*)(ks + tr + d), k2 = *(const f32x4*)(ks + sr + d);
            const f32x4 bt = *(const f32x4*)(bs + tr + d), b2 = *(const f32x4*)(bs + sr + d);
#pragma unroll
            for (int r = 0; r < 4; r++) { const float e = ex2(bt[r] - b2[r]) * k2[r]; aq[r] = fmaf(q4[r], e, aq[r]); ak[r] = fmaf(k4[r], e, ak[r]); }
        }
        const int at = (16 * half + t + 1) * LA + 16 * half + s;
        float sa = (aq[0] + aq[1]) + (aq[2] + aq[3]), sm = (ak[0] + ak[1]) + (ak[2] + ak[3]);
        sa += __shfl_xor(sa, 1, 64);
        sm += __shfl_xor(sm, 1, 64);
        if (tid & 1) Ms[at] = sm; else As[at] = sa;
    } else {
        const int t = tid - 480;
        f32x4 a = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 2
        for (int d = 0; d < DKP; d += 4) a += *(const f32x4*)(qs + t * LQ + d) * *(const f32x4*)(ks + t * LQ + d);
        As[t * LA + t] = (a[0] + a[1]) + (a[2] + a[3]);
    }
    if (wave < 2) {                                              // tokens 16..31 against 0..15: wave 0 A, wave 1 M
        const float* x = wave == 0 ? qs : ks;
        f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 2
        for (int i = 0; i < NK; i++) {
            const int c = 16 * i + 4 * fg;
            const f32x4 ref = *(const f32x4*)(bs + 15 * LQ + c);
            const f32x4 a = *(const f32x4*)(x + (16 + fr) * LQ + c), b = *(const f32x4*)(ks + fr * LQ + c);
            const f32x4 ba = *(const f32x4*)(bs + (16 + fr) * LQ + c), bb = *(const f32x4*)(bs + fr * LQ + c);
#pragma unroll
            for (int r = 0; r < 4; r++) acc = mfma_f32(a[r] * ex2(ba[r] - ref[r]), b[r] * ex2(ref[r] - bb[r]), acc);
        }
        float* dst = wave == 0 ? As : Ms;
#pragma unroll
        for (int r = 0; r < 4; r++) dst[(16 + 4 * fg + r) * LA + fr] = acc[r];
    }
    __syncthreads();
    float* ws = p.ws + (delta_chunk(p, seq, blockIdx.z) * p.H + h) * delta_ws_floats(DKP);
    if (wave < 2) {
        // inverses of the two diagonal blocks of I + N, N = diag(beta) M, from 1 x 1 blocks upwards: with X the inverse of the part inside
        // b x b blocks and N_b the part that a 2b x 2b block adds, X - X N_b X is the inverse inside 2b x 2b blocks
        const int o = 16 * wave;
        float* xt = aux + 256 * wave;                            // X's turn from accumulator to A operand
        const f32x4 na = *(const f32x4*)(Ms + (o + fr) * LA + o + 4 * fg) * be[o + fr];
        f32x4 xa, xd;
#pragma unroll
        for (int r = 0; r < 4; r++) {
            const int c = 4 * fg + r;                            // (row fr, column c) as an A operand, (row c, column fr) as an accumulator
            xa[r] = fr == c ? 1.f : ((fr ^ c) == 1 ? -na[r] : 0.f);
            xd[r] = fr == c ? 1.f : ((fr ^ c) == 1 ? -Ms[(o + c) * LA + o + fr] * be[o + c] : 0.f);
        }
#pragma unroll
        for (int lb = 1; lb < 4; lb++) {                         // b = 2, 4, 8
            f32x4 y = f32x4{0.f, 0.f, 0.f, 0.f}, z = y;
#pragma unroll
            for (int r = 0; r < 4; r++) y = mfma_f32(((fr ^ (4 * fg + r)) >> lb) == 1 ? na[r] : 0.f, xd[r], y);
#pragma unroll
            for (int r = 0; r < 4; r++) z = mfma_f32(xa[r], y[r], z);
            xd -= z;
            if (lb == 3) break;
#pragma unroll
            for (int r = 0; r < 4; r++) xt[(4 * fg + r) * 16 + fr] = xd[r];
            asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
            xa = *(const f32x4*)(xt + fr * 16 + 4 * fg);
        }
#pragma unroll
        for (int r = 0; r < 4; r++) Ms[(o + 4 * fg + r) * LA + o + fr] = xd[r];
    } else {
        // (K e^{b_end - b})^T and e^{b_end}; 32 tokens of a channel side by side
        float* kt = ws + 2 * C * DKP;
#pragma unroll 2
        for (int i = tid - 128; i < C * DKP; i += NT - 128) {
            const int t = i & 31, d = i >> 5;
            kt[d * C + t] = ks[t * LQ + d] * ex2(bs[31 * LQ + d] - bs[t * LQ + d]);
        }
        for (int d = tid - 128; d < DKP; d += NT - 128) ws[3 * C * DKP + d] = ex2(bs[31 * LQ + d]);
    }
    __syncthreads();
    if (wave == 0) {
        // the block below the diagonal: -X22 N21 X11; then A T, T = X diag(beta), in A's place
        const f32x4 n21 = *(const f32x4*)(Ms + (16 + fr) * LA + 4 * fg) * be[16 + fr], x22 = *(const f32x4*)(Ms + (16 + fr) * LA + 16 + 4 * fg);
        f32x4 x11, y = f32x4{0.f, 0.f, 0.f, 0.f}, w = y, aa[3], at[3];
#pragma unroll
        for (int x = 0; x < 3; x++) {
            aa[x] = *(const f32x4*)(As + (16 * (x > 0) + fr) * LA + 16 * (x > 1) + 4 * fg);
            at[x] = w;
        }
#pragma unroll
        for (int r = 0; r < 4; r++) { x11[r] = Ms[(4 * fg + r) * LA + fr]; y = mfma_f32(n21[r], x11[r], y); }
#pragma unroll
        for (int r = 0; r < 4; r++) w = mfma_f32(x22[r], y[r], w);
#pragma unroll
        for (int r = 0; r < 4; r++) {
            const float t00 = x11[r] * be[fr], t10 = -w[r] * be[fr], t11 = Ms[(16 + 4 * fg + r) * LA + 16 + fr] * be[16 + fr];
            at[0] = mfma_f32(aa[0][r], t00, at[0]); at[1] = mfma_f32(aa[1][r], t00, at[1]);
            at[1] = mfma_f32(aa[2][r], t10, at[1]); at[2] = mfma_f32(aa[2][r], t11, at[2]);
            Ms[(16 + 4 * fg + r) * LA + fr] = -w[r];
        }
#pragma unroll
        for (int x = 0; x < 3; x++)
#pragma unroll
            for (int r = 0; r < 4; r++) As[(16 * (x > 0) + 4 * fg + r) * LA + 16 * (x > 1) + fr] = at[x][r];
    } else {
#pragma unroll 2
        for (int i = tid - 64; i < C * DKP / 4; i += NT - 64) {  // q e^b, k e^b in place
            const int t = i / (DKP / 4), d = i % (DKP / 4) * 4;
            const f32x4 b = *(const f32x4*)(bs + t * LQ + d);
            f32x4 q = *(const f32x4*)(qs + t * LQ + d), k = *(const f32x4*)(ks + t * LQ + d);
#pragma unroll
            for (int r = 0; r < 4; r++) { const float e = ex2(b[r]); q[r] *= e; k[r] *= e; }
            *(f32x4*)(qs + t * LQ + d) = q;
            *(f32x4*)(ks + t * LQ + d) = k;
        }
    }
    __syncthreads();
    // rows of T and of A T, blocks (0,0), (1,0), (1,1): B operands of the transposed products, whose accumulators hold four channels of a token
    f32x4 ta[3], ba[3];
#pragma unroll
    for (int x = 0; x < 3; x++) {
        const int at = (16 * (x > 0) + fr) * LA + 16 * (x > 1) + 4 * fg;
        ta[x] = *(const f32x4*)(Ms + at) * *(const f32x4*)(be + 16 * (x > 1) + 4 * fg);
        ba[x] = *(const f32x4*)(As + at);
    }
    auto times = [&](const f32x4 (&x)[2], const f32x4 (&m)[3], f32x4 (&d)[2]) {          // d += (m x)^T
#pragma unroll
        for (int r = 0; r < 4; r++) { d[0] = mfma_f32(x[0][r], m[0][r], d[0]); d[1] = mfma_f32(x[0][r], m[1][r], d[1]); }
#pragma unroll
        for (int r = 0; r < 4; r++) d[1] = mfma_f32(x[1][r], m[2][r], d[1]);
    };
    for (int i = wave; i < NK; i += NW) {                         // 16 key channels: -W and Q'
        f32x4 k[2], w[2], q[2];
#pragma unroll
        for (int sb = 0; sb < 2; sb++) {
#pragma unroll
            for (int r = 0; r < 4; r++) k[sb][r] = -ks[(16 * sb + 4 * fg + r) * LQ + 16 * i + fr];
            w[sb] = f32x4{0.f, 0.f, 0.f, 0.f};
            q[sb] = *(const f32x4*)(qs + (16 * sb + fr) * LQ + 16 * i + 4 * fg);
        }
        times(k, ta, w);
        times(k, ba, q);
#pragma unroll
        for (int tt = 0; tt < 2; tt++) {
            *(f32x4*)(ws + (16 * tt + fr) * DKP + 16 * i + 4 * fg) = w[tt];
            *(f32x4*)(ws + (C + 16 * tt + fr) * DKP + 16 * i + 4 * fg) = q[tt];
        }
    }
    for (int i = wave; i < nvb; i += NW) {                       // 16 value channels: U0 and O0
        f32x4 v[2] = {v4[0], v4[1]}, u[2], o[2];
        if (i != wave) ldv(i, v);
        u[0] = u[1] = o[0] = o[1] = f32x4{0.f, 0.f, 0.f, 0.f};
        times(v, ta, u);
        times(v, ba, o);
        const int c = 16 * i + 4 * fg;
#pragma unroll
        for (int tt = 0; tt < 2; tt++) {
            const int t = 16 * tt + fr;
            float* ub = p.v + (tb + t) * p.ld + (int64_t)h * p.DV + c;
            float* ob = p.o + (tb + t) * p.o_ld + (int64_t)h * p.DV + c;
            if (t >= nv) continue;
            if (p.vec4v) { if (c < p.DV) { *(f32x4*)ub = u[tt]; *(f32x4*)ob = o[tt]; } }
            else
#pragma unroll
                for (int r = 0; r < 4; r++) if (c + r < p.DV) { ub[r] = u[tt][r]; ob[r] = o[tt][r]; }
        }
    }
}

// ------------------------------------------------------------------------------------------
// scan: grid (heads, sequences, slices of 16 NW / KSP value columns).  A wave keeps DK / KSP x 16 of the state in accumulators: 16 columns,
// and with KSP > 1 (few heads and sequences) a part of the key channels — the parts' sums of U and O meet in LDS.
// The next chunk's operands are on their way to registers while the state is updated.
// ------------------------------------------------------------------------------------------
template <int NK, int NW, int KSP> constexpr int delta_scan_lds_bytes() { return 4 * (2 * DELTA_C * (NK * 16 + 4) + NK * 16 * 36 + NK * 16 + (KSP > 1 ? NW * 1024 : 0)); }

template <int NK, int NW, int KSP>
__global__ __launch_bounds__(NW * 64, NK > 8 ? 1 : (NW == 8 ? (KSP > 1 ? 2 : 4) : 3)) void delta_scan_kernel(DeltaArgs p) {
    constexpr int C = DELTA_C, DKP = NK * 16, LQ = DKP + 4, LK = 36, NT = NW * 64, NKW = NK / KSP, NCG = NW / KSP;
    const int h = blockIdx.x, seq = blockIdx.y;
    const int n = p.seq_len[seq];
    if (n < p.len_lo || n > p.len_hi) return;
    extern __shared__ __attribute__((aligned(16))) float dl_sm[];
    float* wl = dl_sm;                   // [C][LQ]   -W
    float* ql = wl + C * LQ;             // [C][LQ]   Q'
    float* kl = ql + C * LQ;             // [DKP][LK] (K e^{b_end - b})^T
    float* dl = kl + DKP * LK;           // [DKP]     e^{b_end}
    f32x4* xb = (f32x4*)(dl + DKP);      // KSP > 1: [part][column group][U, U, O, O][lane]
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int fr = lane & 15, fg = lane >> 4;
    const int cg = wave % NCG, kq = wave / NCG, ch0 = kq * NKW * 16;       // this wave's column group, part and first key channel
    const int col = (blockIdx.z * NCG + cg) * 16 + fr;
    const bool live = col < p.DV, slive = col < p.DVp;
    const int64_t tok0 = p.seq_tok_start[seq];
    const bool fresh = p.seq_pos[seq] == 0;
    float* st = p.state + (int64_t)p.seq_slot[seq] * p.slot_stride + (int64_t)h * p.DK * p.DVp;
    f32x4 S[NKW];
    {   // (clamped addresses instead of branches)
        const int sc = min(col, p.DVp - 1);
#pragma unroll
        for (int i = 0; i < NKW; i++)
#pragma unroll
            for (int r = 0; r < 4; r++) {
                const int row = ch0 + 16 * i + 4 * fg + r;
                const float x = st[min(row, p.DK - 1) * p.DVp + sc];
                S[i][r] = !fresh && slive && row < p.DK ? x : 0.f;
            }
    }
    constexpr int E = 3 * C * DKP / 4, NL = E / NT;              // 16-byte pieces of a chunk's operands, per thread
    static_assert(NKW % 2 == 0 && NW % KSP == 0, "pairs of 16 channels");
    static_assert(E % (3 * NT) == 0 && NT >= DKP, "whole pieces, one decay per thread");
    const int64_t stride = p.H * delta_ws_floats(DKP);
    const float* src = p.ws + (delta_chunk(p, seq, 0) * p.H + h) * delta_ws_floats(DKP);
    f32x4 rg[NL], u[2], o[2];
    float rd = 0.f;
    const int ld = (int)p.ld, old = (int)p.o_ld;
    const char* vb = (const char*)(p.v + tok0 * p.ld + (int64_t)h * p.DV);
    char* ob = (char*)(p.o + tok0 * p.o_ld + (int64_t)h * p.DV);
    const uint32_t cb = 4 * min(col, p.DV - 1);
    auto fetch = [&]() {
#pragma unroll
        for (int i = 0; i < NL; i++) rg[i] = ((const f32x4*)src + i * NT)[tid];
        rd = src[3 * C * DKP + min(tid, DKP - 1)];
    };
    // U0 and O0 of 32 tokens.  Beyond the sequence's end the last token is read again: finite, against zero columns of K, never stored.
    auto fetch_uo = [&](const char* v, const char* oc, int left) {
        if (KSP > 1 && kq > 0) {         // (wave-uniform: the first part starts from U0 and O0)
            u[0] = u[1] = o[0] = o[1] = f32x4{0.f, 0.f, 0.f, 0.f};
            return;
        }
#pragma unroll
        for (int tt = 0; tt < 2; tt++)
#pragma unroll
            for (int r = 0; r < 4; r++) {
                const uint32_t t = min(16 * tt + 4 * fg + r, left - 1);
                const float x = *(const float*)(v + (t * (uint32_t)ld * 4 + cb));
                u[tt][r] = live ? x : 0.f;                       // (the state's padding columns stay zero)
                o[tt][r] = *(const float*)(oc + (t * (uint32_t)old * 4 + cb));
            }
    };
    fetch();
    fetch_uo(vb, ob, n);
    for (int c0 = 0; c0 < n; c0 += C) {
        __syncthreads();                                         // the previous chunk's readers are done
        float *w0 = wl + tid / (DKP / 4) * LQ + tid % (DKP / 4) * 4, *k0 = kl + (tid >> 3) * LK + (tid & 7) * 4;
#pragma unroll
        for (int i = 0; i < NL; i++)
            if (i < NL / 3 * 2) *(f32x4*)(w0 + i * (NT / (DKP / 4)) * LQ) = rg[i];
            else *(f32x4*)(k0 + (i - NL / 3 * 2) * (NT / 8) * LK) = rg[i];
        if (tid < DKP) dl[tid] = rd;
        __syncthreads();
#pragma unroll
        for (int i = 0; i < NKW; i++) {
            f32x4 a[4];
#pragma unroll
            for (int tt = 0; tt < 2; tt++) {
                a[tt] = *(const f32x4*)(wl + (16 * tt + fr) * LQ + ch0 + 16 * i + 4 * fg);
                a[2 + tt] = *(const f32x4*)(ql + (16 * tt + fr) * LQ + ch0 + 16 * i + 4 * fg);
            }
#pragma unroll
            for (int r = 0; r < 4; r++) {
                u[0] = mfma_f32(a[0][r], S[i][r], u[0]); u[1] = mfma_f32(a[1][r], S[i][r], u[1]);
                o[0] = mfma_f32(a[2][r], S[i][r], o[0]); o[1] = mfma_f32(a[3][r], S[i][r], o[1]);
            }
            if (i & 1) __builtin_amdgcn_sched_barrier(0);        // (or all reads are hoisted to the front, and registers spill)
        }
        if constexpr (KSP > 1) {
            f32x4* x = xb + (kq * NCG + cg) * 256 + lane;
            x[0] = u[0]; x[64] = u[1]; x[128] = o[0]; x[192] = o[1];
            __syncthreads();
            u[0] = u[1] = o[0] = o[1] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int q = 0; q < KSP; q++) {
                const f32x4* y = xb + (q * NCG + cg) * 256 + lane;
                u[0] += y[0]; u[1] += y[64];
                if (kq == 0) o[0] += y[128];                     // (the first two parts store 16 tokens each)
                if (kq == 1) o[1] += y[192];
            }
        }
#pragma unroll
        for (int tt = 0; tt < 2; tt++)
#pragma unroll
            for (int r = 0; r < 4; r++) {
                const int t = 16 * tt + 4 * fg + r;
                if (live && c0 + t < n && (KSP == 1 || kq == tt)) *(float*)(ob + ((uint32_t)t * (uint32_t)old * 4 + cb)) = o[tt][r];
            }
        f32x4 ub[2] = {u[0], u[1]};
        __builtin_amdgcn_sched_barrier(0);
        const bool more = c0 + C < n;                            // (the last chunk is fetched once more instead of a branch)
        src += more ? stride : 0; vb += more ? (int64_t)C * ld * 4 : 0; ob += more ? (int64_t)C * old * 4 : 0;
        fetch();
        fetch_uo(vb, ob, more ? n - c0 - C : n - c0);
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int i = 0; i < NKW; i += 2) {
            f32x4 a[2][2];
#pragma unroll
            for (int x = 0; x < 2; x++)
#pragma unroll
                for (int sb = 0; sb < 2; sb++) a[x][sb] = *(const f32x4*)(kl + (ch0 + 16 * (i + x) + fr) * LK + 16 * sb + 4 * fg);
            S[i] *= *(const f32x4*)(dl + ch0 + 16 * i + 4 * fg);
            S[i + 1] *= *(const f32x4*)(dl + ch0 + 16 * (i + 1) + 4 * fg);
#pragma unroll
            for (int sb = 0; sb < 2; sb++)
#pragma unroll
                for (int r = 0; r < 4; r++) { S[i] = mfma_f32(a[0][sb][r], ub[sb][r], S[i]); S[i + 1] = mfma_f32(a[1][sb][r], ub[sb][r], S[i + 1]); }
            __builtin_amdgcn_sched_barrier(0);
        }
    }
    int so = 4 * fg * p.DVp + col;
    asm volatile("" : "+v"(so));                                 // (or addresses are kept in registers all along)
    st += ch0 * p.DVp;
#pragma unroll
    for (int i = 0; i < NKW; i++)
#pragma unroll
        for (int r = 0; r < 4; r++)
            if (slive && ch0 + 16 * i + 4 * fg + r < p.DK) (st + (16 * i + r) * p.DVp)[so] = S[i][r];
}

// ------------------------------------------------------------------------------------------
// token by token.  grid (H, sequences), 512 threads: tv threads side by side on a state row (4 columns each), 512 / tv rows at a time.
// With S' = diag(a) S both S'^T k and S'^T q come from one pass over the state: o = S'^T q + (k . q) u.
// ------------------------------------------------------------------------------------------
static inline int delta_step_lds_bytes(int DK, int DVp, int ranks) {
    int tv = 1;
    while (tv < DVp / 4) tv <<= 1;
    const int nred = tv >= 64 ? LR_STEP_THREADS / tv : LR_STEP_THREADS / 64;
    return 4 * (3 * ((DK + 3) & ~3) + 2 * DVp + 2 * nred * DVp + ranks);
}
template <typename WT> __device__ __forceinline__ float delta_dot16(const WT* w, const float* x);       // 16 bytes of weights
template <> __device__ __forceinline__ float delta_dot16<float>(const float* w, const float* x) {
    const f32x4 a = *(const f32x4*)w, b = *(const f32x4*)x;
    return fmaf(a[3], b[3], fmaf(a[2], b[2], fmaf(a[1], b[1], a[0] * b[0])));
}
template <> __device__ __forceinline__ float delta_dot16<bf16_t>(const bf16_t* w, const float* x) {
    const bf16x8 a = *(const bf16x8*)w;
    float s = 0.f;
#pragma unroll
    for (int i = 0; i < 8; i++) s = fmaf((float)a[i], x[i], s);
    return s;
}

template <bool FUSED, int ROWS, typename ActT>           // ROWS: state rows a thread keeps in registers; ActT: type of `out` and of a2 / g2
__global__ __launch_bounds__(LR_STEP_THREADS, ROWS <= 8 ? 4 : 2) void delta_step_kernel(DeltaArgs p) {
    constexpr int NT = LR_STEP_THREADS, NW = NT / 64;
    const int h = blockIdx.x, seq = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int n = FUSED ? 1 : p.seq_len[seq];
    if (n < p.len_lo || n > p.len_hi) return;
    extern __shared__ __attribute__((aligned(16))) float dl_sm[];
    const int DK4 = (p.DK + 3) & ~3;
    float* sq = dl_sm;                   // [DK]
    float* sk = sq + DK4;                // [DK]
    float* sa = sk + DK4;                // [DK]   decays
    float* sv = sa + DK4;                // [DVp]
    float* sg = sv + p.DVp;              // [DVp]  output gates (FUSED)
    const int nv4 = p.DVp >> 2;
    int tv = 1;
    while (tv < nv4) tv <<= 1;           // host: nv4 <= NT
    const int rg = tid / tv, tc = tid - rg * tv, RG = NT / tv, NRED = tv >= 64 ? RG : NW;
    float* red = sg + p.DVp;             // [NRED][2][DVp]
    float* lr = red + 2 * NRED * p.DVp;  // [a_rkp + g_rkp] (FUSED)
    __shared__ float s_red[NW], s_sum[3];
    const bool live = tc < nv4;
    const int t0 = p.seq_tok_start[seq], pos0 = p.seq_pos[seq], slot = p.seq_slot[seq];
    const int g = h / (p.H / p.G);
    float* st = p.state + (int64_t)slot * p.slot_stride + (int64_t)h * p.DK * p.DVp;
    int so = rg * p.DVp + 4 * tc;        // this thread's place in a pass of RG rows
    const int pass = RG * p.DVp;
    f32x4 s[ROWS];                       // the first ROWS rows of this thread, fetched before anything else is known
#pragma unroll
    for (int i = 0; i < ROWS; i++) {
        const bool ok = live && rg + i * RG < p.DK;
        const f32x4 x = *(const f32x4*)(st + (ok ? i * pass + so : 0));
#pragma unroll
        for (int r = 0; r < 4; r++) s[i][r] = ok && pos0 > 0 ? x[r] : 0.f;
    }
    asm volatile("" : "+v"(so));         // (or the addresses of these loads are kept in registers for the stores)
    for (int i = tid; i < p.DVp; i += NT) { sv[i] = 0.f; sg[i] = 0.f; }
    __syncthreads();
    const float ea = expf(p.a_log[h]);
    for (int it = 0; it < n; it++) {
        const int64_t t = t0 + it;
        if constexpr (FUSED) {
            // causal convolution + silu of this head's channels (n == 1)
            const float* rw = p.raw + t * p.raw_ld;
            float* ring = p.ring + (int64_t)slot * p.ring_slot_stride;
            const int KD = p.G * p.DK;
#pragma unroll 1
            for (int i = tid; i < 2 * p.DK + p.DV; i += NT) {
                const int c = i < p.DK ? g * p.DK + i : (i < 2 * p.DK ? KD + g * p.DK + i - p.DK : 2 * KD + h * p.DV + i - 2 * p.DK);
                const float cur = rw[c];
                float acc = 0.f;
                for (int b = p.taps - 1; b >= 1; b--)
                    if (pos0 - b >= 0) acc = fmaf(ring[(int64_t)((pos0 - b) % p.taps) * p.channels + c], p.conv_w[(int64_t)c * p.taps + p.taps - 1 - b], acc);
                acc = fmaf(cur, p.conv_w[(int64_t)c * p.taps + p.taps - 1], acc);
                ring[(int64_t)(pos0 % p.taps) * p.channels + c] = cur;      // (heads of a group write the same values; nobody reads this row now)
                const float y = lr_silu(acc);
                if (i < p.DK) sq[i] = y;
                else if (i < 2 * p.DK) sk[i - p.DK] = y;
                else sv[i - 2 * p.DK] = y;
            }
            for (int i = tid; i < p.a_rkp + p.g_rkp; i += NT) {
                const int j = i - p.a_rkp;
                lr[i] = j < 0 ? (i < p.a_rank ? p.a1[t * p.lr_ld + i] : 0.f) : (j < p.g_rank ? p.g1[t * p.lr_ld + j] : 0.f);
            }
            __syncthreads();
            // decay and gate projections: four lanes per output
            constexpr int CH = 16 / (int)sizeof(ActT);
#pragma unroll 1
            for (int i = tid >> 2; i < p.DK + p.DV; i += NT / 4) {
                const bool dec = i < p.DK;
                const int rkp = dec ? p.a_rkp : p.g_rkp;
                const ActT* w = dec ? (const ActT*)p.a2 + (int64_t)(h * p.DK + i) * rkp : (const ActT*)p.g2 + (int64_t)(h * p.DV + i - p.DK) * rkp;
                const float* x = dec ? lr : lr + p.a_rkp;
                float a = 0.f;
                for (int e = (tid & 3) * CH; e < rkp; e += 4 * CH) a += delta_dot16<ActT>(w + e, x + e);
                a += __shfl_xor(a, 1, 64);
                a += __shfl_xor(a, 2, 64);
                if ((tid & 3) == 0) {
                    if (dec) sa[i] = expf(-ea * delta_softplus(a + p.dt_bias[h * p.DK + i]));
                    else sg[i - p.DK] = lr_sigmoid(a);
                }
            }
        } else {
            for (int i = tid; i < p.DK; i += NT) {
                sq[i] = p.q[t * p.ld + (int64_t)g * p.DK + i];
                sk[i] = p.k[t * p.ld + (int64_t)g * p.DK + i];
                sa[i] = expf(-ea * delta_softplus(p.z[t * p.z_ld + (int64_t)h * p.DK + i] + p.dt_bias[h * p.DK + i]));
            }
            for (int i = tid; i < p.DV; i += NT) sv[i] = p.v[t * p.ld + (int64_t)h * p.DV + i];
        }
        __syncthreads();
        if (wave < 3) {                  // q . q, k . k, k . q
            const float *x = wave == 1 ? sk : sq, *y = wave == 0 ? sq : sk;
            float a = 0.f;
            for (int i = lane; i < p.DK; i += 64) a = fmaf(x[i], y[i], a);
            a = wave_sum(a);
            if (lane == 0) s_sum[wave] = a;
        }
        __syncthreads();
        const float iq = p.q_scale / sqrtf(s_sum[0] + DELTA_UNIT_EPS), ik = 1.0f / sqrtf(s_sum[1] + DELTA_UNIT_EPS), kq = s_sum[2] * iq * ik;
        const float beta = lr_sigmoid(p.beta[t * p.beta_ld + h]);
        f32x4 ra = f32x4{0.f, 0.f, 0.f, 0.f}, pa = ra;      // S'^T k, S'^T q
#pragma unroll
        for (int i = 0; i < ROWS; i++) {
            const int row = rg + i * RG;
            const bool ok = live && row < p.DK;
            const int rr = ok ? row : 0;
            const float al = sa[rr], kk = ok ? sk[rr] : 0.f, qq = ok ? sq[rr] : 0.f;
#pragma unroll
            for (int r = 0; r < 4; r++) { s[i][r] *= al; ra[r] = fmaf(kk, s[i][r], ra[r]); pa[r] = fmaf(qq, s[i][r], pa[r]); }
        }
#pragma unroll 1
        for (int row = rg + ROWS * RG; live && row < p.DK; row += RG) {     // (a state larger than the registers: streamed)
            f32x4 w = f32x4{0.f, 0.f, 0.f, 0.f};
            if (pos0 + it > 0) w = *(const f32x4*)(st + (int64_t)row * p.DVp + 4 * tc);
            w *= sa[row];
            ra += sk[row] * w; pa += sq[row] * w;
        }
        for (int o = tv; o < 64; o <<= 1)
#pragma unroll
            for (int r = 0; r < 4; r++) { ra[r] += __shfl_xor(ra[r], o, 64); pa[r] += __shfl_xor(pa[r], o, 64); }
        if (live && (tv >= 64 || lane < tv)) {
            float* d = red + (int64_t)(tv >= 64 ? rg : wave) * 2 * p.DVp + 4 * tc;
            *(f32x4*)d = ra;
            *(f32x4*)(d + p.DVp) = pa;
        }
        __syncthreads();
        f32x4 u = f32x4{0.f, 0.f, 0.f, 0.f}, ov = u;
        if (live) {
            ra = u; pa = u;
#pragma unroll 4
            for (int r = 0; r < NRED; r++) { ra += *(const f32x4*)(red + (int64_t)r * 2 * p.DVp + 4 * tc); pa += *(const f32x4*)(red + (int64_t)r * 2 * p.DVp + p.DVp + 4 * tc); }
            u = beta * (*(const f32x4*)(sv + 4 * tc) - ra * ik);
            ov = pa * iq + kq * u;
        }
#pragma unroll
        for (int i = 0; i < ROWS; i++) {
            const int row = rg + i * RG;
            const bool ok = live && row < p.DK;
            const float kk = ok ? sk[ok ? row : 0] * ik : 0.f;
#pragma unroll
            for (int r = 0; r < 4; r++) s[i][r] = fmaf(kk, u[r], s[i][r]);
            if (ok && it == n - 1) *(f32x4*)(st + i * pass + so) = s[i];
        }
#pragma unroll 1
        for (int row = rg + ROWS * RG; live && row < p.DK; row += RG) {
            float* sr = st + (int64_t)row * p.DVp + 4 * tc;
            f32x4 w = f32x4{0.f, 0.f, 0.f, 0.f};
            if (pos0 + it > 0) w = *(const f32x4*)sr;
            *(f32x4*)sr = w * sa[row] + sk[row] * ik * u;
        }
        if constexpr (FUSED) {
            // (columns beyond DV: v, S and hence o are zero)
            float ss = rg == 0 ? (ov[0] * ov[0] + ov[1] * ov[1]) + (ov[2] * ov[2] + ov[3] * ov[3]) : 0.f;
            ss = wave_sum(ss);
            if (lane == 0) s_red[wave] = ss;
            __syncthreads();
            float tot = 0.f;
#pragma unroll
            for (int i = 0; i < NW; i++) tot += s_red[i];
            const float inv = 1.0f / sqrtf(tot / (float)p.DV + p.eps);
            if (live && rg == 0)
#pragma unroll
                for (int r = 0; r < 4; r++)
                    if (4 * tc + r < p.DV)
                        ActIO<ActT>::st((ActT*)p.out + act_index<ActT>(t, (int64_t)h * p.DV + 4 * tc + r, p.out_ld), ov[r] * inv * p.norm_w[4 * tc + r] * sg[4 * tc + r]);
        } else if (live && rg == 0) {
#pragma unroll
            for (int r = 0; r < 4; r++) if (4 * tc + r < p.DV) p.o[t * p.o_ld + (int64_t)h * p.DV + 4 * tc + r] = ov[r];
        }
        __syncthreads();
    }
}

// ---- columns [0, n) and [off2, off2 + n2) of fp32 rows as the operands of two projections (padded with zeros): grid (tokens) ----
struct PackArgs { const float* src; int64_t ld; int n1, np1, n2, np2, off2; void *d1, *d2; };
template <typename ActT>
__global__ __launch_bounds__(64) void pack_rows_kernel(PackArgs p) {
    const int64_t t = blockIdx.x;
    const float* x = p.src + t * p.ld;
    for (int i = threadIdx.x * 4; i < p.np1 + p.np2; i += 256) {
        const bool a = i < p.np1;
        const int c = a ? i : i - p.np1, n = a ? p.n1 : p.n2;
        f32x4 v;
#pragma unroll
        for (int r = 0; r < 4; r++) v[r] = c + r < n ? x[(a ? 0 : p.off2) + c + r] : 0.f;
        act_store4<ActT>((ActT*)(a ? p.d1 : p.d2), t, c, a ? p.np1 : p.np2, v);
    }
}

// launches (delta_inst.hip); nk: template argument of the chunk kernels
void delta_step_launch(hipStream_t st, const DeltaArgs& p, int n_seqs, bool fused, bool f32);
void delta_prep_launch(hipStream_t st, const DeltaArgs& p, dim3 grid, int nk);
void delta_scan_launch(hipStream_t st, const DeltaArgs& p, int n_seqs, int nk);

}  // namespace nvl
