// latent.h — attention over a cached low-rank latent (multi-head latent attention without a rotated part), with an optional sliding
// window.  Per token: c_q = rms(W_dq h) * w, q = W_uq c_q; c = rms(W_dkv h) * w; per head k = W_uk c, v = W_uv c; only c is
// cached.  The concatenated heads are multiplied by sigmoid(W_g h) before the output projection.
//
// Two forms of the same attention, chosen per token:
//   expanded (prompt portions): the latents of the keys the portion can see are gathered from the cache, two projections make
//       every head's K and V^T from them, and latent_prefill_kernel runs flash-style over those.
//   absorbed (one or a few new tokens): q' = W_uk^T q per head, scores q' . c and the weighted sum of c straight from the
//       cached latents (one read of c serves all heads), then W_uv per head.  latent_absorb_q_kernel, latent_decode_kernel
//       (keys split over workgroups, partial results in fp32), latent_uv_kernel (combines the partials, projects, gates).
// Scores, softmax and their sums are fp32; the scale is applied to the fp32 scores.
//
// Cache: blocks of `bs` tokens (64 | bs) named by block tables, as for K/V; a layer's part of a block is [bs][rp] latents, rp =
// kv_rank padded to 64 (the padding is zero).  bf16: fragment-major in units of 16 tokens x 32 columns (common.h fm_index on the
// block's rows), so that a score operand is one contiguous KiB; fp32 mode: row-major.
#pragma once
#include "attn.h"
#include "common.h"

namespace nvl {

__device__ __forceinline__ float lat_sigmoid(float x) { return 1.0f / (1.0f + __expf(-x)); }

struct LatentArgs {
    int H, dim, dp, vp, qrank, qrp, kvrank, rp;   // dp / vp / qrp / rp: padded sizes
    int window;                                   // 0: every earlier token
    float scale, eps;
    const float* proj; int64_t proj_ld;           // [token][c_q : qrp | c : rp | gate : H * vp] of the fused input projection
    const float *cq_norm, *c_norm;                // padded with zeros
    void* cq;                                     // operand of W_uq: [token][qrp]
    void* cache; int64_t block_stride;            // this layer's part of block 0; elements between blocks
    int bs;
    const int32_t *blk_table, *tok_pos, *tok_tbl, *seq_tok_start, *seq_len, *seq_pos;
    int tbl_stride;
    const float* q; int64_t q_ld;                 // [token][H * dp]
    // expanded form
    const int32_t* kbase;                         // per sequence: its first row in the key workspace (-1: the sequence takes the absorbed form)
    void* cg;                                     // gathered latents [rows][rp]
    const void *kx, *vx;                          // bf16: K [rows][H * dp] and V^T [H * vp][rows_pad], both fragment-major; fp32: K, V [rows][H * .]
    int64_t rows_pad;
    void* out; int64_t out_ld;                    // operand of W_o: [token][out_ld], head h at column h * vp
    // absorbed form
    const int32_t* abs_tok;                       // the tokens that take it
    const int32_t* abs_seq;
    int n_abs, n_split;
    const bf16_t *ukt, *uv;                       // per head [rp][dp]; [H * vp][rp]; fragment-major
    bf16_t* qa; int Hp;                           // [n_abs][Hp][rp], Hp = H padded to 16
    float *part_o, *part_ml;                      // [split][n_abs][H][rp], [split][n_abs][H][2]
};

// first key the earliest token of a call can see, rounded down to the 32-row unit the gather copies
__host__ __device__ __forceinline__ int latent_key0(int pos0, int window) {
    const int lo = window > 0 ? pos0 - window + 1 : 0;
    return lo > 0 ? (lo & ~31) : 0;
}

// ---- norms of the two latents; c goes to its cache row.  grid (tokens), 256 threads ----
template <typename ActT>
__global__ __launch_bounds__(256) void latent_norm_kernel(LatentArgs p) {
    __shared__ float red[4];
    const int t = blockIdx.x;
    const float* pr = p.proj + (int64_t)t * p.proj_ld;
    auto rms_of = [&](const float* v, int n) {
        float ss = 0.f;
        for (int i = threadIdx.x; i < n; i += 256) ss = fmaf(v[i], v[i], ss);
        ss = wave_sum(ss);
        __syncthreads();
        if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = ss;
        __syncthreads();
        return sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)n + p.eps);
    };
    const float rq = rms_of(pr, p.qrank), rc = rms_of(pr + p.qrp, p.kvrank);
    for (int i = threadIdx.x; i < p.qrp; i += 256)
        ActIO<ActT>::st((ActT*)p.cq + act_index<ActT>(t, i, p.qrp), (pr[i] / rq) * p.cq_norm[i]);
    int blk, row;
    kv_locate(p.blk_table, p.tok_tbl[t], p.tok_pos[t], p.bs, blk, row);
    ActT* c = (ActT*)p.cache + (int64_t)blk * p.block_stride;
    for (int i = threadIdx.x; i < p.rp; i += 256)
        ActIO<ActT>::st(c + act_index<ActT>(row, i, p.rp), (pr[p.qrp + i] / rc) * p.c_norm[i]);
}

// ---- gather the latents a portion's keys need into contiguous rows: 32 rows (one unit of either layout) per workgroup ----
template <typename ActT>
__global__ __launch_bounds__(256) void latent_gather_kernel(LatentArgs p) {
    const int seq = blockIdx.y;
    if (p.kbase[seq] < 0) return;
    const int pos0 = p.seq_pos[seq], k0 = latent_key0(pos0, p.window), nk = pos0 + p.seq_len[seq] - k0;
    const int r0 = blockIdx.x * 32;
    if (r0 >= nk) return;
    const int key = k0 + r0, bi = key / p.bs, row = key - bi * p.bs;
    const int blk = p.blk_table[(int64_t)seq * p.tbl_stride + bi];
    const char* src = (const char*)((const ActT*)p.cache + (int64_t)blk * p.block_stride + (int64_t)row * p.rp);
    char* dst = (char*)((ActT*)p.cg + (int64_t)(p.kbase[seq] + r0) * p.rp);
    for (int64_t i = threadIdx.x * 16; i < (int64_t)32 * p.rp * (int)sizeof(ActT); i += 256 * 16) *(f32x4*)(dst + i) = *(const f32x4*)(src + i);
}

// ------------------------------------------------------------------------------------------
// expanded form, bf16.  grid (ceil(longest portion / 128), H, sequences), 4 waves of 32 query rows.  S^T = K Q^T and
// O^T += V^T P^T as in attn.h, but K and V^T come fragment-major from memory, so no operand passes through LDS: the K rows of a
// 32-key unit are taken in the order that makes the score accumulators (keys 8 fg + r, 8 fg + 4 + r) the B operand against
// V^T's natural key order.
// ------------------------------------------------------------------------------------------
template <int KS, int DT>
__global__ __launch_bounds__(256) void latent_prefill_kernel(LatentArgs p) {
    constexpr int TQ = 2;
    const int seq = blockIdx.z, h = blockIdx.y, qt = gridDim.x - 1 - blockIdx.x;
    const int n = p.seq_len[seq];
    if (qt * 128 >= n || p.kbase[seq] < 0) return;
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int fq = lane & 15, fg = lane >> 4;
    const int tok0 = p.seq_tok_start[seq], pos0 = p.seq_pos[seq];
    const int k0 = latent_key0(pos0, p.window), kb = p.kbase[seq];
    const int row0 = qt * 128 + wave * 32;
    if (row0 >= n) return;                                   // (no barrier in this kernel)
    bf16x8 qf[TQ][KS];
    int qpos[TQ], qtok[TQ];
    bool qok[TQ];
#pragma unroll
    for (int i = 0; i < TQ; i++) {
        int r = row0 + 16 * i + fq;
        qok[i] = r < n;
        if (!qok[i]) r = n - 1;
        qtok[i] = tok0 + r; qpos[i] = pos0 + r;
        const float* qp = p.q + (int64_t)qtok[i] * p.q_ld + h * p.dp;
#pragma unroll
        for (int ks = 0; ks < KS; ks++) {
            const f32x4 a = *(const f32x4*)(qp + ks * 32 + fg * 8), b = *(const f32x4*)(qp + ks * 32 + fg * 8 + 4);
#pragma unroll
            for (int e = 0; e < 4; e++) { qf[i][ks][e] = (bf16_t)a[e]; qf[i][ks][4 + e] = (bf16_t)b[e]; }
        }
    }
    const int first = pos0 + row0, last = pos0 + min(row0 + 31, n - 1);       // positions of this wave's rows
    int lo = p.window > 0 ? first - p.window + 1 : 0;
    if (lo < k0) lo = k0;
    const int j0 = (lo - k0) & ~63, j1 = last - k0;                            // workspace-relative keys
    const int full_lo = p.window > 0 ? last - p.window + 1 : 0, full_hi = first;   // a tile inside [full_lo, full_hi] needs no mask
    const int kt_ld = p.H * p.dp >> 5;                                          // 1-KiB blocks per 16 key rows of K
    const bf16_t* kx = (const bf16_t*)p.kx;
    const bf16_t* vx = (const bf16_t*)p.vx;
    const int64_t vt_ld = p.rows_pad >> 5;
    f32x4 o[TQ][DT];
    float m_run[TQ], l_run[TQ];
#pragma unroll
    for (int i = 0; i < TQ; i++) {
        m_run[i] = -1e30f; l_run[i] = 0.f;
#pragma unroll
        for (int d = 0; d < DT; d++) o[i][d] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    const float sl2 = p.scale * 1.4426950408889634f;
    for (int j = j0; j <= j1; j += 64) {
        const int nu = j + 32 <= j1 ? 2 : 1;                                   // 32-key units of this step that hold keys
        f32x4 s[TQ][4];
#pragma unroll
        for (int i = 0; i < TQ; i++)
#pragma unroll
            for (int t = 0; t < 4; t++) s[i][t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int t = 0; t < 4; t++) {
            if ((t >> 1) >= nu) continue;
            const int key = kb + j + 32 * (t >> 1) + 8 * (fq >> 2) + (fq & 3) + 4 * (t & 1);     // this lane's K row
            const bf16_t* kr = kx + (((int64_t)(key >> 4) * kt_ld + h * KS) * 64 + (key & 15) + 16 * fg) * 8;
#pragma unroll
            for (int ks = 0; ks < KS; ks++) {
                const bf16x8 kf = *(const bf16x8*)(kr + ks * 512);
#pragma unroll
                for (int i = 0; i < TQ; i++) s[i][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[i][ks], s[i][t], 0, 0, 0);
            }
        }
        // lane: S^T[key = 32 (t / 2) + 8 fg + 4 (t & 1) + r][query fq]
        const bool whole = k0 + j >= full_lo && k0 + j + 63 <= full_hi;
#pragma unroll
        for (int i = 0; i < TQ; i++) {
#pragma unroll
            for (int t = 0; t < 4; t++)
#pragma unroll
                for (int r = 0; r < 4; r++) s[i][t][r] *= sl2;
            if (!whole) {
                const int back = qpos[i] - (k0 + j);                            // tile-relative: keys back - window + 1 .. back
                const int from = p.window > 0 ? back - p.window + 1 : 0;
#pragma unroll
                for (int t = 0; t < 4; t++)
#pragma unroll
                    for (int r = 0; r < 4; r++) {
                        const int k = 32 * (t >> 1) + 8 * fg + 4 * (t & 1) + r;
                        if (k > back || k < from || (t >> 1) >= nu) s[i][t][r] = -INFINITY;
                    }
            }
            float mx = s[i][0][0];
#pragma unroll
            for (int t = 0; t < 4; t++)
#pragma unroll
                for (int r = 0; r < 4; r++) mx = fmaxf(mx, s[i][t][r]);
            mx = rows_max(mx);
            const float m_new = fmaxf(m_run[i], mx);
            const float alpha = __builtin_amdgcn_exp2f(m_run[i] - m_new);
            m_run[i] = m_new;
            float ls = 0.f;
#pragma unroll
            for (int t = 0; t < 4; t++)
#pragma unroll
                for (int r = 0; r < 4; r++) { s[i][t][r] = __builtin_amdgcn_exp2f(s[i][t][r] - m_new); ls += s[i][t][r]; }
            l_run[i] = l_run[i] * alpha + ls;
            if (__any(alpha != 1.0f)) {
#pragma unroll
                for (int d = 0; d < DT; d++) o[i][d] *= alpha;
            }
        }
#pragma unroll
        for (int u = 0; u < 2; u++) {
            if (u >= nu) continue;
            bf16x8 pf[TQ];
#pragma unroll
            for (int i = 0; i < TQ; i++)
#pragma unroll
                for (int r = 0; r < 4; r++) { pf[i][r] = (bf16_t)s[i][2 * u][r]; pf[i][4 + r] = (bf16_t)s[i][2 * u + 1][r]; }
            const bf16_t* vr = vx + (((int64_t)(h * DT) * vt_ld + ((kb + j) >> 5) + u) * 64 + lane) * 8;
#pragma unroll
            for (int d = 0; d < DT; d++) {
                const bf16x8 vf = *(const bf16x8*)(vr + (int64_t)d * vt_ld * 512);
#pragma unroll
                for (int i = 0; i < TQ; i++) o[i][d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pf[i], o[i][d], 0, 0, 0);
            }
        }
    }
#pragma unroll
    for (int i = 0; i < TQ; i++) {
        float l = l_run[i];
        l += __shfl_xor(l, 16, 64);
        l += __shfl_xor(l, 32, 64);
        if (!qok[i]) continue;
        const float inv = 1.0f / l;
        const float* gt = p.proj + (int64_t)qtok[i] * p.proj_ld + p.qrp + p.rp + h * p.vp;
#pragma unroll
        for (int d = 0; d < DT; d++) {
            const f32x4 g = *(const f32x4*)(gt + 16 * d + 4 * fg);
            f32x4 v = o[i][d] * inv;
#pragma unroll
            for (int r = 0; r < 4; r++) v[r] *= lat_sigmoid(g[r]);
            act_store4<bf16_t>((bf16_t*)p.out, qtok[i], h * p.vp + 16 * d + 4 * fg, p.out_ld, v);
        }
    }
}

// ---- expanded form, any size: one 256-thread workgroup per (token, head), online softmax over 256 keys at a time, plain fp32
// arithmetic.  The fp32 mode's kernel, and the bf16 mode's for heads wider than the instances above. ----
template <typename T>
__device__ __forceinline__ float lat_k(const LatentArgs& p, int64_t row, int64_t col) { return ((const T*)p.kx)[act_index<T>(row, col, (int64_t)p.H * p.dp)]; }
template <typename T> __device__ __forceinline__ float lat_v(const LatentArgs& p, int64_t row, int64_t col);
template <> __device__ __forceinline__ float lat_v<float>(const LatentArgs& p, int64_t row, int64_t col) { return ((const float*)p.vx)[row * (p.H * p.vp) + col]; }
template <> __device__ __forceinline__ float lat_v<bf16_t>(const LatentArgs& p, int64_t row, int64_t col) { return (float)((const bf16_t*)p.vx)[fm_index(col, row, p.rows_pad)]; }
template <typename T>
__global__ __launch_bounds__(256) void latent_plain_kernel(LatentArgs p) {
    __shared__ float red[4], sp[256];
    extern __shared__ __attribute__((aligned(16))) float lat_sm[];     // q [dp] | o [vp]
    const int seq = blockIdx.z, h = blockIdx.y, r = blockIdx.x, tid = threadIdx.x;
    if (r >= p.seq_len[seq] || p.kbase[seq] < 0) return;
    const int64_t t = p.seq_tok_start[seq] + r;
    const int pos0 = p.seq_pos[seq], pos = pos0 + r, k0 = latent_key0(pos0, p.window);
    int lo = p.window > 0 ? pos - p.window + 1 : 0;
    if (lo < 0) lo = 0;
    float* sq = lat_sm;
    float* so = sq + p.dp;
    for (int i = tid; i < p.dp; i += 256) sq[i] = p.q[t * p.q_ld + h * p.dp + i];
    for (int i = tid; i < p.vp; i += 256) so[i] = 0.f;
    float m = -1e30f, l = 0.f;
    __syncthreads();
    auto bmax = [&](float v) { v = wave_max(v); if ((tid & 63) == 0) red[tid >> 6] = v; __syncthreads(); v = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])); __syncthreads(); return v; };
    auto bsum = [&](float v) { v = wave_sum(v); if ((tid & 63) == 0) red[tid >> 6] = v; __syncthreads(); v = red[0] + red[1] + red[2] + red[3]; __syncthreads(); return v; };
    for (int base = lo; base <= pos; base += 256) {
        const int key = base + tid;
        float s = -INFINITY;
        if (key <= pos) {
            float a = 0.f;
            const int64_t row = p.kbase[seq] + key - k0;
            for (int d = 0; d < p.dim; d++) a = fmaf(sq[d], lat_k<T>(p, row, h * p.dp + d), a);
            s = a * p.scale;
        }
        const float mn = fmaxf(m, bmax(s)), alpha = expf(m - mn);
        const float e = key <= pos ? expf(s - mn) : 0.f;
        m = mn;
        l = l * alpha + bsum(e);
        sp[tid] = e;
        __syncthreads();
        const int nk = min(256, pos - base + 1);
        for (int i = tid; i < p.vp; i += 256) {
            float a = so[i] * alpha;
            for (int j = 0; j < nk; j++) a = fmaf(sp[j], lat_v<T>(p, p.kbase[seq] + base + j - k0, h * p.vp + i), a);
            so[i] = a;
        }
        __syncthreads();
    }
    for (int i = tid; i < p.vp; i += 256) {
        const float g = p.proj[t * p.proj_ld + p.qrp + p.rp + h * p.vp + i];
        ActIO<T>::st((T*)p.out + act_index<T>(t, h * p.vp + i, p.out_ld), so[i] / l * (1.0f / (1.0f + expf(-g))));
    }
}

// ------------------------------------------------------------------------------------------
// absorbed form (bf16)
// ------------------------------------------------------------------------------------------
// q'[token][head][:] = W_uk[head]^T q[token][head]: grid (H, rp / 64, ceil(n_abs / 16)), one 16-column tile per wave, K = dp
static __global__ __launch_bounds__(256) void latent_absorb_q_kernel(LatentArgs p) {
    const int h = blockIdx.x, nt = blockIdx.y * 4 + (threadIdx.x >> 6), mt = blockIdx.z, lane = threadIdx.x & 63;
    const int fr = lane & 15, fg = lane >> 4, nks = p.dp >> 5;
    const int i = mt * 16 + fr;
    const bool ok = i < p.n_abs;
    const float* qp = ok ? p.q + (int64_t)p.abs_tok[i] * p.q_ld + h * p.dp + fg * 8 : nullptr;
    const bf16_t* w = p.ukt + (int64_t)h * p.rp * p.dp + ((int64_t)nt * nks * 64 + lane) * 8;
    f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int ks = 0; ks < nks; ks++) {
        const bf16x8 wf = *(const bf16x8*)(w + ks * 512);
        bf16x8 af = {};
        if (ok) {
            const f32x4 a = *(const f32x4*)(qp + ks * 32), b = *(const f32x4*)(qp + ks * 32 + 4);
#pragma unroll
            for (int e = 0; e < 4; e++) { af[e] = (bf16_t)a[e]; af[4 + e] = (bf16_t)b[e]; }
        }
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf, af, acc, 0, 0, 0);
    }
    if (!ok) return;
    bf16x4 o;
#pragma unroll
    for (int r = 0; r < 4; r++) o[r] = (bf16_t)acc[r];
    *(bf16x4*)(p.qa + ((int64_t)i * p.Hp + h) * p.rp + nt * 16 + 4 * fg) = o;
}

// grid (ceil(H / 16), n_abs, n_split), 4 waves, 64 keys per step (inside one block: 64 | bs).  Wave w scores keys 16 w .. of the step
// (operand blocks straight from the cache, copied to an LDS image on the way), the waves agree on the maximum, exchange the
// weights through LDS, and wave w accumulates its rp / 4 latent columns over all 64 keys from the image by transposed reads.
template <int NR>                  // rp = 64 NR
constexpr int latent_decode_lds_bytes() { return 2 * 64 * NR * 64 * 2 + 16 * 16 * 8 + 2 * 4 * 16 * 4; }
template <int NR>
__global__ __launch_bounds__(256) void latent_decode_kernel(LatentArgs p) {
    constexpr int IMG = 64 * NR * 64 * 2, KSN = 2 * NR;
    extern __shared__ __attribute__((aligned(16))) char lat_smc[];
    char* pl = lat_smc + 2 * IMG;                            // weights: [key quad][query][4] bf16
    float* wmax = (float*)(pl + 16 * 16 * 8);                // [4 waves][16]
    float* wsum = wmax + 64;
    const int ht = blockIdx.x, ia = blockIdx.y, z = blockIdx.z;
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int fq = lane & 15, fg = lane >> 4;
    const int tok = p.abs_tok[ia], seq = p.abs_seq[ia];
    const int pos = p.tok_pos[tok];
    int lo = p.window > 0 ? pos - p.window + 1 : 0;
    if (lo < 0) lo = 0;
    const int kt_first = lo >> 6, n_kt = (pos >> 6) - kt_first + 1, per = (n_kt + p.n_split - 1) / p.n_split;
    const int kt0 = kt_first + z * per, kt1 = min(kt0 + per, kt_first + n_kt);
    const int32_t* tbl = p.blk_table + (int64_t)seq * p.tbl_stride;
    bf16x8 qf[KSN];
#pragma unroll
    for (int ks = 0; ks < KSN; ks++) qf[ks] = *(const bf16x8*)(p.qa + ((int64_t)ia * p.Hp + ht * 16 + fq) * p.rp + ks * 32 + fg * 8);
    f32x4 o[NR];
#pragma unroll
    for (int i = 0; i < NR; i++) o[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    float m = -1e30f, l = 0.f;
    const float sl2 = p.scale * 1.4426950408889634f;
    const int tr_row = 4 * fg + (fq >> 2), tr_p = fq & 3;
    auto src_of = [&](int kt) {
        const int key = kt * 64, bi = key / p.bs, row = key - bi * p.bs;
        const int blk = __builtin_amdgcn_readfirstlane(tbl[bi]);
        return (const bf16_t*)p.cache + (int64_t)blk * p.block_stride + (int64_t)(row + 16 * wave) * p.rp + lane * 8;
    };
    bf16x8 a[KSN];
    if (kt0 < kt1) {
        const bf16_t* s = src_of(kt0);
#pragma unroll
        for (int ks = 0; ks < KSN; ks++) a[ks] = *(const bf16x8*)(s + ks * 512);
    }
    for (int kt = kt0; kt < kt1; kt++) {
        char* img = lat_smc + ((kt - kt0) & 1) * IMG;
        f32x4 s = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < KSN; ks++) {
            s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[ks], qf[ks], s, 0, 0, 0);
            *(bf16x8*)(img + ((wave * KSN + ks) * 64 + lane) * 16) = a[ks];
        }
        if (kt + 1 < kt1) {
            const bf16_t* sn = src_of(kt + 1);
#pragma unroll
            for (int ks = 0; ks < KSN; ks++) a[ks] = *(const bf16x8*)(sn + ks * 512);
        }
        const int key = kt * 64 + 16 * wave + 4 * fg;
        float mx = -INFINITY;
#pragma unroll
        for (int r = 0; r < 4; r++) {
            s[r] = (key + r >= lo && key + r <= pos) ? s[r] * sl2 : -INFINITY;
            mx = fmaxf(mx, s[r]);
        }
        mx = rows_max(mx);
        if (fg == 0) wmax[wave * 16 + fq] = mx;
        __syncthreads();
        const float mn = fmaxf(m, fmaxf(fmaxf(wmax[fq], wmax[16 + fq]), fmaxf(wmax[32 + fq], wmax[48 + fq])));
        const float alpha = __builtin_amdgcn_exp2f(m - mn);
        m = mn;
        bf16x4 pw;
        float ls = 0.f;
#pragma unroll
        for (int r = 0; r < 4; r++) { const float e = __builtin_amdgcn_exp2f(s[r] - mn); ls += e; pw[r] = (bf16_t)e; }
        l = l * alpha + ls;
        *(bf16x4*)(pl + ((4 * wave + fg) * 16 + fq) * 8) = pw;
        __syncthreads();
        bf16x8 pf[2];
#pragma unroll
        for (int u = 0; u < 2; u++) {
            const bf16x4 x = *(const bf16x4*)(pl + ((8 * u + fg) * 16 + fq) * 8), y = *(const bf16x4*)(pl + ((8 * u + 4 + fg) * 16 + fq) * 8);
#pragma unroll
            for (int r = 0; r < 4; r++) { pf[u][r] = x[r]; pf[u][4 + r] = y[r]; }
        }
#pragma unroll
        for (int i = 0; i < NR; i++) {
            const int col = (wave * NR + i) * 16 + 4 * tr_p;
            o[i] *= alpha;
            // element (row, col) of a 16-row tile of the image: block col / 32, lane (row & 15) + 16 ((col & 31) / 8), 2 (col & 7) bytes in
            const int off = ((col >> 5) * 64 + tr_row + 16 * ((col & 31) >> 3)) * 16 + 2 * (col & 7);
#pragma unroll
            for (int u = 0; u < 2; u++) {
                const bf16x4 x = lds_read_tr4(img + (2 * u) * (KSN * 1024) + off), y = lds_read_tr4(img + (2 * u + 1) * (KSN * 1024) + off);
                bf16x8 cf;
#pragma unroll
                for (int r = 0; r < 4; r++) { cf[r] = x[r]; cf[4 + r] = y[r]; }
                o[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(cf, pf[u], o[i], 0, 0, 0);
            }
        }
    }
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    if (fg == 0) wsum[wave * 16 + fq] = l;
    __syncthreads();
    const int h = ht * 16 + fq;
    if (h >= p.H) return;
    const int64_t at = ((int64_t)z * p.n_abs + ia) * p.H + h;
    if (wave == 0 && fg == 0) { p.part_ml[2 * at] = m; p.part_ml[2 * at + 1] = (wsum[fq] + wsum[16 + fq]) + (wsum[32 + fq] + wsum[48 + fq]); }
#pragma unroll
    for (int i = 0; i < NR; i++) *(f32x4*)(p.part_o + at * p.rp + (wave * NR + i) * 16 + 4 * fg) = o[i];
}

// combines the key splits, projects by W_uv and gates: grid (H, vp / 16, ceil(n_abs / 16)), 4 waves share K = rp
static __global__ __launch_bounds__(256) void latent_uv_kernel(LatentArgs p) {
    __shared__ f32x4 red[4][64];
    const int h = blockIdx.x, vt = blockIdx.y, mt = blockIdx.z, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int fr = lane & 15, fg = lane >> 4, nks = p.rp >> 5;
    const int i = mt * 16 + fr;
    const bool ok = i < p.n_abs;
    float M = -1e30f, L = 0.f;
    if (ok) {
        for (int z = 0; z < p.n_split; z++) M = fmaxf(M, p.part_ml[2 * (((int64_t)z * p.n_abs + i) * p.H + h)]);
        for (int z = 0; z < p.n_split; z++) {
            const float* ml = p.part_ml + 2 * (((int64_t)z * p.n_abs + i) * p.H + h);
            L += ml[1] * __builtin_amdgcn_exp2f(ml[0] - M);
        }
    }
    const float invL = ok ? 1.0f / L : 0.f;
    const bf16_t* w = p.uv + ((int64_t)(h * (p.vp >> 4) + vt) * nks * 64 + lane) * 8;
    f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int ks = wave; ks < nks; ks += 4) {
        const bf16x8 wf = *(const bf16x8*)(w + ks * 512);
        bf16x8 af = {};
        if (ok) {
            f32x4 a = f32x4{0.f, 0.f, 0.f, 0.f}, b = a;
            for (int z = 0; z < p.n_split; z++) {
                const int64_t at = ((int64_t)z * p.n_abs + i) * p.H + h;
                const float e = __builtin_amdgcn_exp2f(p.part_ml[2 * at] - M);
                const float* po = p.part_o + at * p.rp + ks * 32 + fg * 8;
                a += e * *(const f32x4*)po;
                b += e * *(const f32x4*)(po + 4);
            }
#pragma unroll
            for (int e = 0; e < 4; e++) { af[e] = (bf16_t)(a[e] * invL); af[4 + e] = (bf16_t)(b[e] * invL); }
        }
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf, af, acc, 0, 0, 0);
    }
    red[wave][lane] = acc;
    __syncthreads();
    if (wave || !ok) return;
    acc = (red[0][lane] + red[1][lane]) + (red[2][lane] + red[3][lane]);
    const int64_t t = p.abs_tok[i];
    const int col = h * p.vp + vt * 16 + 4 * fg;
    const f32x4 g = *(const f32x4*)(p.proj + t * p.proj_ld + p.qrp + p.rp + col);
#pragma unroll
    for (int r = 0; r < 4; r++) acc[r] *= lat_sigmoid(g[r]);
    act_store4<bf16_t>((bf16_t*)p.out, t, col, p.out_ld, acc);
}

}  // namespace nvl
