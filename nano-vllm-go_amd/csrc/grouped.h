// grouped.h — grouped-query attention of models described by a list of layers: H query heads share G key/value heads, query/key and
// value sizes differ freely, and every score passes through
//     s = q . k * scale;   s <- softcap tanh(s / softcap);   s <- s - r1 ln(1 + r2 (i - j))
// (cap and bias are optional, r1 and r2 belong to the query head) before a softmax over the keys of a KeyMask (common.h) and, with a sink,
// one more entry of the denominator that has a score of its own and neither key nor value.  Queries and keys may be normed (per head or
// over the whole projection) and rotated first: grouped_qk_*_kernel, on the fp32 rows the projection leaves.  The values may be mixed with
// those of an earlier layer before they are cached; the concatenated heads are multiplied by sigmoid(gate) where there is a gate.
// Norms, angles, scores, cap, bias, softmax and their sums are fp32.
//
// Cache: blocks of `bs` tokens (64 | bs) named by block tables.  A layer's part of a block is [G][bs][dp] keys, then [G][vp][bs] values,
// dp / vp = padded head sizes (the padding is zero).  bf16: both are stored as the MFMA operand blocks they are read as (common.h
// fm_index), so every operand of either kernel is one contiguous KiB of the cache: the keys of a 32-token unit in the order that
// makes the score accumulators (keys 8 fg + r, 8 fg + 4 + r) the B operand against the values' natural order (grouped_k_row), the
// values transposed.  fp32 mode: plain rows, values [G][bs][vp].
//
// A "query row" is a (token, head of the group) pair, token-major, so that all heads of a group use one pass over K and V:
//   grouped_prefill_kernel : 8 waves x 32 rows, 64-key tiles of K and V^T through a 3-slot LDS ring filled by LDS-DMA (as latent.h)
//   grouped_short_kernel   : sequences with few query rows (decoding, short portions): 16 rows, key tiles dealt over waves and workgroups
//   grouped_plain_kernel   : fp32 mode, and heads wider than the instances above
#pragma once
#include "attn.h"
#include "common.h"
#include "latent.h"

namespace nvl {

struct GroupedArgs {
    int H, G, group, dim, dp, vdim, vp;
    KeyMask mask;
    float scale, softcap;                         // softcap 0: none
    const float *r1, *r2;                         // [H] or NULL: no distance bias
    const float* sink;                            // [H] scores of the denominator's own entry, or NULL
    float out_scale;
    const void* q; int64_t q_ld;                  // queries of head h at column h dp, its gate at column gate_col + h vp: bf16 (fragment-major) or the fp32 rows of proj
    int gate_col;                                 // < 0: no gate
    const float* proj; int64_t proj_ld;           // fp32 mode: [token][q : H dp | k : G dp | v : G vp | gate : H vp | ...] of the fused input projection
    int k_off, v_off;                             // k_off < 0: the keys are in the cache already
    // normed and / or rotated queries and keys (grouped_qk_*_kernel): fp32 columns [0, H dp) and [qk_koff, + G dp) of proj
    int qk_koff, qk_norm, rot;                    // qk_norm: 0 none, 1 per head, 2 over the projection; rot: rotated dimensions
    const float *q_norm, *k_norm;                 // [dim] or [heads dim]
    const f32x2* turn;                            // [position][rot / 2] (cos, sin)
    float eps;
    void* q_out;                                  // what `q` is read from: [token][q_ld]
    const int32_t *tok_pos, *tok_tbl; int rows;
    int mix;                                      // values: 0 as they are, 1 also the model's first (kept in vfirst), 2 mixed with vfirst
    const float* lambda; float* vfirst; int64_t vfirst_ld;      // [token][G vp]
    void* cache; int64_t block_stride; int bs;    // this layer's part of block 0; elements between blocks
    const int32_t *blk_table, *seq_tok_start, *seq_len, *seq_pos;
    int tbl_stride;
    int short_rows;                               // sequences with up to this many query rows belong to grouped_short_kernel
    void* out; int64_t out_ld;                    // operand of W_o: [token][out_ld], head h at column h * vp
    int table;                                    // grouped_prefill_kernel: the distance bias comes from a table in LDS (it has room for it)
    float* part; int32_t* part_cnt;               // keys split over workgroups: partial results, arrival tickets (zero between launches)
};

// ---- fp32 mode: keys and values of the batch's tokens into the cache (bf16: gemm.h EPI_GROUPED): grid (32-token units of a sequence's new positions, sequences, G) ----
static __global__ __launch_bounds__(256) void grouped_place_kernel(GroupedArgs p) {
    const int seq = blockIdx.y, g = blockIdx.z, n = p.seq_len[seq], pos0 = p.seq_pos[seq], tok0 = p.seq_tok_start[seq];
    const int u0 = (pos0 & ~31) + blockIdx.x * 32;                     // first position of the unit
    const int a = max(u0, pos0), b = min(u0 + 32, pos0 + n);           // positions [a, b) are written
    if (a >= b) return;
    const int bi = u0 / p.bs, row0 = u0 - bi * p.bs;
    float* base = (float*)p.cache + (int64_t)p.blk_table[(int64_t)seq * p.tbl_stride + bi] * p.block_stride;
    float* kc = base + (int64_t)g * p.bs * p.dp;
    float* vc = base + (int64_t)p.G * p.bs * p.dp + (int64_t)g * p.bs * p.vp;
    const float lam = p.mix == 2 ? *p.lambda : 0.f;
    for (int pos = a; pos < b; pos++) {
        const int64_t t = tok0 + pos - pos0;
        const int row = row0 + pos - u0;
        const float* pr = p.proj + t * p.proj_ld;
        if (p.k_off >= 0) for (int c = threadIdx.x; c < p.dp; c += 256) kc[(int64_t)row * p.dp + c] = pr[p.k_off + g * p.dp + c];
        for (int c = threadIdx.x; c < p.vp; c += 256) {
            float v = pr[p.v_off + g * p.vp + c];
            float* f = p.vfirst + t * p.vfirst_ld + g * p.vp + c;
            if (p.mix == 1) *f = v;
            else if (p.mix == 2) v = (1.0f - lam) * v + lam * *f;
            vc[(int64_t)row * p.vp + c] = v;
        }
    }
}

// ---- queries and keys of the batch's tokens: RMS norm, rotation; queries to q_out, keys to their cache rows ----
// where the key of token t and head g goes (its channel 0): bf16 an operand block's row, fp32 mode a plain row
template <typename T>
__device__ __forceinline__ T* grouped_key_row(const GroupedArgs& p, int64_t t, int g, int& row) {
    int blk;
    kv_locate(p.blk_table, p.tok_tbl[t], p.tok_pos[t], p.bs, blk, row);
    if (sizeof(T) == 2) row = grouped_k_row(row);
    return (T*)p.cache + (int64_t)blk * p.block_stride + (int64_t)g * p.bs * p.dp;
}
// channel c of a head whose fp32 row is x and norm weight w (NULL: none), already scaled by inv: rotated
__device__ __forceinline__ float grouped_turn(const GroupedArgs& p, const float* x, const float* w, float inv, const f32x2* turn, int c) {
    auto at = [&](int i) { return w ? x[i] * inv * w[i] : x[i]; };
    if (c >= p.dim) return 0.f;
    if (c >= p.rot) return at(c);
    const int half = p.rot >> 1;
    const f32x2 cs = turn[c < half ? c : c - half];
    return c < half ? at(c) * cs[0] - at(c + half) * cs[1] : at(c) * cs[0] + at(c - half) * cs[1];
}
// one wave per (token, head), no workgroup to wait for: small batches, fp32 mode.  A head of up to 256 channels stays in registers, four a
// lane, and pairs meet by a shuffle; a norm over the projection reads the whole row in every wave (it comes from L2).
template <typename T>
__global__ __launch_bounds__(256) void grouped_qk_row_kernel(GroupedArgs p) {
    const int heads = p.H + p.G, id = blockIdx.x * 4 + __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
    if (id >= p.rows * heads) return;
    const int64_t t = id / heads;
    const int h = id - (int)t * heads;
    const bool is_q = h < p.H;
    const int hh = is_q ? h : h - p.H, half = p.rot >> 1, c = lane * 4;
    const float* row = p.proj + t * p.proj_ld + (is_q ? 0 : p.qk_koff);
    const float* x = row + (int64_t)hh * p.dp;
    const float* w = is_q ? p.q_norm : p.k_norm;
    if (p.qk_norm == 2) w += (int64_t)hh * p.dim;
    const bool whole = p.dp <= 256, fast = whole && p.dim % 4 == 0 && half % 4 == 0;      // a lane's channels are data or padding, turn or do not, as one
    const f32x2* turn = p.rot ? p.turn + (int64_t)p.tok_pos[t] * half : nullptr;
    f32x4 v = f32x4{0.f, 0.f, 0.f, 0.f}, ww = f32x4{1.f, 1.f, 1.f, 1.f};
    if (c < p.dp) v = *(const f32x4*)(x + c);
    if (fast && p.qk_norm && c < p.dim) {
#pragma unroll
        for (int r = 0; r < 4; r++) ww[r] = w[c + r];
    }
    f32x2 cs[4];
#pragma unroll
    for (int r = 0; r < 4; r++) cs[r] = fast && c < p.rot ? turn[(c < half ? c : c - half) + r] : f32x2{1.f, 0.f};
    float inv = 1.f, ss = 0.f;
    if (p.qk_norm == 1) {
        ss = v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3];       // (padding is zero)
        for (int i = c + 256; i < p.dp; i += 256) { const f32x4 u = *(const f32x4*)(x + i); ss += u[0] * u[0] + u[1] * u[1] + u[2] * u[2] + u[3] * u[3]; }
        inv = 1.0f / sqrtf(wave_sum(ss) / (float)p.dim + p.eps);
    } else if (p.qk_norm == 2) {
        const int n = (is_q ? p.H : p.G) * p.dp;
#pragma unroll 8
        for (int i = c; i < n; i += 256) { const f32x4 u = *(const f32x4*)(row + i); ss += u[0] * u[0] + u[1] * u[1] + u[2] * u[2] + u[3] * u[3]; }
        inv = 1.0f / sqrtf(wave_sum(ss) / ((float)p.dim * (is_q ? p.H : p.G)) + p.eps);
    }
    int krow = 0;
    T* dst = is_q ? (T*)p.q_out : grouped_key_row<T>(p, t, hh, krow);
    auto put = [&](int i, f32x4 y) {
        if (is_q) act_store4<T>(dst, t, h * p.dp + i, p.q_ld, y);
        else act_store4<T>(dst, krow, i, p.dp, y);
    };
    if (fast) {
        if (p.qk_norm) v *= inv * ww;
        const int other = c < half ? lane + (half >> 2) : lane - (half >> 2);
        f32x4 y;
#pragma unroll
        for (int r = 0; r < 4; r++) {
            const float u = __shfl(v[r], other & 63, 64);
            y[r] = c < p.rot ? (c < half ? v[r] * cs[r][0] - u * cs[r][1] : v[r] * cs[r][0] + u * cs[r][1]) : v[r];
        }
        if (c < p.dp) put(c, y);
        return;
    }
    for (int i = c; i < p.dp; i += 256) {
        f32x4 y;
#pragma unroll
        for (int r = 0; r < 4; r++) y[r] = grouped_turn(p, x, p.qk_norm ? w : nullptr, inv, turn, i + r);
        put(i, y);
    }
}
// Prompts, bf16: one workgroup per 16 tokens, a wave per head.  A lane is a row of the operand blocks it writes (token l & 15, channels
// 8 (l >> 4) ..), so a query head's stores are whole KiB; rows of keys are 16-byte pieces of the cache's blocks.
static __global__ __launch_bounds__(1024) void grouped_qk_tile_kernel(GroupedArgs p) {
    __shared__ float sums[2][16][16];                 // [q, k][wave][token]
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int tok = blockIdx.x * 16 + (lane & 15), c0 = (lane >> 4) * 8;
    const bool ok = tok < p.rows;
    const int64_t t = ok ? tok : p.rows - 1;
    const float* row = p.proj + t * p.proj_ld + c0;
    auto head_x = [&](int h) { return row + (h < p.H ? (int64_t)h * p.dp : p.qk_koff + (int64_t)(h - p.H) * p.dp); };
    auto squares = [&](const float* x) {              // of this lane's token
        float a = 0.f;
        for (int b = 0; b < p.dp; b += 32) {
            const f32x4 u = *(const f32x4*)(x + b), v = *(const f32x4*)(x + b + 4);
            a += (u[0] * u[0] + u[1] * u[1]) + (u[2] * u[2] + u[3] * u[3]) + (v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3]);
        }
        a += __shfl_xor(a, 16, 64);
        return a + __shfl_xor(a, 32, 64);
    };
    if (p.qk_norm == 2) {
        float sq = 0.f, sk = 0.f;
        for (int h = wave; h < p.H + p.G; h += 16) (h < p.H ? sq : sk) += squares(head_x(h));
        if (lane < 16) { sums[0][wave][lane] = sq; sums[1][wave][lane] = sk; }
        __syncthreads();
    }
    const f32x2* turn = p.rot ? p.turn + (int64_t)p.tok_pos[t] * (p.rot >> 1) : nullptr;
    const bool whole8 = (p.rot >> 1) % 8 == 0 && p.dim % 8 == 0;      // a lane's eight channels turn, and pair, as one
    for (int h = wave; h < p.H + p.G; h += 16) {
        const bool is_q = h < p.H;
        const float* x = head_x(h);
        const float* w = is_q ? p.q_norm : p.k_norm;
        float inv = 1.f;
        if (p.qk_norm == 1) inv = 1.0f / sqrtf(squares(x) / (float)p.dim + p.eps);
        else if (p.qk_norm == 2) {
            float s = 0.f;
#pragma unroll
            for (int i = 0; i < 16; i++) s += sums[!is_q][i][lane & 15];
            inv = 1.0f / sqrtf(s / ((float)p.dim * (is_q ? p.H : p.G)) + p.eps);
            w += (int64_t)(is_q ? h : h - p.H) * p.dim;
        }
        int krow = 0;
        bf16_t* dst = is_q ? (bf16_t*)p.q_out : grouped_key_row<bf16_t>(p, t, h - p.H, krow);
        for (int b = 0; b < p.dp; b += 32) {
            const int c = b + c0, half = p.rot >> 1;
            float v[8];
            if (whole8) {
                auto take = [&](int i, float (&y)[8]) {       // eight normed channels
                    const f32x4 u0 = *(const f32x4*)(x - c0 + i), u1 = *(const f32x4*)(x - c0 + i + 4);
#pragma unroll
                    for (int r = 0; r < 8; r++) { y[r] = r < 4 ? u0[r] : u1[r - 4]; if (p.qk_norm) y[r] *= inv * w[i + r]; }
                };
                if (c >= p.dim) {
#pragma unroll
                    for (int r = 0; r < 8; r++) v[r] = 0.f;
                } else {
                    take(c, v);
                    if (c < p.rot) {
                        float y[8];
                        take(c < half ? c + half : c - half, y);
                        const f32x2* cs = turn + (c < half ? c : c - half);
#pragma unroll
                        for (int r = 0; r < 8; r++) v[r] = c < half ? v[r] * cs[r][0] - y[r] * cs[r][1] : v[r] * cs[r][0] + y[r] * cs[r][1];
                    }
                }
            } else {
#pragma unroll
                for (int r = 0; r < 8; r++) v[r] = grouped_turn(p, x - c0, p.qk_norm ? w : nullptr, inv, turn, c + r);
            }
            bf16x8 out;
#pragma unroll
            for (int r = 0; r < 8; r++) out[r] = (bf16_t)v[r];
            if (!ok) continue;
            if (is_q) *(bf16x8*)(dst + fm_index(t, (int64_t)h * p.dp + c, p.q_ld)) = out;
            else *(bf16x8*)(dst + fm_index(krow, c, p.dp)) = out;
        }
    }
}

// The same with the heads in registers (a wave's up to HPW heads of 32 NB channels, all of them turning): one pass over the fp32 rows.
template <int NB, int HPW>
__global__ __launch_bounds__(1024) void grouped_qk_regs_kernel(GroupedArgs p) {
    __shared__ float sums[2][16][16];                 // [q, k][wave][token]
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), heads = p.H + p.G;
    const int tok = blockIdx.x * 16 + (lane & 15), c0 = (lane >> 4) * 8;
    const bool ok = tok < p.rows;
    const int64_t t = ok ? tok : p.rows - 1;
    const float* row = p.proj + t * p.proj_ld + c0;
    float x[HPW][NB][8], ss[HPW];
#pragma unroll
    for (int j = 0; j < HPW; j++) {
        const int h = wave + 16 * j;
#pragma unroll
        for (int b = 0; b < NB; b++) {
            f32x4 u = f32x4{0.f, 0.f, 0.f, 0.f}, v = u;
            if (h < heads) {
                const float* src = row + (h < p.H ? (int64_t)h * p.dp : p.qk_koff + (int64_t)(h - p.H) * p.dp) + b * 32;
                u = *(const f32x4*)src; v = *(const f32x4*)(src + 4);
            }
#pragma unroll
            for (int r = 0; r < 4; r++) { x[j][b][r] = u[r]; x[j][b][4 + r] = v[r]; }
        }
        ss[j] = 0.f;
#pragma unroll
        for (int b = 0; b < NB; b++)
#pragma unroll
            for (int r = 0; r < 8; r++) ss[j] = fmaf(x[j][b][r], x[j][b][r], ss[j]);
        ss[j] += __shfl_xor(ss[j], 16, 64);
        ss[j] += __shfl_xor(ss[j], 32, 64);
    }
    if (p.qk_norm == 2) {
        float sq = 0.f, sk = 0.f;
#pragma unroll
        for (int j = 0; j < HPW; j++) (wave + 16 * j < p.H ? sq : sk) += ss[j];
        if (lane < 16) { sums[0][wave][lane] = sq; sums[1][wave][lane] = sk; }
        __syncthreads();
        sq = sk = 0.f;
#pragma unroll
        for (int i = 0; i < 16; i++) { sq += sums[0][i][lane & 15]; sk += sums[1][i][lane & 15]; }
#pragma unroll
        for (int j = 0; j < HPW; j++) ss[j] = wave + 16 * j < p.H ? sq / p.H : sk / p.G;
    }
    const f32x2* turn = p.turn + (int64_t)p.tok_pos[t] * (p.rot >> 1) + c0;
#pragma unroll
    for (int j = 0; j < HPW; j++) {
        const int h = wave + 16 * j;
        if (h >= heads) continue;
        const bool is_q = h < p.H;
        if (p.qk_norm) {
            const float inv = 1.0f / sqrtf(ss[j] / (float)p.dim + p.eps);
            const float* w = (is_q ? p.q_norm : p.k_norm) + (p.qk_norm == 2 ? (int64_t)(is_q ? h : h - p.H) * p.dim : 0) + c0;
#pragma unroll
            for (int b = 0; b < NB; b++) {
                const f32x4 u = *(const f32x4*)(w + b * 32), v = *(const f32x4*)(w + b * 32 + 4);
#pragma unroll
                for (int r = 0; r < 8; r++) x[j][b][r] *= inv * (r < 4 ? u[r] : v[r - 4]);
            }
        }
        int krow = 0;
        bf16_t* dst = is_q ? (bf16_t*)p.q_out : grouped_key_row<bf16_t>(p, t, h - p.H, krow);
#pragma unroll
        for (int b = 0; b < NB / 2; b++) {
            bf16x8 lo, hi;
#pragma unroll
            for (int r = 0; r < 8; r += 2) {
                const f32x4 cs = *(const f32x4*)(turn + b * 32 + r);         // (cos, sin) of two pairs
#pragma unroll
                for (int e = 0; e < 2; e++) {
                    const float u = x[j][b][r + e], v = x[j][b + NB / 2][r + e];
                    lo[r + e] = (bf16_t)(u * cs[2 * e] - v * cs[2 * e + 1]);
                    hi[r + e] = (bf16_t)(v * cs[2 * e] + u * cs[2 * e + 1]);
                }
            }
            if (!ok) continue;
            const int c = b * 32 + c0;
            if (is_q) { *(bf16x8*)(dst + fm_index(t, (int64_t)h * p.dp + c, p.q_ld)) = lo; *(bf16x8*)(dst + fm_index(t, (int64_t)h * p.dp + c + NB * 16, p.q_ld)) = hi; }
            else { *(bf16x8*)(dst + fm_index(krow, c, p.dp)) = lo; *(bf16x8*)(dst + fm_index(krow, c + NB * 16, p.dp)) = hi; }
        }
    }
}

// ---- scores in the exp2 domain ----
struct GroupedScore {       // constants of one query row
    float sc, c2, nr1, r2;
    bool cap, bias;
    __device__ __forceinline__ GroupedScore(const GroupedArgs& p, int head) {
        constexpr float L2E = 1.4426950408889634f;
        cap = p.softcap > 0.f; bias = p.r1 != nullptr;
        sc = cap ? p.scale / p.softcap * (2.0f * L2E) : p.scale * L2E;      // cap: exp2(s sc) = exp(2 s scale / softcap)
        c2 = -2.0f * p.softcap * L2E;                                       // softcap tanh(x) = softcap - 2 softcap / (exp(2 x) + 1); the softmax drops the first term
        nr1 = bias ? -p.r1[head] : 0.f; r2 = bias ? p.r2[head] : 0.f;       // r1 ln(.) log2(e) = r1 log2(.)
    }
};
// raw scores of one 64-key tile (tile-relative key 32 (t / 2) + 8 fg + 4 (t & 1) + r; `back`: the query's own place, tile-relative)
// tab: NULL, or the (negative) biases of this lane's keys in key order; FAST: capped, with a table that holds softcap - bias
template <bool FAST = false>
__device__ __forceinline__ void grouped_scores(const GroupedScore& f, f32x4 (&s)[4], int back, int fg, const float* tab = nullptr) {
    if constexpr (FAST) {
#pragma unroll
        for (int t = 0; t < 4; t++)
#pragma unroll
            for (int r = 0; r < 4; r++)
                s[t][r] = fmaf(f.c2, __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(s[t][r] * f.sc) + 1.0f), tab[32 * (t >> 1) + 4 * (t & 1) + r]);
        return;
    }
    if (f.cap) {
#pragma unroll
        for (int t = 0; t < 4; t++)
#pragma unroll
            for (int r = 0; r < 4; r++) s[t][r] = f.c2 * __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(s[t][r] * f.sc) + 1.0f);
    } else {
#pragma unroll
        for (int t = 0; t < 4; t++) s[t] *= f.sc;
    }
    if (tab) {
#pragma unroll
        for (int t = 0; t < 4; t++)
#pragma unroll
            for (int r = 0; r < 4; r++) s[t][r] += tab[32 * (t >> 1) + 4 * (t & 1) + r];
    } else if (f.bias) {
        const float b = fmaf(f.r2, (float)(back - 8 * fg), 1.0f);
#pragma unroll
        for (int t = 0; t < 4; t++)
#pragma unroll
            for (int r = 0; r < 4; r++) s[t][r] = fmaf(f.nr1, __builtin_amdgcn_logf(fmaf(-f.r2, (float)(32 * (t >> 1) + 4 * (t & 1) + r), b)), s[t][r]);
    }
}
// from, keep: the query's first key (KeyMask::lo) and the end of the kept tokens, tile-relative
__device__ __forceinline__ void grouped_mask(f32x4 (&s)[4], int back, int from, int keep, int fg) {
#pragma unroll
    for (int t = 0; t < 4; t++)
#pragma unroll
        for (int r = 0; r < 4; r++) {
            const int k = 32 * (t >> 1) + 8 * fg + 4 * (t & 1) + r;
            if (k > back || (k < from && k >= keep)) s[t][r] = -INFINITY;
        }
}
__device__ __forceinline__ bf16x8 grouped_load_q(const GroupedArgs& p, int64_t tok, int head, int ks, int fg) {
    return *(const bf16x8*)((const bf16_t*)p.q + fm_index(tok, (int64_t)head * p.dp + ks * 32 + fg * 8, p.q_ld));
}
// the sink's score in the exp2 domain
__device__ __forceinline__ float grouped_sink(const GroupedArgs& p, int head) { return p.sink ? p.sink[head] * 1.4426950408889634f : -INFINITY; }
// four channels of a finished row: gate, store
__device__ __forceinline__ void grouped_store(const GroupedArgs& p, int64_t tok, int head, int c, f32x4 v) {
    if (p.gate_col >= 0) {
        const bf16x4 g = *(const bf16x4*)((const bf16_t*)p.q + fm_index(tok, p.gate_col + (int64_t)head * p.vp + c, p.q_ld));
#pragma unroll
        for (int r = 0; r < 4; r++) v[r] *= lat_sigmoid((float)g[r]);
    }
    v *= p.out_scale;
    act_store4<bf16_t>((bf16_t*)p.out, tok, head * p.vp + c, p.out_ld, v);
}

template <int KS, int DT> constexpr int grouped_prefill_pieces() { return 4 * KS + 2 * DT; }       // 1-KiB operand blocks of a tile
template <int KS, int DT> constexpr int grouped_prefill_ring_bytes() { return 3 * ((grouped_prefill_pieces<KS, DT>() + 7) / 8 * 8) * 1024; }

// grid (G, sequences, 256-row tiles); dynamic LDS: the ring, (block, row) of every key tile the workgroup walks, and with p.table the
// distance biases of the group's heads: [head][GROUPED_TAB_PAD + span + GROUPED_TAB_PAD], falling distances, so that consecutive keys are
// consecutive.  A wave's tiles reach at most 31 rows + 63 keys beyond its rows' windows on either side: the padding.
constexpr int GROUPED_TAB_PAD = 96;
// (20 modulo 64: the heads of a group then read from different banks; never less than keys + 2 PAD)
__host__ __device__ __forceinline__ int grouped_tab_span(int keys) { return ((keys + 2 * GROUPED_TAB_PAD + 43) & ~63) + 20; }
// FAST: scores that the cap bounds from both sides and biases that only lower them, from the table.  Their exponentials are taken as
// they are: no running maximum, no rescaling.  (GROUPED_FAST_CAP: the sum of 2^20 weights stays finite; a query sees its own key, so a
// weight that underflows is below 2^-30 of the sum.)  The other modes share the other instance.
constexpr float GROUPED_FAST_CAP = 60.0f;
template <int KS, int DT, bool FAST>
__global__ __launch_bounds__(512, (KS <= 2 && DT <= 4) ? 4 : 2) void grouped_prefill_kernel(GroupedArgs p) {
    constexpr int TQ = 2, PIECES = grouped_prefill_pieces<KS, DT>(), PW = (PIECES + 7) / 8, TILE = PW * 8 * 1024, NBUF = 3;
    extern __shared__ __attribute__((aligned(16))) char grp_sm[];
    int2* stile = (int2*)(grp_sm + NBUF * TILE);
    // kv head fastest, query tile slowest and last first: the longest workgroups are dispatched first
    const int kvh = blockIdx.x, seq = blockIdx.y, qt = gridDim.z - 1 - blockIdx.z;
    const int R = p.seq_len[seq] * p.group;
    if (R <= p.short_rows || qt * 256 >= R) return;
    const int tok0 = p.seq_tok_start[seq], pos0 = p.seq_pos[seq];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int fq = lane & 15, fg = lane >> 4;
    // key tiles of the workgroup, and of this wave (rows w_row0 .. + 31)
    const int wg_first = pos0 + qt * 256 / p.group, wg_last = pos0 + (min(qt * 256 + 255, R - 1)) / p.group;
    const int t0 = p.mask.lo(wg_first) >> 6, n_kt = (wg_last >> 6) + 1;
    const int keep_kt = (p.mask.keep + 63) >> 6, n_pre = min(t0, keep_kt), n_tiles = n_pre + n_kt - t0;      // (tiles of kept tokens before the window's)
    auto tile_at = [&](int i) { return i < n_pre ? i : t0 + i - n_pre; };
    const int w_row0 = qt * 256 + wave * 32;
    const bool w_live = w_row0 < R;
    const int first = pos0 + min(w_row0, R - 1) / p.group, last = pos0 + min(w_row0 + 31, R - 1) / p.group;
    const int wt0 = w_live ? p.mask.lo(first) >> 6 : n_kt, wt1 = w_live ? (last >> 6) + 1 : 0;
    const int full_lo = p.mask.lo(last), full_hi = first;
    for (int i = tid; i < n_tiles; i += 512) {
        const int key = tile_at(i) * 64, bi = key / p.bs;
        stile[i] = make_int2(p.blk_table[(int64_t)seq * p.tbl_stride + bi], key - bi * p.bs);
    }
    auto row_of = [&](int i, bool& ok) { const int r = w_row0 + 16 * i + fq; ok = r < R; return ok ? r : R - 1; };
    bf16x8 qf[TQ][KS];
    int qpos[TQ], qlo[TQ];
    float r1v[TQ], r2v[TQ], m_run[TQ];
#pragma unroll
    for (int i = 0; i < TQ; i++) {
        bool ok;
        const int row = row_of(i, ok), si = row / p.group, head = kvh * p.group + row - si * p.group;
        qpos[i] = pos0 + si;
        qlo[i] = p.mask.lo(qpos[i]);
        m_run[i] = p.sink ? grouped_sink(p, head) : -1e30f;
#pragma unroll
        for (int ks = 0; ks < KS; ks++) qf[i][ks] = grouped_load_q(p, tok0 + si, head, ks, fg);
        const GroupedScore f(p, head);
        r1v[i] = f.nr1; r2v[i] = f.r2;
    }
    GroupedScore f(p, 0);
#pragma unroll
    for (int i = 0; i < TQ; i++) {
#pragma unroll
        for (int ks = 0; ks < KS; ks++) asm volatile("" : "+v"(qf[i][ks]));      // complete before the first DMA is issued (attn.h)
        asm volatile("" : "+v"(r1v[i]), "+v"(r2v[i]), "+v"(m_run[i]));
    }
    asm volatile("" : "+v"(f.nr1), "+v"(f.r2));
    // distances of visible keys: 0 .. dmax; entry x of a head's table belongs to distance dmax + PAD - x
    float* const tabs = (float*)(stile + p.table);            // (p.table: entries of stile)
    const int dmax = (p.mask.span() > 0 ? min(p.mask.span() - 1, wg_last) : wg_last), span = grouped_tab_span(dmax + 1);
    if (p.table)
        for (int h = 0; h < p.group; h++) {
            const float nr1 = -p.r1[kvh * p.group + h], r2 = p.r2[kvh * p.group + h], top = FAST ? p.softcap * 1.4426950408889634f : 0.f;
            for (int x = tid; x < span; x += 512) {
                const int d = dmax + GROUPED_TAB_PAD - x;
                tabs[h * span + x] = d > 0 ? fmaf(nr1, __builtin_amdgcn_logf(fmaf(r2, (float)d, 1.0f)), top) : top;
            }
        }
    __syncthreads();                      // stile (and the table) are visible
    const float* tab[TQ];
#pragma unroll
    for (int i = 0; i < TQ; i++) {
        bool ok;
        const int row = row_of(i, ok), h = row % p.group;
        tab[i] = FAST || p.table ? tabs + h * span + dmax + GROUPED_TAB_PAD - qpos[i] + 8 * fg : nullptr;      // + key = the key's entry
    }
    // LDS-DMA: wave w moves pieces w * PW .. of [K: 16-key tile, k-step | V^T: d, 32-key unit]; surplus pieces repeat the last one
    int64_t src[PW];
#pragma unroll
    for (int i = 0; i < PW; i++) {
        int pc = wave * PW + i;
        if (pc >= PIECES) pc = PIECES - 1;
        if (pc < 4 * KS) src[i] = (int64_t)kvh * p.bs * p.dp + pc * 512 + lane * 8;
        else {
            const int v = pc - 4 * KS;
            src[i] = (int64_t)p.G * p.bs * p.dp + (int64_t)kvh * p.bs * p.vp + ((int64_t)(v >> 1) * (p.bs >> 5) + (v & 1)) * 512 + lane * 8;
        }
    }
    const uint32_t smem_lds = (uint32_t)(size_t)(__attribute__((address_space(3))) char*)grp_sm;
    auto issue = [&](int it, int buf) {
        const int2 tl = stile[it];
        const int blk = __builtin_amdgcn_readfirstlane(tl.x), row = __builtin_amdgcn_readfirstlane(tl.y);
        const bf16_t* base = (const bf16_t*)p.cache + (int64_t)blk * p.block_stride;
        const uint32_t dst = smem_lds + buf * TILE + wave * (PW * 1024);
#pragma unroll
        for (int i = 0; i < PW; i++) {
            // a tile's 64 keys are 64 dp elements of the key blocks and two operand blocks of every value row
            const bool is_k = wave * PW + i < 4 * KS;
            const uint64_t a = (uint64_t)(base + src[i] + (int64_t)row * (is_k ? p.dp : 16));
            asm volatile("s_mov_b32 m0, %0\n\ts_nop 4\n\tglobal_load_lds_dwordx4 %1, off" ::"s"(dst + i * 1024), "v"(a) : "memory");
        }
    };
    f32x4 o[TQ][DT], lacc[TQ];
    const float l0 = p.sink ? 1.0f : 0.0f;                    // (the sink's own weight, relative to m_run)
#pragma unroll
    for (int i = 0; i < TQ; i++) {
        lacc[i] = f32x4{l0, l0, l0, l0};
#pragma unroll
        for (int d = 0; d < DT; d++) o[i][d] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    bf16x8 ones;
#pragma unroll
    for (int e = 0; e < 8; e++) ones[e] = (bf16_t)1.0f;
    issue(0, 0);
    if (1 < n_tiles) issue(1, 1);
    int buf = 0;
    for (int it = 0; it < n_tiles; it++) {
        if (it + 1 < n_tiles) wait_vm<PW>(); else wait_vm<0>();      // my pieces of this tile have landed
        __builtin_amdgcn_s_barrier();
        if (it + 2 < n_tiles) { int nb = buf + 2; if (nb >= NBUF) nb -= NBUF; issue(it + 2, nb); }
        const int kt = tile_at(it);
        const char* kimg = grp_sm + buf * TILE + lane * 16;
        const char* vimg = kimg + 4 * KS * 1024;
        buf = buf + 1 == NBUF ? 0 : buf + 1;
        if ((kt < wt0 && kt >= keep_kt) || kt >= wt1) continue;      // (wave-uniform)
        f32x4 s[TQ][4];
#pragma unroll
        for (int i = 0; i < TQ; i++)
#pragma unroll
            for (int t = 0; t < 4; t++) s[i][t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int t = 0; t < 4; t++)
#pragma unroll
            for (int ks = 0; ks < KS; ks++) {
                const bf16x8 kf = *(const bf16x8*)(kimg + (t * KS + ks) * 1024);
#pragma unroll
                for (int i = 0; i < TQ; i++) s[i][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[i][ks], s[i][t], 0, 0, 0);
            }
        const bool whole = (kt * 64 >= full_lo || kt * 64 + 63 < p.mask.keep) && kt * 64 + 63 <= full_hi;
#pragma unroll
        for (int i = 0; i < TQ; i++) {
            if constexpr (!FAST) { f.nr1 = r1v[i]; f.r2 = r2v[i]; }
            grouped_scores<FAST>(f, s[i], qpos[i] - kt * 64, fg, FAST || p.table ? tab[i] + kt * 64 : nullptr);
        }
        if (!whole)
#pragma unroll
            for (int i = 0; i < TQ; i++) grouped_mask(s[i], qpos[i] - kt * 64, qlo[i] - kt * 64, p.mask.keep - kt * 64, fg);
        if constexpr (!FAST) {
            float m_new[TQ];
            bool moved = false;
#pragma unroll
            for (int i = 0; i < TQ; i++) {
                m_new[i] = vmax2(m_run[i], rows_max(vmax16(s[i][0], s[i][1], s[i][2], s[i][3])));
                moved |= m_new[i] > m_run[i] + 8.0f;            // (weights up to 2^8 over the reference do no harm)
            }
            if (__any(moved)) {
#pragma unroll
                for (int i = 0; i < TQ; i++) {
                    const float alpha = __builtin_amdgcn_exp2f(m_run[i] - m_new[i]);
                    lacc[i] *= alpha;
#pragma unroll
                    for (int d = 0; d < DT; d++) o[i][d] *= alpha;
                    m_run[i] = m_new[i];
                }
            }
        }
#pragma unroll
        for (int i = 0; i < TQ; i++)
#pragma unroll
            for (int t = 0; t < 4; t++)
#pragma unroll
                for (int r = 0; r < 4; r++) s[i][t][r] = __builtin_amdgcn_exp2f(FAST ? s[i][t][r] : s[i][t][r] - m_run[i]);
#pragma unroll
        for (int u = 0; u < 2; u++) {
            bf16x8 pf[TQ];
#pragma unroll
            for (int i = 0; i < TQ; i++) {
                pf[i] = latent_pack_p(s[i][2 * u], s[i][2 * u + 1]);
                lacc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ones, pf[i], lacc[i], 0, 0, 0);      // denominators out of the same rounded weights
            }
#pragma unroll
            for (int d = 0; d < DT; d++) {
                const bf16x8 vf = *(const bf16x8*)(vimg + (2 * d + u) * 1024);
#pragma unroll
                for (int i = 0; i < TQ; i++) o[i][d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pf[i], o[i][d], 0, 0, 0);
            }
        }
    }
    if (!w_live) return;
#pragma unroll
    for (int i = 0; i < TQ; i++) {
        bool ok;
        const int row = row_of(i, ok), si = row / p.group, head = kvh * p.group + row - si * p.group;
        if (!ok) continue;
        const float inv = 1.0f / lacc[i][0];
#pragma unroll
        for (int d = 0; d < DT; d++) grouped_store(p, tok0 + si, head, 16 * d + 4 * fg, o[i][d] * inv);
    }
}

// grid (G x 16-row tiles, sequences, key splits).  Wave w of workgroup z takes the key tiles z NW + w, + NW gridDim.z, ...; operands
// come straight from the cache.  The waves' results are combined through LDS; with gridDim.z > 1 every workgroup leaves a partial
// record {O^T [DT][64 lanes] f32x4, (m, l)[16]} (the lanes of live rows) and the one that draws the last ticket combines them in z order.
constexpr int GROUPED_SPLITS = 16;          // most workgroups the keys of a row tile are split over
template <int DT> constexpr int grouped_part_floats() { return DT * 256 + 32; }
__device__ __forceinline__ void grouped_part_store2(float* p, float a, float b) {
    __hip_atomic_store((unsigned long long*)p, __builtin_bit_cast(unsigned long long, f32x2{a, b}), __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
}
__device__ __forceinline__ void grouped_part_store(float* p, f32x4 v) { grouped_part_store2(p, v[0], v[1]); grouped_part_store2(p + 2, v[2], v[3]); }
__device__ __forceinline__ void grouped_part_load2(const float* p, float& a, float& b) {
    const f32x2 v = __builtin_bit_cast(f32x2, __hip_atomic_load((const unsigned long long*)p, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT));
    a = v[0]; b = v[1];
}
__device__ __forceinline__ f32x4 grouped_part_load(const float* p) {
    float a, b, c, d;
    grouped_part_load2(p, a, b); grouped_part_load2(p + 2, c, d);
    return f32x4{a, b, c, d};
}
template <int KS, int DT, int NW>
__global__ __launch_bounds__(NW * 64) void grouped_short_kernel(GroupedArgs p) {
    extern __shared__ __attribute__((aligned(16))) char grp_sm[];       // [NW][DT][64] f32x4
    __shared__ float red_m[NW][16], red_l[NW][16];
    __shared__ int ticket;
    const int kvh = blockIdx.x % p.G, rt = blockIdx.x / p.G, seq = blockIdx.y;
    const int R = p.seq_len[seq] * p.group;
    if (R > p.short_rows || rt * 16 >= R) return;
    const int tok0 = p.seq_tok_start[seq], pos0 = p.seq_pos[seq];
    const int32_t* tbl = p.blk_table + (int64_t)seq * p.tbl_stride;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int fq = lane & 15, fg = lane >> 4;
    const bool ok = rt * 16 + fq < R;
    const int row = ok ? rt * 16 + fq : R - 1, si = row / p.group, head = kvh * p.group + row - si * p.group;
    const int first = pos0 + rt * 16 / p.group, last = pos0 + min(rt * 16 + 15, R - 1) / p.group, qpos = pos0 + si;
    const int t0 = p.mask.lo(first) >> 6, n_kt = (last >> 6) + 1, qlo = p.mask.lo(qpos);
    const int n_pre = min(t0, (p.mask.keep + 63) >> 6), n_tiles = n_pre + n_kt - t0;      // (tiles of kept tokens before the window's)
    const int full_lo = p.mask.lo(last), full_hi = first;
    const int64_t tok = tok0 + si;
    bf16x8 qf[KS], kf[4][KS], vf[DT][2];
#pragma unroll
    for (int ks = 0; ks < KS; ks++) qf[ks] = grouped_load_q(p, tok, head, ks, fg);
    const GroupedScore f(p, head);
    f32x4 o[DT];
#pragma unroll
    for (int d = 0; d < DT; d++) o[d] = f32x4{0.f, 0.f, 0.f, 0.f};
    float m = -1e30f, l = 0.f;
    const int64_t v_ld = p.bs >> 5;
    for (int it = blockIdx.z * NW + wave; it < n_tiles; it += NW * gridDim.z) {
        const int kt = it < n_pre ? it : t0 + it - n_pre;
        const int bi = kt * 64 / p.bs, r0 = kt * 64 - bi * p.bs;
        const bf16_t* base = (const bf16_t*)p.cache + (int64_t)__builtin_amdgcn_readfirstlane(tbl[bi]) * p.block_stride + lane * 8;
        const bf16_t* kp = base + ((int64_t)kvh * p.bs + r0) * p.dp;
        const bf16_t* vp = base + (int64_t)p.G * p.bs * p.dp + (int64_t)kvh * p.bs * p.vp + (r0 >> 5) * 512;
#pragma unroll
        for (int t = 0; t < 4; t++)
#pragma unroll
            for (int ks = 0; ks < KS; ks++) kf[t][ks] = *(const bf16x8*)(kp + (t * KS + ks) * 512);
#pragma unroll
        for (int d = 0; d < DT; d++)
#pragma unroll
            for (int u = 0; u < 2; u++) vf[d][u] = *(const bf16x8*)(vp + (d * v_ld + u) * 512);
        f32x4 s[4];
#pragma unroll
        for (int t = 0; t < 4; t++) {
            s[t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int ks = 0; ks < KS; ks++) s[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[t][ks], qf[ks], s[t], 0, 0, 0);
        }
        const int back = qpos - kt * 64;
        grouped_scores(f, s, back, fg);
        if (!((kt * 64 >= full_lo || kt * 64 + 63 < p.mask.keep) && kt * 64 + 63 <= full_hi)) grouped_mask(s, back, qlo - kt * 64, p.mask.keep - kt * 64, fg);
        float mx = -INFINITY;
#pragma unroll
        for (int t = 0; t < 4; t++)
#pragma unroll
            for (int r = 0; r < 4; r++) mx = fmaxf(mx, s[t][r]);
        const float mn = fmaxf(m, rows_max(mx)), alpha = __builtin_amdgcn_exp2f(m - mn);
        m = mn;
        l *= alpha;
#pragma unroll
        for (int t = 0; t < 4; t++)
#pragma unroll
            for (int r = 0; r < 4; r++) { s[t][r] = __builtin_amdgcn_exp2f(s[t][r] - mn); l += s[t][r]; }
        const bf16x8 p0 = latent_pack_p(s[0], s[1]), p1 = latent_pack_p(s[2], s[3]);
#pragma unroll
        for (int d = 0; d < DT; d++) {
            o[d] *= alpha;
            o[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[d][0], p0, o[d], 0, 0, 0);
            o[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[d][1], p1, o[d], 0, 0, 0);
        }
    }
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    if (fg == 0) { red_m[wave][fq] = m; red_l[wave][fq] = l; }
    f32x4* po = (f32x4*)grp_sm;
#pragma unroll
    for (int d = 0; d < DT; d++) po[(wave * DT + d) * 64 + lane] = o[d];
    __syncthreads();
    float ms = red_m[0][fq], L = 0.f, sc[NW];
#pragma unroll
    for (int w = 1; w < NW; w++) ms = fmaxf(ms, red_m[w][fq]);
#pragma unroll
    for (int w = 0; w < NW; w++) { sc[w] = __builtin_amdgcn_exp2f(red_m[w][fq] - ms); L += red_l[w][fq] * sc[w]; }      // (a wave without a tile: l = 0, O = 0)
    const int nz = gridDim.z, pair = seq * gridDim.x + blockIdx.x;
    const float sink = grouped_sink(p, head);
    if (nz == 1 && p.sink) L += __builtin_amdgcn_exp2f(sink - ms);       // (a sink far above every score: inf, and the row is zero)
    float* rec = p.part + ((int64_t)pair * nz + blockIdx.z) * grouped_part_floats<DT>();
    for (int d = wave; d < DT; d += NW) {
        f32x4 a = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int w = 0; w < NW; w++) a += po[(w * DT + d) * 64 + lane] * sc[w];
        if (!ok) continue;
        if (nz > 1) grouped_part_store(rec + (d * 64 + lane) * 4, a);
        else grouped_store(p, tok, head, 16 * d + 4 * fg, a * (1.0f / L));
    }
    if (nz == 1) return;
    if (wave == 0 && fg == 0 && ok) grouped_part_store2(rec + DT * 256 + 2 * fq, ms, L);
    // Partial results go past the L2 of this XCD (agent-scope stores) and are read past the reader's, so no cache has to be written back
    // or invalidated: it is enough that they have arrived when the ticket is drawn.
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
    if (tid == 0) ticket = __hip_atomic_fetch_add(p.part_cnt + pair, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    __syncthreads();
    if (ticket != nz - 1) return;
    if (tid == 0) __hip_atomic_store(p.part_cnt + pair, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);      // for the next launch
    if (!ok) return;
    const float* rec0 = p.part + (int64_t)pair * nz * grouped_part_floats<DT>();
    float M = p.sink ? sink : -1e30f, LL = p.sink ? 1.0f : 0.f, mz[GROUPED_SPLITS];
#pragma unroll
    for (int z = 0; z < GROUPED_SPLITS; z++)
        if (z < nz) {
            float lz;
            grouped_part_load2(rec0 + (int64_t)z * grouped_part_floats<DT>() + DT * 256 + 2 * fq, mz[z], lz);
            const float mn = fmaxf(M, mz[z]);
            LL = LL * __builtin_amdgcn_exp2f(M - mn) + lz * __builtin_amdgcn_exp2f(mz[z] - mn);
            M = mn;
        }
    for (int d = wave; d < DT; d += NW) {
        f32x4 a = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int z = 0; z < GROUPED_SPLITS; z++)
            if (z < nz) a += grouped_part_load(rec0 + (int64_t)z * grouped_part_floats<DT>() + (d * 64 + lane) * 4) * __builtin_amdgcn_exp2f(mz[z] - M);
        grouped_store(p, tok, head, 16 * d + 4 * fg, a * (1.0f / LL));
    }
}

// ---- any size: one 256-thread workgroup per (token, head), online softmax over 256 keys at a time, plain fp32 arithmetic ----
template <typename T>
__global__ __launch_bounds__(256) void grouped_plain_kernel(GroupedArgs p) {
    __shared__ float red[4], sp[256];
    extern __shared__ __attribute__((aligned(16))) float grp_f[];      // q [dp] | o [vp]
    const int seq = blockIdx.z, h = blockIdx.y, r = blockIdx.x, tid = threadIdx.x, kvh = h / p.group;
    if (r >= p.seq_len[seq]) return;
    constexpr bool FM = sizeof(T) == 2;
    const int64_t t = p.seq_tok_start[seq] + r;
    const int pos = p.seq_pos[seq] + r, lo = p.mask.lo(pos), n_pre = min(lo, p.mask.keep), n_keys = n_pre + pos - lo + 1;
    auto key_at = [&](int i) { return i < n_pre ? i : lo + i - n_pre; };
    const int32_t* tbl = p.blk_table + (int64_t)seq * p.tbl_stride;
    float *sq = grp_f, *so = grp_f + p.dp;
    for (int i = tid; i < p.dp; i += 256) sq[i] = (float)((const T*)p.q)[act_index<T>(t, h * p.dp + i, p.q_ld)];
    for (int i = tid; i < p.vp; i += 256) so[i] = 0.f;
    const float r1 = p.r1 ? p.r1[h] : 0.f, r2 = p.r1 ? p.r2[h] : 0.f;
    float m = p.sink ? p.sink[h] : -1e30f, l = p.sink ? 1.f : 0.f;
    __syncthreads();
    auto bmax = [&](float v) { v = wave_max(v); if ((tid & 63) == 0) red[tid >> 6] = v; __syncthreads(); v = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])); __syncthreads(); return v; };
    auto bsum = [&](float v) { v = wave_sum(v); if ((tid & 63) == 0) red[tid >> 6] = v; __syncthreads(); v = red[0] + red[1] + red[2] + red[3]; __syncthreads(); return v; };
    auto part = [&](int key, int& row) { const int bi = key / p.bs; row = key - bi * p.bs; return (const T*)p.cache + (int64_t)tbl[bi] * p.block_stride; };
    for (int base = 0; base < n_keys; base += 256) {
        const bool live = base + tid < n_keys;
        const int key = key_at(base + tid);
        float s = -INFINITY;
        if (live) {
            int row;
            const T* k = part(key, row) + (int64_t)kvh * p.bs * p.dp;
            if (FM) row = grouped_k_row(row);
            float a = 0.f;
            for (int d = 0; d < p.dim; d++) a = fmaf(sq[d], (float)k[act_index<T>(row, d, p.dp)], a);
            s = a * p.scale;
            if (p.softcap > 0.f) s = p.softcap * tanhf(s / p.softcap);
            if (p.r1) s -= r1 * log1pf(r2 * (float)(pos - key));
        }
        const float mn = fmaxf(m, bmax(s)), alpha = expf(m - mn);
        const float e = live ? expf(s - mn) : 0.f;
        m = mn;
        l = l * alpha + bsum(e);
        sp[tid] = e;
        __syncthreads();
        const int nk = min(256, n_keys - base);
        for (int i = tid; i < p.vp; i += 256) {
            float a = so[i] * alpha;
            for (int j = 0; j < nk; j++) {
                int row;
                const T* v = part(key_at(base + j), row) + (int64_t)p.G * p.bs * p.dp + (int64_t)kvh * p.bs * p.vp;
                a = fmaf(sp[j], (float)(FM ? v[fm_index(i, row, p.bs)] : v[(int64_t)row * p.vp + i]), a);
            }
            so[i] = a;
        }
        __syncthreads();
    }
    for (int i = tid; i < p.vp; i += 256) {
        float o = so[i] / l * p.out_scale;
        if (p.gate_col >= 0) o *= 1.0f / (1.0f + expf(-(float)((const T*)p.q)[act_index<T>(t, p.gate_col + h * p.vp + i, p.q_ld)]));
        ActIO<T>::st((T*)p.out + act_index<T>(t, h * p.vp + i, p.out_ld), o);
    }
}

// launches (grouped_inst.hip): the instance follows from p.dp and p.vp
void grouped_prefill_launch(hipStream_t st, const GroupedArgs& p, dim3 grid, size_t lds, bool fast);
void grouped_short_launch(hipStream_t st, const GroupedArgs& p, dim3 grid);
void grouped_qk_launch(hipStream_t st, const GroupedArgs& p, bool f32);
constexpr int GROUPED_QK_ROW_MAX = 512;           // bf16: larger batches are worked in tiles of 16 tokens

}  // namespace nvl
