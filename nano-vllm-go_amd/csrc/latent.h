// latent.h — attention over a cached low-rank latent (multi-head latent attention), with an optional sliding window and an optional
// rotated part.  Per token: c_q = rms(W_dq h) * w, q = W_uq c_q; c = rms(W_dkv h) * w; per head k = W_uk c, v = W_uv c; only c is
// cached.  The concatenated heads are multiplied by sigmoid(W_g h) (per channel or per head) before the output projection.
// Rotated part (rot > 0): every head of q has `rot` more dimensions, turned by the token's position; their key is ONE vector per
// token, shared by the heads, turned before it is cached beside c; the two scores add up.
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
// kv_rank padded to 64, and after them [bs][rotp] rotated keys, rotp = rot padded to 32 (the padding is zero).  A layer may read
// another layer's part (it then has no W_dkv).  bf16: fragment-major in units of 16 tokens x 32 columns (common.h fm_index on the
// block's rows), so that a score operand is one contiguous KiB; fp32 mode: row-major.
#pragma once
#include "attn.h"
#include "common.h"

namespace nvl {

constexpr int LAT_SPLITS = 16;          // most workgroups the keys of a token are split over (absorbed form)
__device__ __forceinline__ float lat_sigmoid(float x) { return 1.0f / (1.0f + __expf(-x)); }

struct LatentArgs {
    int H, dim, dn, dp, vp, qrank, qrp, kvrank, rp;   // dn / vp / qrp / rp: padded sizes; dp = dn + rotp: a head's columns of q
    int rot, rotp;                                // rotated dimensions per head (0: none), padded
    const f32x2* turn;                            // [position][rot / 2] (cos, sin)
    int turn_q;                                   // whoever reads q turns it (16 | rot); else latent_turn_q_kernel has done it
    int window;                                   // 0: every earlier token
    float scale, eps;
    const float* proj; int64_t proj_ld;           // [token][c_q : qrp | c : rp | rotated key : rotp | gate] of the fused input projection
    int own;                                      // the layer makes its own latents (else: no c and rotated key columns)
    int gate_off, gate_head;                      // first gate column; one gate per head instead of one per channel
    const float *cq_norm, *c_norm;                // padded with zeros
    void* cq;                                     // operand of W_uq: [token][qrp]
    void* cache; int64_t block_stride;            // this layer's part of block 0; elements between blocks
    int bs;
    const int32_t *blk_table, *tok_pos, *tok_tbl, *seq_tok_start, *seq_len, *seq_pos;
    int tbl_stride;
    const float* q; int64_t q_ld;                 // [token][H * dp], per head [unrotated : dn | to be rotated : rotp]
    // expanded form
    const int32_t* kbase;                         // per sequence: its first row in the key workspace (-1: the sequence takes the absorbed form)
    void *cg, *kr;                                // gathered latents [rows][rp] and rotated keys [rows][rotp]
    const void *kx, *vx;                          // bf16: K [rows][H * dn] and V^T [H * vp][rows_pad], both fragment-major; fp32: K, V [rows][H * .]
    int64_t rows_pad;
    void* out; int64_t out_ld;                    // operand of W_o: [token][out_ld], head h at column h * vp
    // absorbed form
    const int32_t* abs_tok;                       // the tokens that take it
    const int32_t* abs_seq;
    int n_abs, n_split;
    const bf16_t *ukt, *uv;                       // per head [rp][dn]; [H * vp][rp]; fragment-major
    bf16_t* qa; int Hp;                           // [n_abs][Hp][rp + rotp], Hp = H padded to 16
    float *part_o, *part_ml;                      // [split][n_abs][H][rp], [split][n_abs][H][2]
};

// first key the earliest token of a call can see, rounded down to the 32-row unit the gather copies
__host__ __device__ __forceinline__ int latent_key0(int pos0, int window) {
    const int lo = window > 0 ? pos0 - window + 1 : 0;
    return lo > 0 ? (lo & ~31) : 0;
}

// dimension i of a vector of `rot` dimensions turned by position pos: pairs (i, i + rot / 2)
__device__ __forceinline__ float lat_turn(const LatentArgs& p, const float* x, int i, int pos) {
    const int half = p.rot >> 1;
    if (i >= p.rot) return 0.f;
    const int j = i < half ? i : i - half;
    const f32x2 cs = p.turn[(int64_t)pos * half + j];
    const float u = x[j], v = x[j + half];
    return i < half ? u * cs[0] - v * cs[1] : v * cs[0] + u * cs[1];
}
__device__ __forceinline__ float lat_gate(const LatentArgs& p, int64_t tok, int h, int col) {      // col: column of W_o's operand inside head h
    return p.proj[tok * p.proj_ld + p.gate_off + (p.gate_head ? h : h * p.vp + col)];
}
__device__ __forceinline__ f32x4 lat_gate4(const LatentArgs& p, int64_t tok, int h, int col) {
    if (!p.gate_head) return *(const f32x4*)(p.proj + tok * p.proj_ld + p.gate_off + h * p.vp + col);
    const float g = lat_gate(p, tok, h, col);
    return f32x4{g, g, g, g};
}

// ---- norms of the two latents; c goes to its cache row.  grid (tokens), 256 threads ----
template <typename ActT>
__global__ __launch_bounds__(256) void latent_norm_kernel(LatentArgs p) {
    __shared__ float red[8];
    const int t = blockIdx.x;
    const float* pr = p.proj + (int64_t)t * p.proj_ld;
    float sq = 0.f, sc = 0.f;          // (the padding columns of c_q and c are zero)
    for (int i = threadIdx.x * 4; i < p.qrp; i += 1024) { const f32x4 v = *(const f32x4*)(pr + i); sq += (v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3]); }
    if (p.own) for (int i = threadIdx.x * 4; i < p.rp; i += 1024) { const f32x4 v = *(const f32x4*)(pr + p.qrp + i); sc += (v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3]); }
    sq = wave_sum(sq); sc = wave_sum(sc);
    if ((threadIdx.x & 63) == 0) { red[threadIdx.x >> 6] = sq; red[4 + (threadIdx.x >> 6)] = sc; }
    __syncthreads();
    const float rq = sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)p.qrank + p.eps), rc = sqrtf((red[4] + red[5] + red[6] + red[7]) / (float)p.kvrank + p.eps);
    for (int i = threadIdx.x * 4; i < p.qrp; i += 1024) act_store4<ActT>((ActT*)p.cq, t, i, p.qrp, *(const f32x4*)(pr + i) / rq * *(const f32x4*)(p.cq_norm + i));
    if (!p.own) return;
    int blk, row;
    const int pos = p.tok_pos[t];
    kv_locate(p.blk_table, p.tok_tbl[t], pos, p.bs, blk, row);
    ActT* c = (ActT*)p.cache + (int64_t)blk * p.block_stride;
    for (int i = threadIdx.x * 4; i < p.rp; i += 1024) act_store4<ActT>(c, row, i, p.rp, *(const f32x4*)(pr + p.qrp + i) / rc * *(const f32x4*)(p.c_norm + i));
    ActT* kr = c + (int64_t)p.bs * p.rp;
    for (int i = threadIdx.x; i < p.rotp; i += 256) ActIO<ActT>::st(kr + act_index<ActT>(row, i, p.rotp), lat_turn(p, pr + p.qrp + p.rp, i, pos));
}

// ---- q's rotated part in place, for sizes its readers do not turn themselves: grid (tokens, heads) ----
static __global__ __launch_bounds__(64) void latent_turn_q_kernel(LatentArgs p) {
    const int64_t t = blockIdx.x;
    float* q = (float*)p.q + t * p.q_ld + (int64_t)blockIdx.y * p.dp + p.dn;
    const int half = p.rot >> 1;
    for (int i = threadIdx.x; i < half; i += 64) {
        const f32x2 cs = p.turn[(int64_t)p.tok_pos[t] * half + i];
        const float u = q[i], v = q[i + half];
        q[i] = u * cs[0] - v * cs[1];
        q[i + half] = v * cs[0] + u * cs[1];
    }
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
    if (!p.rot) return;
    const char* rs = (const char*)((const ActT*)p.cache + (int64_t)blk * p.block_stride + (int64_t)p.bs * p.rp + (int64_t)row * p.rotp);
    char* rd = (char*)((ActT*)p.kr + (int64_t)(p.kbase[seq] + r0) * p.rotp);
    for (int i = threadIdx.x * 16; i < 32 * p.rotp * (int)sizeof(ActT); i += 256 * 16) *(f32x4*)(rd + i) = *(const f32x4*)(rs + i);
}

// ------------------------------------------------------------------------------------------
// expanded form, bf16.  S^T = K Q^T and O^T += V^T P^T as in attn.h; 32 query rows of one head per wave.  K and V^T come
// fragment-major from memory; the K rows of a 32-key unit are taken in the order that makes the score accumulators
// (keys 8 fg + r, 8 fg + 4 + r) the B operand against V^T's natural key order.
//   latent_prefill_kernel      : 8 waves (256 query rows) share 64-key tiles of K and V^T through a 3-slot LDS ring filled by LDS-DMA two
//                                tiles ahead, one barrier per tile; a tile is a set of 1-KiB operand blocks, so the image is
//                                lane-linear and every fragment read conflict-free (the K row order is chosen by the DMA's source)
//   latent_prefill_wide_kernel : 4 waves, operands straight from memory (heads of 256 x 256: three slots would not fit LDS)
// A negative scale is moved onto the queries, so that the row maximum can be taken before scaling; zero: latent_plain_kernel.
// ------------------------------------------------------------------------------------------
struct LatentRows {            // the query rows of one wave
    int tok0, pos0, n, k0, row0, first, last;
    __device__ __forceinline__ LatentRows(const LatentArgs& p, int seq, int row0_) {
        n = p.seq_len[seq]; tok0 = p.seq_tok_start[seq]; pos0 = p.seq_pos[seq]; k0 = latent_key0(pos0, p.window); row0 = row0_;
        first = pos0 + row0; last = pos0 + min(row0 + 31, n - 1);
    }
    __device__ __forceinline__ int row(int i, int fq, bool& ok) const { const int r = row0 + 16 * i + fq; ok = r < n; return ok ? r : n - 1; }
    __device__ __forceinline__ int key_lo(const LatentArgs& p) const { const int lo = p.window > 0 ? first - p.window + 1 : 0; return lo > k0 ? lo - k0 : 0; }
};
template <int KS>
__device__ __forceinline__ void latent_load_q(const LatentArgs& p, int64_t tok, int pos, int h, int fg, bf16x8 (&qf)[KS]) {
    const float* qp = p.q + tok * p.q_ld + h * p.dp;
    const float sg = p.scale < 0.f ? -1.f : 1.f;
#pragma unroll
    for (int ks = 0; ks < KS; ks++) {
        f32x4 a = *(const f32x4*)(qp + ks * 32 + fg * 8), b = *(const f32x4*)(qp + ks * 32 + fg * 8 + 4);
        const int j = ks * 32 - p.dn + fg * 8, half = p.rot >> 1;
        if (p.turn_q && j >= 0 && j < p.rot) {      // eight dimensions on one side of the pairs (16 | rot)
            const bool lo = j < half;
            const float* other = qp + p.dn + (lo ? j + half : j - half);
            const float* cs = (const float*)(p.turn + (int64_t)pos * half + (lo ? j : j - half));
            const float sn = lo ? -1.f : 1.f;
#pragma unroll
            for (int e = 0; e < 4; e += 2) {
                const f32x4 c0 = *(const f32x4*)(cs + 2 * e), c1 = *(const f32x4*)(cs + 2 * e + 8);
                const f32x2 o0 = *(const f32x2*)(other + e), o1 = *(const f32x2*)(other + e + 4);
                a[e] = fmaf(o0[0] * sn, c0[1], a[e] * c0[0]); a[e + 1] = fmaf(o0[1] * sn, c0[3], a[e + 1] * c0[2]);
                b[e] = fmaf(o1[0] * sn, c1[1], b[e] * c1[0]); b[e + 1] = fmaf(o1[1] * sn, c1[3], b[e + 1] * c1[2]);
            }
        }
#pragma unroll
        for (int e = 0; e < 4; e++) { qf[ks][e] = (bf16_t)(a[e] * sg); qf[ks][4 + e] = (bf16_t)(b[e] * sg); }
    }
}
// this lane's K row inside a 32-key unit for score tile t
__device__ __forceinline__ int latent_k_row(int t, int fq) { return 8 * (fq >> 2) + (fq & 3) + 4 * (t & 1); }
// scores of one 64-key tile (tile-relative key 32 (t / 2) + 8 fg + 4 (t & 1) + r) -> weights, running maximum and rescale
template <int DT>
__device__ __forceinline__ void latent_softmax(f32x4 (&s)[4], bool whole, int back, int window, int fg, float sl2, float& m_run, f32x4& lacc, f32x4 (&o)[DT]) {
    if (!whole) {
        const int from = window > 0 ? back - window + 1 : 0;
#pragma unroll
        for (int t = 0; t < 4; t++)
#pragma unroll
            for (int r = 0; r < 4; r++) {
                const int k = 32 * (t >> 1) + 8 * fg + 4 * (t & 1) + r;
                if (k > back || k < from) s[t][r] = -INFINITY;
            }
    }
    const float m_new = vmax2(m_run, rows_max(vmax16(s[0], s[1], s[2], s[3])) * sl2);
    if (__any(m_new != m_run)) {
        const float alpha = __builtin_amdgcn_exp2f(m_run - m_new);
        lacc *= alpha;
#pragma unroll
        for (int d = 0; d < DT; d++) o[d] *= alpha;
        m_run = m_new;
    }
#pragma unroll
    for (int t = 0; t < 4; t++)
#pragma unroll
        for (int r = 0; r < 4; r++) s[t][r] = __builtin_amdgcn_exp2f(fmaf(s[t][r], sl2, -m_run));
}
__device__ __forceinline__ bf16x8 latent_pack_p(const f32x4& a, const f32x4& b) {
    bf16x8 p;
#pragma unroll
    for (int r = 0; r < 4; r++) { p[r] = (bf16_t)a[r]; p[4 + r] = (bf16_t)b[r]; }
    return p;
}
template <int DT>
__device__ __forceinline__ void latent_store_o(const LatentArgs& p, int64_t tok, int h, int fg, float inv, const f32x4 (&o)[DT]) {
#pragma unroll
    for (int d = 0; d < DT; d++) {
        const f32x4 g = lat_gate4(p, tok, h, 16 * d + 4 * fg);
        f32x4 v = o[d] * inv;
#pragma unroll
        for (int r = 0; r < 4; r++) v[r] *= lat_sigmoid(g[r]);
        act_store4<bf16_t>((bf16_t*)p.out, tok, h * p.vp + 16 * d + 4 * fg, p.out_ld, v);
    }
}

template <int KS, int DT> constexpr int latent_prefill_pieces() { return 4 * KS + 2 * DT; }       // 1-KiB blocks of a tile
template <int KS, int DT> constexpr int latent_prefill_lds_bytes() { return 3 * ((latent_prefill_pieces<KS, DT>() + 7) / 8 * 8) * 1024; }
template <int N> __device__ __forceinline__ void wait_vm() { asm volatile("s_waitcnt vmcnt(%0)" ::"n"(N) : "memory"); }

template <int KS, int DT>
__global__ __launch_bounds__(512, (KS <= 2 && DT <= 4) ? 4 : 2) void latent_prefill_kernel(LatentArgs p) {
    constexpr int TQ = 2, PIECES = latent_prefill_pieces<KS, DT>(), PW = (PIECES + 7) / 8, TILE = PW * 8 * 1024, NBUF = 3;
    extern __shared__ __attribute__((aligned(16))) char lat_smc[];
    // head fastest, query tile slowest and last first: the longest workgroups are dispatched first
    const int h = blockIdx.x, seq = blockIdx.y, qt = gridDim.z - 1 - blockIdx.z;
    if (qt * 256 >= p.seq_len[seq] || p.kbase[seq] < 0) return;
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int fq = lane & 15, fg = lane >> 4;
    const LatentRows w(p, seq, qt * 256 + wave * 32);
    const bool w_live = w.row0 < w.n;
    bf16x8 qf[TQ][KS];
    int qpos[TQ];
#pragma unroll
    for (int i = 0; i < TQ; i++) {
        bool ok;
        const int r = w.row(i, fq, ok);
        qpos[i] = w.pos0 + r;
        latent_load_q<KS>(p, w.tok0 + r, qpos[i], h, fg, qf[i]);
    }
#pragma unroll
    for (int i = 0; i < TQ; i++)
#pragma unroll
        for (int ks = 0; ks < KS; ks++) asm volatile("" : "+v"(qf[i][ks]));      // complete before the first DMA is issued (attn.h)
    // workspace-relative keys: the workgroup's tiles, and the part of them this wave's rows can see
    const LatentRows wg(p, seq, qt * 256);
    const int kb = p.kbase[seq];
    const int wg_last = wg.pos0 + min(qt * 256 + 255, wg.n - 1) - wg.k0;
    const int t0 = wg.key_lo(p) >> 6, n_kt = (wg_last >> 6) + 1;
    const int wt0 = w_live ? w.key_lo(p) >> 6 : n_kt, wt1 = w_live ? ((w.last - w.k0) >> 6) + 1 : 0;
    const int full_lo = (p.window > 0 ? w.last - p.window + 1 : 0) - w.k0, full_hi = w.first - w.k0;
    // LDS-DMA: wave w moves pieces w * PW .. of [K: tile t, k-step | V^T: d, 32-key unit]; surplus pieces repeat the last one
    const int64_t k_ld = (int64_t)(p.H * p.dn >> 5), r_ld = p.rotp >> 5, v_ld = p.rows_pad >> 5;
    const int ksn = p.dn >> 5;                                // k-steps of the heads' own keys; the shared rotated keys follow
    const bf16_t* src[PW];
    int64_t step[PW];
#pragma unroll
    for (int i = 0; i < PW; i++) {
        int pc = wave * PW + i;
        if (pc >= PIECES) pc = PIECES - 1;
        if (pc < 4 * KS) {
            const int t = pc / KS, ks = pc - t * KS, key = kb + 32 * (t >> 1) + latent_k_row(t, fq);
            const bool rk = ks >= ksn;
            const int64_t ld = rk ? r_ld : k_ld;
            src[i] = (const bf16_t*)(rk ? p.kr : p.kx) + (((int64_t)(key >> 4) * ld + (rk ? ks - ksn : h * ksn + ks)) * 64 + (key & 15) + 16 * fg) * 8;
            step[i] = 4 * ld * 512;
        } else {
            const int v = pc - 4 * KS, d = v >> 1, u = v & 1;
            src[i] = (const bf16_t*)p.vx + (((int64_t)(h * DT + d) * v_ld + (kb >> 5) + u) * 64 + lane) * 8;
            step[i] = 2 * 512;
        }
    }
    const uint32_t smem_lds = (uint32_t)(size_t)(__attribute__((address_space(3))) char*)lat_smc;
    auto issue = [&](int kt, int buf) {
        const uint32_t dst = smem_lds + buf * TILE + wave * (PW * 1024);
#pragma unroll
        for (int i = 0; i < PW; i++) {
            const uint64_t a = (uint64_t)(src[i] + (int64_t)kt * step[i]);
            asm volatile("s_mov_b32 m0, %0\n\ts_nop 4\n\tglobal_load_lds_dwordx4 %1, off" ::"s"(dst + i * 1024), "v"(a) : "memory");
        }
    };
    f32x4 o[TQ][DT], lacc[TQ];
    float m_run[TQ];
#pragma unroll
    for (int i = 0; i < TQ; i++) {
        m_run[i] = -1e30f; lacc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int d = 0; d < DT; d++) o[i][d] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    bf16x8 ones;
#pragma unroll
    for (int e = 0; e < 8; e++) ones[e] = (bf16_t)1.0f;
    const float sl2 = fabsf(p.scale) * 1.4426950408889634f;
    issue(t0, 0);
    if (t0 + 1 < n_kt) issue(t0 + 1, 1);
    int buf = 0;
    for (int kt = t0; kt < n_kt; kt++) {
        if (kt + 1 < n_kt) wait_vm<PW>(); else wait_vm<0>();      // my pieces of tile kt have landed
        __builtin_amdgcn_s_barrier();
        if (kt + 2 < n_kt) { int nb = buf + 2; if (nb >= NBUF) nb -= NBUF; issue(kt + 2, nb); }
        const char* kimg = lat_smc + buf * TILE + lane * 16;
        const char* vimg = kimg + 4 * KS * 1024;
        buf = buf + 1 == NBUF ? 0 : buf + 1;
        if (kt < wt0 || kt >= wt1) continue;                      // (wave-uniform)
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
        const bool whole = kt * 64 >= full_lo && kt * 64 + 63 <= full_hi;
#pragma unroll
        for (int i = 0; i < TQ; i++) latent_softmax<DT>(s[i], whole, qpos[i] - w.k0 - kt * 64, p.window, fg, sl2, m_run[i], lacc[i], o[i]);
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
        const int r = w.row(i, fq, ok);
        if (ok) latent_store_o<DT>(p, w.tok0 + r, h, fg, 1.0f / lacc[i][0], o[i]);
    }
}

template <int KS, int DT>
__global__ __launch_bounds__(256) void latent_prefill_wide_kernel(LatentArgs p) {
    constexpr int TQ = 1;
    const int h = blockIdx.x, seq = blockIdx.y, qt = gridDim.z - 1 - blockIdx.z;
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int fq = lane & 15, fg = lane >> 4;
    const int row0 = qt * 64 + wave * 16;
    if (row0 >= p.seq_len[seq] || p.kbase[seq] < 0) return;      // (no barrier in this kernel)
    const LatentRows w(p, seq, row0);
    const int last = w.pos0 + min(row0 + 15, w.n - 1);
    bool ok;
    const int r0 = w.row(0, fq, ok), qpos = w.pos0 + r0;
    bf16x8 qf[KS];
    latent_load_q<KS>(p, w.tok0 + r0, qpos, h, fg, qf);
    const int kb = p.kbase[seq], j1 = last - w.k0;
    const int full_lo = (p.window > 0 ? last - p.window + 1 : 0) - w.k0, full_hi = w.first - w.k0;
    const int64_t k_ld = (int64_t)(p.H * p.dn >> 5), r_ld = p.rotp >> 5, v_ld = p.rows_pad >> 5;
    const int ksn = p.dn >> 5;
    f32x4 o[DT], lacc = f32x4{0.f, 0.f, 0.f, 0.f};
    float m_run = -1e30f;
#pragma unroll
    for (int d = 0; d < DT; d++) o[d] = f32x4{0.f, 0.f, 0.f, 0.f};
    bf16x8 ones;
#pragma unroll
    for (int e = 0; e < 8; e++) ones[e] = (bf16_t)1.0f;
    const float sl2 = fabsf(p.scale) * 1.4426950408889634f;
    for (int j = w.key_lo(p) & ~63; j <= j1; j += 64) {
        f32x4 s[4];
#pragma unroll
        for (int t = 0; t < 4; t++) {
            s[t] = f32x4{0.f, 0.f, 0.f, 0.f};
            const int key = kb + j + 32 * (t >> 1) + latent_k_row(t, fq);
            const int64_t lo = ((key & 15) + 16 * fg) * 8;
            const bf16_t* kn = (const bf16_t*)p.kx + ((int64_t)(key >> 4) * k_ld + h * ksn) * 512 + lo;
            const bf16_t* kr = (const bf16_t*)p.kr + ((int64_t)(key >> 4) * r_ld - ksn) * 512 + lo;
#pragma unroll
            for (int ks = 0; ks < KS; ks++) s[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*(const bf16x8*)((ks < ksn ? kn : kr) + ks * 512), qf[ks], s[t], 0, 0, 0);
        }
        latent_softmax<DT>(s, j >= full_lo && j + 63 <= full_hi, qpos - w.k0 - j, p.window, fg, sl2, m_run, lacc, o);
#pragma unroll
        for (int u = 0; u < 2; u++) {
            const bf16x8 pf = latent_pack_p(s[2 * u], s[2 * u + 1]);
            lacc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ones, pf, lacc, 0, 0, 0);
            const bf16_t* vr = (const bf16_t*)p.vx + (((int64_t)(h * DT) * v_ld + ((kb + j) >> 5) + u) * 64 + lane) * 8;
#pragma unroll
            for (int d = 0; d < DT; d++) o[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*(const bf16x8*)(vr + (int64_t)d * v_ld * 512), pf, o[d], 0, 0, 0);
        }
    }
    if (ok) latent_store_o<DT>(p, w.tok0 + r0, h, fg, 1.0f / lacc[0], o);
}

// ---- expanded form, any size: one 256-thread workgroup per (token, head), online softmax over 256 keys at a time, plain fp32
// arithmetic.  The fp32 mode's kernel, and the bf16 mode's for heads wider than the instances above. ----
template <typename T>
__device__ __forceinline__ float lat_k(const LatentArgs& p, int64_t row, int64_t col) { return ((const T*)p.kx)[act_index<T>(row, col, (int64_t)p.H * p.dn)]; }
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
    for (int i = tid; i < p.dp; i += 256) {
        const float* qh = p.q + t * p.q_ld + h * p.dp;
        sq[i] = i < p.dn || !p.turn_q ? qh[i] : lat_turn(p, qh + p.dn, i - p.dn, pos);
    }
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
            for (int d = 0; d < p.dim; d++) a = fmaf(sq[d], lat_k<T>(p, row, h * p.dn + d), a);
            for (int d = 0; d < p.rot; d++) a = fmaf(sq[p.dn + d], (float)((const T*)p.kr)[act_index<T>(row, d, p.rotp)], a);
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
        const float g = lat_gate(p, t, h, i);
        ActIO<T>::st((T*)p.out + act_index<T>(t, h * p.vp + i, p.out_ld), so[i] / l * (1.0f / (1.0f + expf(-g))));
    }
}

// ------------------------------------------------------------------------------------------
// absorbed form (bf16)
// ------------------------------------------------------------------------------------------
// q'[token][head][:] = W_uk[head]^T q[token][head]: grid (H, rp / 64 (+ 1: the rotated part), ceil(n_abs / 16)), one 16-column tile per
// wave, K = dn
static __global__ __launch_bounds__(256) void latent_absorb_q_kernel(LatentArgs p) {
    const int h = blockIdx.x, nt = blockIdx.y * 4 + (threadIdx.x >> 6), mt = blockIdx.z, lane = threadIdx.x & 63;
    const int fr = lane & 15, fg = lane >> 4, nks = p.dn >> 5;
    const int64_t rt = p.rp + p.rotp;
    if (nt * 16 >= p.rp) {                                    // (workgroup-uniform: 64 | rp)
        for (int e = threadIdx.x; e < 16 * p.rotp; e += 256) {
            const int j = mt * 16 + e / p.rotp, d = e % p.rotp;
            if (j >= p.n_abs) break;
            const int64_t t = p.abs_tok[j];
            const float* qr = p.q + t * p.q_ld + h * p.dp + p.dn;
            p.qa[((int64_t)j * p.Hp + h) * rt + p.rp + d] = (bf16_t)(p.turn_q ? lat_turn(p, qr, d, p.tok_pos[t]) : qr[d]);
        }
        return;
    }
    const int i = mt * 16 + fr;
    const bool ok = i < p.n_abs;
    const float* qp = ok ? p.q + (int64_t)p.abs_tok[i] * p.q_ld + h * p.dp + fg * 8 : nullptr;
    const bf16_t* w = p.ukt + (int64_t)h * p.rp * p.dn + ((int64_t)nt * nks * 64 + lane) * 8;
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
    *(bf16x4*)(p.qa + ((int64_t)i * p.Hp + h) * rt + nt * 16 + 4 * fg) = o;
}

// grid (ceil(H / 16), n_abs, n_split), 4 waves, 64 keys per step (inside one block: 64 | bs).  Wave w scores keys 16 w .. of the step
// (operand blocks straight from the cache, copied to an LDS image on the way), the waves agree on the maximum, exchange the
// weights through LDS, and wave w accumulates its rp / 4 latent columns over all 64 keys from the image by transposed reads.
// KR: 32-column steps of the rotated keys, which only the scores take.
template <int NR>                  // rp = 64 NR
constexpr int latent_decode_lds_bytes() { return 2 * 64 * NR * 64 * 2 + 16 * 16 * 8 + 2 * 4 * 16 * 4; }
template <int NR, int KR>
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
    bf16x8 qf[KSN + KR];
#pragma unroll
    for (int ks = 0; ks < KSN + KR; ks++) qf[ks] = *(const bf16x8*)(p.qa + ((int64_t)ia * p.Hp + ht * 16 + fq) * (NR * 64 + KR * 32) + ks * 32 + fg * 8);
    f32x4 o[NR];
#pragma unroll
    for (int i = 0; i < NR; i++) o[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    float m = -1e30f, l = 0.f;
    const float sl2 = p.scale * 1.4426950408889634f;
    const int tr_row = 4 * fg + (fq >> 2), tr_p = fq & 3;
    bf16x8 a[KSN + KR];
    auto fetch = [&](int kt) {
        const int key = kt * 64, bi = key / p.bs, row = key - bi * p.bs;
        const int blk = __builtin_amdgcn_readfirstlane(tbl[bi]);
        const bf16_t* b = (const bf16_t*)p.cache + (int64_t)blk * p.block_stride + lane * 8;
        const int64_t r16 = row + 16 * wave;
#pragma unroll
        for (int ks = 0; ks < KSN; ks++) a[ks] = *(const bf16x8*)(b + r16 * p.rp + ks * 512);
#pragma unroll
        for (int ks = 0; ks < KR; ks++) a[KSN + ks] = *(const bf16x8*)(b + (int64_t)p.bs * p.rp + r16 * (KR * 32) + ks * 512);
    };
    if (kt0 < kt1) fetch(kt0);
    for (int kt = kt0; kt < kt1; kt++) {
        char* img = lat_smc + ((kt - kt0) & 1) * IMG;
        f32x4 s = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < KSN; ks++) {
            s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[ks], qf[ks], s, 0, 0, 0);
            *(bf16x8*)(img + ((wave * KSN + ks) * 64 + lane) * 16) = a[ks];
        }
#pragma unroll
        for (int ks = KSN; ks < KSN + KR; ks++) s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[ks], qf[ks], s, 0, 0, 0);
        if (kt + 1 < kt1) fetch(kt + 1);
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

// combines the key splits, projects by W_uv and gates: grid (H, ceil(vp / 256), ceil(n_abs / 16)), 16 waves, one 16-column tile of V each.
// The combined latents of the 16 tokens are made once per workgroup (fragment-major bf16 in LDS) while the weight fragments are in flight.
static __global__ __launch_bounds__(1024) void latent_uv_kernel(LatentArgs p) {
    extern __shared__ __attribute__((aligned(16))) char lat_smc[];       // [rp / 32][64 lanes][16 B]
    __shared__ float sw[16][LAT_SPLITS];                                  // weight of a split's partial, 1 / L folded in
    const int h = blockIdx.x, vt = blockIdx.y * 16 + (threadIdx.x >> 6), mt = blockIdx.z, lane = threadIdx.x & 63;
    const int fr = lane & 15, fg = lane >> 4, nks = p.rp >> 5, tid = threadIdx.x;
    constexpr int MAXKS = 16;
    const bool v_live = vt * 16 < p.vp;
    bf16x8 wf[MAXKS];
    const bf16_t* w = p.uv + ((int64_t)(h * (p.vp >> 4) + vt) * nks * 64 + lane) * 8;
#pragma unroll
    for (int ks = 0; ks < MAXKS; ks++) { wf[ks] = bf16x8{}; if (v_live && ks < nks) wf[ks] = *(const bf16x8*)(w + ks * 512); }
    if (tid < 256) {
        const int i = mt * 16 + (tid >> 4), z = tid & 15;                 // 16 tokens x 16 splits
        float m = -1e30f, l = 0.f;
        if (i < p.n_abs && z < p.n_split) {
            const float* ml = p.part_ml + 2 * (((int64_t)z * p.n_abs + i) * p.H + h);
            m = ml[0]; l = ml[1];
        }
        float M = m;
#pragma unroll
        for (int o = 8; o > 0; o >>= 1) M = fmaxf(M, __shfl_xor(M, o, 16));
        const float e = __builtin_amdgcn_exp2f(m - M);
        float L = l * e;
#pragma unroll
        for (int o = 8; o > 0; o >>= 1) L += __shfl_xor(L, o, 16);
        sw[tid >> 4][z] = L > 0.f ? e / L : 0.f;
    }
    __syncthreads();
    for (int c = tid; c < 16 * (p.rp >> 2); c += 1024) {                   // 4 latent columns of one token
        const int r = c / (p.rp >> 2), col = (c - r * (p.rp >> 2)) * 4, i = mt * 16 + r;
        f32x4 a = f32x4{0.f, 0.f, 0.f, 0.f};
        if (i < p.n_abs)
#pragma unroll 8
            for (int z = 0; z < p.n_split; z++) a += sw[r][z] * *(const f32x4*)(p.part_o + (((int64_t)z * p.n_abs + i) * p.H + h) * p.rp + col);
        bf16x4 b;
#pragma unroll
        for (int e = 0; e < 4; e++) b[e] = (bf16_t)a[e];
        *(bf16x4*)(lat_smc + (((col >> 5) * 64 + r + 16 * ((col & 31) >> 3)) * 16 + 2 * (col & 7))) = b;
    }
    __syncthreads();
    const int i = mt * 16 + fr;
    if (!v_live) return;
    f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < MAXKS; ks++)
        if (ks < nks) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[ks], *(const bf16x8*)(lat_smc + (ks * 64 + lane) * 16), acc, 0, 0, 0);
    if (i >= p.n_abs) return;
    const int64_t t = p.abs_tok[i];
    const int col = h * p.vp + vt * 16 + 4 * fg;
    const f32x4 g = lat_gate4(p, t, h, vt * 16 + 4 * fg);
#pragma unroll
    for (int r = 0; r < 4; r++) acc[r] *= lat_sigmoid(g[r]);
    act_store4<bf16_t>((bf16_t*)p.out, t, col, p.out_ld, acc);
}

// launches (latent_inst.hip): the instance follows from the padded sizes
void latent_prefill_launch(hipStream_t st, const LatentArgs& p, int n_seqs, int max_len);
void latent_decode_launch(hipStream_t st, const LatentArgs& p, dim3 grid);

}  // namespace nvl
