// linrec_inst.hip — the instances of the linear recurrences' kernels (linrec.h) and their launches.  NVL_LINREC_INST: 1 the chunk kernel
// with one decay per head, 2 with a decay per key channel, 0 everything else, so that a build runs them side by side.
#ifndef NVL_LINREC_INST
#error "NVL_LINREC_INST: 0, 1 or 2"
#endif
#include "linrec.h"

namespace nvl {
template <bool CH> void linrec_chunk_ch(hipStream_t st, const LinRecArgs& p, int n_seqs, int nk, int nw, bool par);

#if NVL_LINREC_INST > 0
template <int NK, int NW, bool CH, int MODE>
static void chunk(hipStream_t st, const LinRecArgs& p, int n_seqs) {
    NVL_LDS_ATTR((linrec_chunk_kernel<NK, NW, CH, MODE>), 160 * 1024);
    hipLaunchKernelGGL((linrec_chunk_kernel<NK, NW, CH, MODE>), dim3(p.H, n_seqs, p.n_slices * (MODE ? p.n_super : 1)), dim3(NW * 64),
                       (linrec_chunk_lds_bytes<NK, NW, CH>(p.rank)), st, p);
}
template <int NK, int NW, bool CH>
static void chunk_modes(hipStream_t st, const LinRecArgs& p, int n_seqs, bool par) {
    if (!par) { chunk<NK, NW, CH, 0>(st, p, n_seqs); return; }
    chunk<NK, NW, CH, 1>(st, p, n_seqs);
    hipLaunchKernelGGL((linrec_prefix_kernel<CH>), dim3(p.H, n_seqs, cdiv((int64_t)p.DK * p.DVp, 1024)), dim3(256), 0, st, p);
    chunk<NK, NW, CH, 2>(st, p, n_seqs);
}
template <bool CH> void linrec_chunk_ch(hipStream_t st, const LinRecArgs& p, int n_seqs, int nk, int nw, bool par) {
#define NVL_LC(NKv) do { if (nw == 4) chunk_modes<NKv, 4, CH>(st, p, n_seqs, par); else chunk_modes<NKv, 8, CH>(st, p, n_seqs, par); } while (0)
    if (nk == 2) NVL_LC(2); else if (nk == 4) NVL_LC(4); else if (nk == 8) NVL_LC(8); else NVL_LC(16);
#undef NVL_LC
}
template void linrec_chunk_ch<NVL_LINREC_INST == 2>(hipStream_t, const LinRecArgs&, int, int, int, bool);
#else
void linrec_chunk_launch(hipStream_t st, const LinRecArgs& p, int n_seqs, bool ch, int nk, int nw, bool par) {
    if (ch) linrec_chunk_ch<true>(st, p, n_seqs, nk, nw, par); else linrec_chunk_ch<false>(st, p, n_seqs, nk, nw, par);
}
template <int KIND, typename ActT>
static void step(hipStream_t st, const LinRecArgs& p, int n_seqs) {
    int tv = 1;
    while (tv < p.DVp / 4) tv <<= 1;
    const int rows = cdiv(p.DK, LR_STEP_THREADS / tv), lds = linrec_step_lds_bytes(p.DK, p.DVp);        // rows: state rows per thread
    const dim3 grid(p.H, n_seqs);
    if (rows <= 4) hipLaunchKernelGGL((linrec_step_kernel<KIND, 4, ActT>), grid, dim3(LR_STEP_THREADS), lds, st, p);
    else if (rows <= 8) hipLaunchKernelGGL((linrec_step_kernel<KIND, 8, ActT>), grid, dim3(LR_STEP_THREADS), lds, st, p);
    else hipLaunchKernelGGL((linrec_step_kernel<KIND, 16, ActT>), grid, dim3(LR_STEP_THREADS), lds, st, p);
    NVL_HIP(hipGetLastError());
}
void linrec_step_launch(hipStream_t st, const LinRecArgs& p, int n_seqs, bool ch, bool fused, bool f32) {
    if (!fused) { if (ch) step<1, float>(st, p, n_seqs); else step<0, float>(st, p, n_seqs); }
    else if (f32) { if (ch) step<3, float>(st, p, n_seqs); else step<2, float>(st, p, n_seqs); }
    else { if (ch) step<3, bf16_t>(st, p, n_seqs); else step<2, bf16_t>(st, p, n_seqs); }
}
#endif
}  // namespace nvl
