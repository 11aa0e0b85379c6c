// delta_inst.hip — the instances of the channel-wise delta rule's kernels (delta.h) and their launches.
#include "delta.h"

namespace nvl {
template <bool FUSED, int ROWS, typename ActT>
static void step(hipStream_t st, const DeltaArgs& p, dim3 grid, int lds) {
    NVL_LDS_ATTR((delta_step_kernel<FUSED, ROWS, ActT>), 128 * 1024);
    hipLaunchKernelGGL((delta_step_kernel<FUSED, ROWS, ActT>), grid, dim3(LR_STEP_THREADS), lds, st, p);
}
template <bool FUSED, typename ActT>
static void step_rows(hipStream_t st, const DeltaArgs& p, int n_seqs) {
    const int lds = delta_step_lds_bytes(p.DK, p.DVp, FUSED ? p.a_rkp + p.g_rkp : 0);
    const dim3 grid(p.H, n_seqs);
    int tv = 1;
    while (tv < p.DVp / 4) tv <<= 1;
    const int rows = cdiv(p.DK, LR_STEP_THREADS / tv);        // state rows per thread
    if (rows <= 4) step<FUSED, 4, ActT>(st, p, grid, lds); else if (rows <= 8) step<FUSED, 8, ActT>(st, p, grid, lds); else step<FUSED, 16, ActT>(st, p, grid, lds);
    NVL_HIP(hipGetLastError());
}
void delta_step_launch(hipStream_t st, const DeltaArgs& p, int n_seqs, bool fused, bool f32) {
    if (!fused) step_rows<false, float>(st, p, n_seqs);
    else if (f32) step_rows<true, float>(st, p, n_seqs);
    else step_rows<true, bf16_t>(st, p, n_seqs);
}
template <int NK>
static void prep(hipStream_t st, const DeltaArgs& p, dim3 grid) {
    constexpr int lds = delta_prep_lds_bytes<NK>();
    NVL_LDS_ATTR((delta_prep_kernel<NK>), lds);
    hipLaunchKernelGGL((delta_prep_kernel<NK>), grid, dim3(512), lds, st, p);
}
void delta_prep_launch(hipStream_t st, const DeltaArgs& p, dim3 grid, int nk) {
    if (nk == 2) prep<2>(st, p, grid); else if (nk == 4) prep<4>(st, p, grid); else if (nk == 8) prep<8>(st, p, grid); else prep<16>(st, p, grid);
}
template <int NK, int NW, int KSP>
static void scan(hipStream_t st, const DeltaArgs& p, int n_seqs) {
    constexpr int lds = delta_scan_lds_bytes<NK, NW, KSP>();
    NVL_LDS_ATTR((delta_scan_kernel<NK, NW, KSP>), lds);
    hipLaunchKernelGGL((delta_scan_kernel<NK, NW, KSP>), dim3(p.H, n_seqs, cdiv(p.DV, 16 * NW / KSP)), dim3(NW * 64), lds, st, p);
}
// columns per workgroup, and with few of them the key channels split over the waves too
template <int NK, int LOW>
static void scan_shape(hipStream_t st, const DeltaArgs& p, int n_seqs) {
    const int pairs = p.H * n_seqs;
    if (pairs * cdiv(p.DV, 64) < 128) scan<NK, 4, LOW>(st, p, n_seqs);
    else if (p.DV <= 64 || pairs * cdiv(p.DV, 128) < 256) scan<NK, 4, 1>(st, p, n_seqs);
    else scan<NK, 8, 1>(st, p, n_seqs);
}
void delta_scan_launch(hipStream_t st, const DeltaArgs& p, int n_seqs, int nk) {
    if (nk == 2) scan<2, 4, 1>(st, p, n_seqs);
    else if (nk == 4) scan_shape<4, 2>(st, p, n_seqs); else if (nk == 8) scan_shape<8, 4>(st, p, n_seqs); else scan_shape<16, 4>(st, p, n_seqs);
}
}  // namespace nvl
