// grouped_inst.hip — the instances of the grouped-query attention kernels (grouped.h) and their launches.  NVL_GROUPED_INST: the prefill
// kernel's operand blocks of a query/key head (1, 2, 4, 8), or 0 for everything else, so that a build runs them side by side.
#ifndef NVL_GROUPED_INST
#error "NVL_GROUPED_INST: 0, 1, 2, 4 or 8"
#endif
#include "grouped.h"

namespace nvl {
template <int KS> void grouped_prefill_ks(hipStream_t st, const GroupedArgs& p, dim3 grid, size_t lds, bool fast);

#if NVL_GROUPED_INST > 0
template <int KS, int DT, bool FAST>
static void prefill(hipStream_t st, const GroupedArgs& p, dim3 grid, size_t lds) {
    NVL_LDS_ATTR((grouped_prefill_kernel<KS, DT, FAST>), 160 * 1024);
    hipLaunchKernelGGL((grouped_prefill_kernel<KS, DT, FAST>), grid, dim3(512), lds, st, p);
}
template <int KS> void grouped_prefill_ks(hipStream_t st, const GroupedArgs& p, dim3 grid, size_t lds, bool fast) {
#define NVL_GP(DTv) do { if (fast) prefill<KS, DTv, true>(st, p, grid, lds); else prefill<KS, DTv, false>(st, p, grid, lds); } while (0)
    const int dt = p.vp >> 4;
    if (dt == 2) NVL_GP(2); else if (dt == 4) NVL_GP(4);
    else if constexpr (KS == 8) NVL_GP(8);        // (256 x 256 has no room for its ring of tiles)
    else if (dt == 8) NVL_GP(8); else NVL_GP(16);
#undef NVL_GP
}
template void grouped_prefill_ks<NVL_GROUPED_INST>(hipStream_t, const GroupedArgs&, dim3, size_t, bool);
#else
void grouped_prefill_launch(hipStream_t st, const GroupedArgs& p, dim3 grid, size_t lds, bool fast) {
    switch (p.dp >> 5) {
        case 1: grouped_prefill_ks<1>(st, p, grid, lds, fast); break;
        case 2: grouped_prefill_ks<2>(st, p, grid, lds, fast); break;
        case 4: grouped_prefill_ks<4>(st, p, grid, lds, fast); break;
        default: grouped_prefill_ks<8>(st, p, grid, lds, fast);
    }
}
template <int KS, int DT>
static void run_short(hipStream_t st, const GroupedArgs& p, dim3 grid) {
    constexpr int nw = DT <= 8 ? 8 : 4;
    NVL_LDS_ATTR((grouped_short_kernel<KS, DT, nw>), nw * DT * 1024);
    hipLaunchKernelGGL((grouped_short_kernel<KS, DT, nw>), grid, dim3(nw * 64), nw * DT * 1024, st, p);
}
template <int KS>
static void run_short_ks(hipStream_t st, const GroupedArgs& p, dim3 grid) {
    switch (p.vp >> 4) {
        case 2: run_short<KS, 2>(st, p, grid); break;
        case 4: run_short<KS, 4>(st, p, grid); break;
        case 8: run_short<KS, 8>(st, p, grid); break;
        default: run_short<KS, 16>(st, p, grid);
    }
}
template <int NB>
static bool qk_regs(hipStream_t st, const GroupedArgs& p) {
    const dim3 grid(cdiv(p.rows, 16)), block(1024);
    switch (cdiv(p.H + p.G, 16)) {
        case 1: hipLaunchKernelGGL((grouped_qk_regs_kernel<NB, 1>), grid, block, 0, st, p); return true;
        case 2: hipLaunchKernelGGL((grouped_qk_regs_kernel<NB, 2>), grid, block, 0, st, p); return true;
        case 3: hipLaunchKernelGGL((grouped_qk_regs_kernel<NB, 3>), grid, block, 0, st, p); return true;
        default: return false;
    }
}
void grouped_qk_launch(hipStream_t st, const GroupedArgs& p, bool f32) {
    const dim3 waves(cdiv((int64_t)p.rows * (p.H + p.G), 4));
    if (f32) hipLaunchKernelGGL((grouped_qk_row_kernel<float>), waves, dim3(256), 0, st, p);
    else if (p.rows <= GROUPED_QK_ROW_MAX) hipLaunchKernelGGL((grouped_qk_row_kernel<bf16_t>), waves, dim3(256), 0, st, p);
    else if (p.dim == p.dp && p.rot == p.dp && ((p.dp == 64 && qk_regs<2>(st, p)) || (p.dp == 128 && qk_regs<4>(st, p)))) return;
    else hipLaunchKernelGGL(grouped_qk_tile_kernel, dim3(cdiv(p.rows, 16)), dim3(1024), 0, st, p);
}
void grouped_short_launch(hipStream_t st, const GroupedArgs& p, dim3 grid) {
    switch (p.dp >> 5) {
        case 1: run_short_ks<1>(st, p, grid); break;
        case 2: run_short_ks<2>(st, p, grid); break;
        case 4: run_short_ks<4>(st, p, grid); break;
        default: run_short_ks<8>(st, p, grid);
    }
}
#endif
}  // namespace nvl
