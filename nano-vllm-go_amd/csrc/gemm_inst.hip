// gemm_inst.hip — the projection kernels (gemm.h) of one epilogue: compiled once per value of NVL_GEMM_INST (0 fp32 mode, else
// 1 + GemmEpi), so that a build runs them side by side.
#ifndef NVL_GEMM_INST
#error "NVL_GEMM_INST: 0, or 1 + an epilogue"
#endif
#include "gemm.h"

namespace nvl {
#if NVL_GEMM_INST == 0
#define NVL_X(E) template void launch_gemm_f32<E, float>(hipStream_t, const GemmArgs&);
NVL_GEMM_F32_INSTANCES(NVL_X)
#elif NVL_GEMM_INST == 1
template void launch_gemm_bf16<EPI_STORE, float>(hipStream_t, const GemmArgs&);
template void launch_gemm_bf16<EPI_STORE, bf16_t>(hipStream_t, const GemmArgs&);
#else
constexpr int INST = NVL_GEMM_INST - 1;
using InstT = std::conditional_t<INST == EPI_RESID, float, bf16_t>;
template void launch_gemm_bf16<INST, InstT>(hipStream_t, const GemmArgs&);
#endif
}  // namespace nvl
