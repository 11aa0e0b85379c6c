// latent_inst.hip — the instances of the latent attention kernels (latent.h) and their launches.
#include <stdexcept>
#include "latent.h"

namespace nvl {
template <int KS, int DT>
static void prefill(hipStream_t st, const LatentArgs& p, dim3 grid) {
    constexpr int lds = latent_prefill_lds_bytes<KS, DT>();
    NVL_LDS_ATTR((latent_prefill_kernel<KS, DT>), lds);
    hipLaunchKernelGGL((latent_prefill_kernel<KS, DT>), grid, dim3(512), lds, st, p);
}
template <int KS>
static void prefill_ks(hipStream_t st, const LatentArgs& p, dim3 grid) {
    if (p.vp == 32) prefill<KS, 2>(st, p, grid); else if (p.vp == 64) prefill<KS, 4>(st, p, grid);
    else if constexpr (KS > 4) prefill<KS, 8>(st, p, grid);
    else if (p.vp == 128) prefill<KS, 8>(st, p, grid); else prefill<KS, 16>(st, p, grid);
}
void latent_prefill_launch(hipStream_t st, const LatentArgs& p, int n_seqs, int max_len) {
    const dim3 grid(p.H, n_seqs, cdiv(max_len, 256));
    if (p.dp == 256 && p.vp == 256) hipLaunchKernelGGL((latent_prefill_wide_kernel<8, 16>), dim3(p.H, n_seqs, cdiv(max_len, 64)), dim3(256), 0, st, p);
    else switch (p.dp) {
        case 32: prefill_ks<1>(st, p, grid); break;
        case 64: prefill_ks<2>(st, p, grid); break;
        case 96: prefill_ks<3>(st, p, grid); break;
        case 128: prefill_ks<4>(st, p, grid); break;
        case 192: prefill_ks<6>(st, p, grid); break;
        default: prefill_ks<8>(st, p, grid);
    }
}
template <int NR, int KR>
static void decode(hipStream_t st, const LatentArgs& p, dim3 grid) {
    constexpr int lds = latent_decode_lds_bytes<NR>();
    NVL_LDS_ATTR((latent_decode_kernel<NR, KR>), lds);
    hipLaunchKernelGGL((latent_decode_kernel<NR, KR>), grid, dim3(256), lds, st, p);
}
template <int NR>
static void decode_nr(hipStream_t st, const LatentArgs& p, dim3 grid) {
    if (p.rotp == 0) decode<NR, 0>(st, p, grid); else if (p.rotp == 32) decode<NR, 1>(st, p, grid);
    else if (p.rotp == 64) decode<NR, 2>(st, p, grid); else decode<NR, 4>(st, p, grid);
}
void latent_decode_launch(hipStream_t st, const LatentArgs& p, dim3 grid) {
    switch (p.rp / 64) {
        case 1: decode_nr<1>(st, p, grid); break; case 2: decode_nr<2>(st, p, grid); break; case 3: decode_nr<3>(st, p, grid); break;
        case 4: decode_nr<4>(st, p, grid); break; case 6: decode_nr<6>(st, p, grid); break; case 8: decode_nr<8>(st, p, grid); break;
        default: throw std::runtime_error("latent attention: no absorbed instance for this latent size");
    }
}
}  // namespace nvl
