// Launch templates of the paged-decode kernels (K3), shared by the translation units that instantiate them: one per group of
// head dims, so that they compile side by side.
#pragma once
#include "paged_decode_body.h"

struct DecodePlan {
  int g_chunk;  // q heads served per workgroup (template G)
  int n_chunks;
  int nload;
  int tile;
  int unit;
  int nsplit;
  bool uniform;
  bool mfma;  // tensor-core variant (paged_decode_mfma.hip)
  bool wide;  // vector kernel, TPL adjacent kv heads per workgroup (whole-row loads)
};

// head dim 256 (paged_decode_d256.hip)
int mv_paged_decode_launch_d256(const DecodeParams &p, const DecodePlan &pl, int batch, int dtype, int flags, hipStream_t stream);

namespace {

template <typename Tag, int D, int G, int NLOAD, bool ROPE>
void launch_gr(const DecodeParams &p, const DecodePlan &pl, int batch, hipStream_t stream) {
  dim3 block(256);
  if constexpr (G <= 4) {
    if (pl.wide) {
      dim3 grid(p.n_kv_heads / (64 / (D / elem<Tag>::VEC)), pl.nsplit, batch);
      if (pl.uniform)
        hipLaunchKernelGGL((paged_decode_kernel<Tag, D, G, NLOAD, true, true, ROPE>), grid, block, 0, stream, p);
      else
        hipLaunchKernelGGL((paged_decode_kernel<Tag, D, G, NLOAD, false, true, ROPE>), grid, block, 0, stream, p);
      return;
    }
  }
  dim3 grid(p.n_kv_heads * pl.n_chunks, pl.nsplit, batch);
  if (pl.uniform)
    hipLaunchKernelGGL((paged_decode_kernel<Tag, D, G, NLOAD, true, false, ROPE>), grid, block, 0, stream, p);
  else
    hipLaunchKernelGGL((paged_decode_kernel<Tag, D, G, NLOAD, false, false, ROPE>), grid, block, 0, stream, p);
}

template <typename Tag, int D, int G, int NLOAD>
void launch_g(const DecodeParams &p, const DecodePlan &pl, int batch, hipStream_t stream) {
  if constexpr (elem<Tag>::VEC == 8 && G <= 4) {   // (rope fusion: 16-bit dtypes, up to 4 query heads per kv head)
    if (p.positions != nullptr) return launch_gr<Tag, D, G, NLOAD, true>(p, pl, batch, stream);
  }
  launch_gr<Tag, D, G, NLOAD, false>(p, pl, batch, stream);
}

template <typename Tag, int D>
int launch_d(const DecodeParams &p, const DecodePlan &pl, int batch, int dtype, int flags, hipStream_t stream) {
  if constexpr (D == 128)
  if (pl.mfma) {
    const int klds = (flags & MV_DECODE_KLDS_ON) ? 1 : ((flags & MV_DECODE_KLDS_OFF) ? 0 : -1);
    const int rc = mv_paged_decode_mfma_launch(p, pl.n_chunks, pl.nsplit, batch, dtype, klds, stream);
    if (rc != MV_OK) return rc;
    if (pl.nsplit > 1) {
      hipLaunchKernelGGL((paged_decode_reduce_kernel<Tag, D>), dim3(batch * p.n_heads), dim3(128), 0,
                         stream, p.ws_acc, p.ws_ml, (typename elem<Tag>::T *)p.out, pl.nsplit, p.n_heads, p.out_stride,
                         p.mask);
      MV_LAUNCH_CHECK();
    }
    return MV_OK;
  }
  switch (pl.g_chunk) {
    case 1: launch_g<Tag, D, 1, 8>(p, pl, batch, stream); break;
    case 2: launch_g<Tag, D, 2, 8>(p, pl, batch, stream); break;
    case 3: launch_g<Tag, D, 3, 8>(p, pl, batch, stream); break;
    case 4: launch_g<Tag, D, 4, 8>(p, pl, batch, stream); break;
    case 5: launch_g<Tag, D, 5, 4>(p, pl, batch, stream); break;
    case 6: launch_g<Tag, D, 6, 4>(p, pl, batch, stream); break;
    case 7: launch_g<Tag, D, 7, 4>(p, pl, batch, stream); break;
    case 8: launch_g<Tag, D, 8, 4>(p, pl, batch, stream); break;
    default: return MV_E_SHAPE;
  }
  MV_LAUNCH_CHECK();
  if (pl.nsplit > 1) {
    hipLaunchKernelGGL((paged_decode_reduce_kernel<Tag, D>), dim3(batch * p.n_heads), dim3(128), 0,
                       stream, p.ws_acc, p.ws_ml, (typename elem<Tag>::T *)p.out, pl.nsplit, p.n_heads, p.out_stride,
                         p.mask);
    MV_LAUNCH_CHECK();
  }
  return MV_OK;
}

}  // namespace
