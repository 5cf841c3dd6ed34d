// Generic tile family: plain, fp32 and fp16-slab epilogues, and the family's dispatch.
#include "gemm_tiles.h"

int gemm_tiles_dispatch(int epi, int tile_cfg, DLI_GEMM_ARGS) {
  switch (epi) {
    case EPI_BF16: return dispatch_tiles<EPI_BF16>(tile_cfg, DLI_GEMM_PASS);
    case EPI_F32: return dispatch_tiles<EPI_F32>(tile_cfg, DLI_GEMM_PASS);
    case EPI_SLAB16:
      if (C != nullptr || splits < 2) return (int)hipErrorInvalidValue;
      return dispatch_tiles<EPI_SLAB16>(tile_cfg, DLI_GEMM_PASS);
    default: break;
  }
  if (epi_pairs(epi)) return gemm_tiles_pairs_dispatch(epi, tile_cfg, DLI_GEMM_PASS);
  return gemm_tiles_act_dispatch(epi, tile_cfg, DLI_GEMM_PASS);
}

int gemm_tiles_set_slab_store(int mode) {
  gemm_tiles_pairs_set_slab_store(mode);
  gemm_tiles_act_set_slab_store(mode);
  return set_slab_store_tu(mode);
}
