// Generic tile family: epilogues with a bias or a GELU.
#include "gemm_tiles.h"

int gemm_tiles_act_dispatch(int epi, int tile_cfg, DLI_GEMM_ARGS) {
  switch (epi) {
    case EPI_BIAS_GELU: return dispatch_tiles<EPI_BIAS_GELU>(tile_cfg, DLI_GEMM_PASS);
    case EPI_BIAS: return dispatch_tiles<EPI_BIAS>(tile_cfg, DLI_GEMM_PASS);
    case EPI_GELU_ERF: return dispatch_tiles<EPI_GELU_ERF>(tile_cfg, DLI_GEMM_PASS);
    default: return DLI_NOT_MINE;
  }
}

int gemm_tiles_act_set_slab_store(int mode) { return set_slab_store_tu(mode); }
