// Generic tile family: epilogues that pair a gate block with the up block beside it.
#include "gemm_tiles.h"

int gemm_tiles_pairs_dispatch(int epi, int tile_cfg, DLI_GEMM_ARGS) {
  switch (epi) {
    case EPI_SILU: return dispatch_tiles<EPI_SILU>(tile_cfg, DLI_GEMM_PASS);
    case EPI_CLAMP: return dispatch_tiles<EPI_CLAMP>(tile_cfg, DLI_GEMM_PASS);
    case EPI_RELU: return dispatch_tiles<EPI_RELU>(tile_cfg, DLI_GEMM_PASS);
    default: return DLI_NOT_MINE;
  }
}

int gemm_tiles_pairs_set_slab_store(int mode) { return set_slab_store_tu(mode); }
