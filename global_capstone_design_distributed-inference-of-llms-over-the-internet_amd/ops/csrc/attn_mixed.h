// Shared by the kernels of head-mixing attention (attention_mixed.hip, attention_mixed_mfma.hip): arguments and the layout of
// a cache page.
#pragma once
#include "common.h"
#include "act_io.h"

namespace mp {

struct MixedArgs {
  const void* z;         // [T, zs] projected rows
  int64_t zs;
  void* qn;              // [T, H D] q'
  const float *qg, *kg;  // [D] gains
  const float* talk;     // [H, H]
  const float* rope;     // [positions, rot] cosines, then sines
  const float* vrope;    // [positions, V]
  void* cache;           // [pages, G, page (D + V)]
  const int64_t* slots;
  const int32_t* bt;
  int bt_stride;
  const int32_t *q_seq, *q_ctx;
  void* out;             // row-major [T, os] or packed
  int64_t os;
  int H, G, D, V, rot, page_log2, packed_mt;
  float scale, cap, eps;
};

// element offset of value column v of key ``off`` of a page, after the page's key rows
__device__ __forceinline__ int64_t val_at(int off, int v, int V, int blk_log2) {
  return ((int64_t)(off >> blk_log2) * V + v) * (1 << blk_log2) + (off & ((1 << blk_log2) - 1));
}
__device__ __forceinline__ int val_block_log2(int page_log2) { return min(page_log2, 5); }

}  // namespace mp
