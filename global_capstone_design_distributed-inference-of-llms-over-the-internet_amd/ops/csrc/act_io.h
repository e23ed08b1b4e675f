// Loads and stores of activations in either element type (bf16 or fp32) as fp32 registers, and the
// two activation layouts a kernel may write: row-major, or packed for the decode GEMM (bf16 only).
#pragma once
#include "common.h"

namespace mp {

__device__ __forceinline__ float to_f(bf16_t v) { return bf2f(v); }
__device__ __forceinline__ float to_f(float v) { return v; }
__device__ __forceinline__ void from_f(float f, bf16_t& o) { o = f2bf(f); }
__device__ __forceinline__ void from_f(float f, float& o) { o = f; }

template <typename T>
__device__ __forceinline__ float ld_f(const T* p, int64_t i) {
  return to_f(p[i]);
}

// VEC consecutive elements -> fp32 (VEC 4 / 8: one or two aligned vector loads)
template <int VEC>
__device__ __forceinline__ void ld_vec(const float* p, float (&v)[VEC]) {
  if constexpr (VEC % 4 == 0) {
#pragma unroll
    for (int i = 0; i < VEC; i += 4) {
      const f32x4 a = *reinterpret_cast<const f32x4*>(p + i);
#pragma unroll
      for (int j = 0; j < 4; ++j) v[i + j] = a[j];
    }
  } else {
#pragma unroll
    for (int i = 0; i < VEC; ++i) v[i] = p[i];
  }
}
template <int VEC>
__device__ __forceinline__ void ld_vec(const bf16_t* p, float (&v)[VEC]) {
  if constexpr (VEC == 8) {
    const u16x8 a = *reinterpret_cast<const u16x8*>(p);
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = bf2f(a[j]);
  } else if constexpr (VEC == 4) {
    const u16x4 a = *reinterpret_cast<const u16x4*>(p);
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j] = bf2f(a[j]);
  } else {
#pragma unroll
    for (int i = 0; i < VEC; ++i) v[i] = bf2f(p[i]);
  }
}
template <int VEC>
__device__ __forceinline__ void st_vec(float* p, const float (&v)[VEC]) {
  if constexpr (VEC % 4 == 0) {
#pragma unroll
    for (int i = 0; i < VEC; i += 4) *reinterpret_cast<f32x4*>(p + i) = (f32x4){v[i], v[i + 1], v[i + 2], v[i + 3]};
  } else {
#pragma unroll
    for (int i = 0; i < VEC; ++i) p[i] = v[i];
  }
}
template <int VEC>
__device__ __forceinline__ void st_vec(bf16_t* p, const float (&v)[VEC]) {
  if constexpr (VEC == 8) {
    u16x8 a;
#pragma unroll
    for (int j = 0; j < 8; ++j) a[j] = f2bf(v[j]);
    *reinterpret_cast<u16x8*>(p) = a;
  } else if constexpr (VEC == 4) {
    u16x4 a;
#pragma unroll
    for (int j = 0; j < 4; ++j) a[j] = f2bf(v[j]);
    *reinterpret_cast<u16x4*>(p) = a;
  } else {
#pragma unroll
    for (int i = 0; i < VEC; ++i) p[i] = f2bf(v[i]);
  }
}

// element (row, col) of an activation of width K; packed_mt > 0: the packed layout with that many row tiles
template <typename T>
__device__ __forceinline__ void st_act(T* p, int row, int col, int K, int packed_mt, float f) {
  from_f(f, p[packed_mt > 0 ? apk_off(row, col, packed_mt) : (int64_t)row * K + col]);
}
// VEC columns from an aligned col (8 | col / VEC chunks never straddle a packed 8-column group)
template <int VEC, typename T>
__device__ __forceinline__ void st_act_vec(T* p, int row, int col, int K, int packed_mt, const float (&v)[VEC]) {
  st_vec<VEC>(p + (packed_mt > 0 ? apk_off(row, col, packed_mt) : (int64_t)row * K + col), v);
}

}  // namespace mp
