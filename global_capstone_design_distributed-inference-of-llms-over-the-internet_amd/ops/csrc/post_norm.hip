// Bandwidth-bound kernels of post-norm decoders with a 32-bit residual stream.
//
//   embed_pos       res[t] = table[id] + sinusoid(position), fp32; plus the activation copy of it
//   residual_norm   res[t] += rms(y[t]) * w (w = norm gain x layer scale, fp32); plus the copy
//                   y: activation rows, or the S fp32 split-K slabs of the projection that made it
//   rows_norm       out[i] = rms(res[rows[i]]) * w
//   relu2           out = max(x, 0)^2
//
// The activation copy feeds the next GEMM: row-major, or the packed decode-GEMM layout
// (common.h apk_off) when packed_mt > 0.
#include "common.h"
#include "act_io.h"

namespace mp {

template <typename T>
__global__ __launch_bounds__(256) void embed_pos_kernel(const int64_t* __restrict__ ids, const T* __restrict__ table,
                                                        int64_t vocab, const int64_t* __restrict__ pos,
                                                        const double* __restrict__ inv, float* __restrict__ res,
                                                        T* __restrict__ xb, int W, int packed_mt) {
  const int t = blockIdx.x;
  int64_t id = ids[t];
  if (id < 0 || id >= vocab) id = 0;  // never read out of bounds; the host validates ids
  const double p = (double)pos[t];
  const T* src = table + id * W;
  for (int i = threadIdx.x; 2 * i < W; i += blockDim.x) {
    // the angle is reduced in double: a long context's angle has few fraction bits left in fp32
    constexpr double TWO_PI = 6.283185307179586476925286766559;
    double a = p * inv[i];
    a -= TWO_PI * floor(a / TWO_PI);
    float s, c;
    sincosf((float)a, &s, &c);
    const float x0 = ld_f(src, 2 * i) + s;
    res[(int64_t)t * W + 2 * i] = x0;
    st_act(xb, t, 2 * i, W, packed_mt, x0);
    if (2 * i + 1 < W) {
      const float x1 = ld_f(src, 2 * i + 1) + c;
      res[(int64_t)t * W + 2 * i + 1] = x1;
      st_act(xb, t, 2 * i + 1, W, packed_mt, x1);
    }
  }
}

// SRC: 0 = rows of T, 1 = S fp32 slabs, 2 = no y: out rows = rms(res[rows]) * w (rows_norm)
template <typename T, int VEC, int MAXC, int SRC, int NT>
__global__ __launch_bounds__(NT) void residual_norm_kernel(const T* __restrict__ y, int64_t ys,
                                                            const float* __restrict__ part, int S, int64_t slab,
                                                            float* __restrict__ res, const float* __restrict__ w,
                                                            T* __restrict__ xb, const int32_t* __restrict__ rows,
                                                            int W, float eps, int packed_mt) {
  __shared__ float red[16];
  const int orow = blockIdx.x;
  const int row = SRC == 2 && rows != nullptr ? rows[orow] : orow;
  const int nch = W / VEC;
  float v[MAXC][VEC], r[MAXC][VEC], g[MAXC][VEC];
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < MAXC; ++k) {
    const int c = min((int)threadIdx.x + NT * k, nch - 1) * VEC;
    ld_vec<VEC>(res + (int64_t)row * W + c, r[k]);
    ld_vec<VEC>(w + c, g[k]);
    if constexpr (SRC == 0) {
      ld_vec<VEC>(y + (int64_t)row * ys + c, v[k]);
    } else if constexpr (SRC == 1) {
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[k][j] = 0.f;
      for (int s = 0; s < S; s += 4) {  // four slabs' loads in flight, added in slab order
        float p[4][VEC];
#pragma unroll
        for (int i = 0; i < 4; ++i) ld_vec<VEC>(part + min(s + i, S - 1) * slab + (int64_t)row * ys + c, p[i]);
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (s + i < S)
#pragma unroll
            for (int j = 0; j < VEC; ++j) v[k][j] += p[i][j];
      }
    } else {
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[k][j] = r[k][j];
    }
  }
#pragma unroll
  for (int k = 0; k < MAXC; ++k)
    if ((int)threadIdx.x + NT * k < nch)
#pragma unroll
      for (int j = 0; j < VEC; ++j) ss += v[k][j] * v[k][j];
  const float sc = 1.f / sqrtf(block_sum(ss, red) / (float)W + eps);
#pragma unroll
  for (int k = 0; k < MAXC; ++k) {
    const int ch = threadIdx.x + NT * k;
    if (ch >= nch) continue;
    float o[VEC];
#pragma unroll
    for (int j = 0; j < VEC; ++j) o[j] = SRC == 2 ? v[k][j] * sc * g[k][j] : r[k][j] + v[k][j] * sc * g[k][j];
    if constexpr (SRC != 2) st_vec<VEC>(res + (int64_t)row * W + ch * VEC, o);
    if (xb != nullptr) st_act_vec<VEC>(xb, orow, ch * VEC, W, packed_mt, o);
  }
}

template <typename T, int VEC>
__global__ __launch_bounds__(256) void relu2_kernel(const T* __restrict__ x, int64_t xs, T* __restrict__ out, int64_t M,
                                                    int F, int packed_mt) {
  const int nch = F / VEC;
  const int64_t n = M * nch;
  for (int64_t i = blockIdx.x * (int64_t)blockDim.x + threadIdx.x; i < n; i += (int64_t)gridDim.x * blockDim.x) {
    const int64_t t = i / nch;
    const int c = (int)(i - t * nch) * VEC;
    float v[VEC];
    ld_vec<VEC>(x + t * xs + c, v);
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      const float a = fmaxf(v[j], 0.f);
      v[j] = a * a;
    }
    st_act_vec<VEC>(out, (int)t, c, F, packed_mt, v);
  }
}

template <typename T, int SRC>
static int launch_residual_norm(const void* y, int64_t ys, const float* part, int S, int64_t slab, float* res,
                                const float* w, void* xb, const int32_t* rows, int n, int W, float eps, int packed_mt,
                                hipStream_t stream) {
#define MP_RN(VEC_, MAXC_, NT_)                                                                                     \
  hipLaunchKernelGGL((residual_norm_kernel<T, VEC_, MAXC_, SRC, NT_>), dim3(n), dim3(NT_), 0, stream, (const T*)y, ys, \
                     part, S, slab, res, w, (T*)xb, rows, W, eps, packed_mt)
  if (W % 4 == 0 && (SRC == 2 || ys % 4 == 0)) {
    const int ch = W / 4;
    if (n <= 256 && ch > 256 && ch <= 2048) {  // few rows: latency is what there is to save
      if (ch <= 1024) MP_RN(4, 1, 1024);
      else MP_RN(4, 2, 1024);
    } else if (ch <= 256) MP_RN(4, 1, 256);
    else if (ch <= 512) MP_RN(4, 2, 256);
    else if (ch <= 1024) MP_RN(4, 4, 256);
    else if (ch <= 2048) MP_RN(4, 8, 256);
    else if (ch <= 4096) MP_RN(4, 16, 256);
    else return -1;
  } else {
    if (W > 16 * 256) return -1;
    MP_RN(1, 16, 256);
  }
#undef MP_RN
  return (int)hipGetLastError();
}

}  // namespace mp

extern "C" int mp_embed_pos(const int64_t* ids, const void* table, int64_t vocab, const int64_t* pos, const double* inv,
                            float* res, void* xb, int T, int W, int packed_mt, int f32, hipStream_t stream) {
  using namespace mp;
  (void)hipGetLastError();
  if (T == 0) return 0;
  if (f32)
    hipLaunchKernelGGL(embed_pos_kernel<float>, dim3(T), dim3(256), 0, stream, ids, (const float*)table, vocab, pos,
                       inv, res, (float*)xb, W, packed_mt);
  else
    hipLaunchKernelGGL(embed_pos_kernel<bf16_t>, dim3(T), dim3(256), 0, stream, ids, (const bf16_t*)table, vocab, pos,
                       inv, res, (bf16_t*)xb, W, packed_mt);
  return (int)hipGetLastError();
}

// part != null: y is the S slabs [S][n][ys]; y == part == null: rows_norm
extern "C" int mp_residual_norm(const void* y, int64_t ys, const float* part, int S, int64_t slab, float* res,
                                const float* w, void* xb, const int32_t* rows, int n, int W, float eps, int packed_mt,
                                int f32, hipStream_t stream) {
  using namespace mp;
  (void)hipGetLastError();
  if (n == 0) return 0;
  if (part != nullptr) {
    if (f32) return -2;
    return launch_residual_norm<bf16_t, 1>(y, ys, part, S, slab, res, w, xb, rows, n, W, eps, packed_mt, stream);
  }
  if (y == nullptr)
    return f32 ? launch_residual_norm<float, 2>(y, ys, part, S, slab, res, w, xb, rows, n, W, eps, packed_mt, stream)
               : launch_residual_norm<bf16_t, 2>(y, ys, part, S, slab, res, w, xb, rows, n, W, eps, packed_mt, stream);
  return f32 ? launch_residual_norm<float, 0>(y, ys, part, S, slab, res, w, xb, rows, n, W, eps, packed_mt, stream)
             : launch_residual_norm<bf16_t, 0>(y, ys, part, S, slab, res, w, xb, rows, n, W, eps, packed_mt, stream);
}

extern "C" int mp_relu2(const void* x, int64_t xs, void* out, int64_t M, int F, int packed_mt, int f32,
                        hipStream_t stream) {
  using namespace mp;
  (void)hipGetLastError();
  if (M == 0) return 0;
  const int vec = F % 8 == 0 && xs % 8 == 0 ? 8 : 1;
  int64_t g = (M * (F / vec) + 255) / 256;
  const dim3 grid((unsigned)(g > 8192 ? 8192 : g));
#define MP_R2(T_, V_) \
  hipLaunchKernelGGL((relu2_kernel<T_, V_>), grid, dim3(256), 0, stream, (const T_*)x, xs, (T_*)out, M, F, packed_mt)
  if (f32) {
    if (vec == 8) MP_R2(float, 8); else MP_R2(float, 1);
  } else {
    if (vec == 8) MP_R2(bf16_t, 8); else MP_R2(bf16_t, 1);
  }
#undef MP_R2
  return (int)hipGetLastError();
}
