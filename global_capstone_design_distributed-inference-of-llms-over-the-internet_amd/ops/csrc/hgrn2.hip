// HGRN2 recurrence for gfx950: gated linear attention whose forget gate also decides what is written.
//
//   q_t = silu(zq_t)   f_t = lower + (1 - lower) sigmoid(zf_t + b)   k_t = 1 - f_t
//   S_t = diag(f_t) S_{t-1} + k_t v_t^T      o_t = S_t^T q_t         y_t = rms(o_t) * w   (per head)
//
// z rows are [zq (H D) | zf (H D) | v (H V)], the fused input projection.  The state S [D, V] of a
// (session, head) lives in fp32 and everything between z and y is fp32.
//
//   hgrn2_scan_kernel   one workgroup per (segment, head), the state streamed through registers once a
//                       token: the decode step (one token per row), and any (D, V) the chunk form
//                       does not cover
//   hgrn2_chunk_kernel  prompts: 16-token blocks on fp32 MFMA, the state resident in registers
#include "common.h"
#include "act_io.h"

namespace mp {

__device__ __forceinline__ float sigmoid_f(float x) { return 1.f / (1.f + expf(-x)); }

struct Hgrn2Args {
  const void* z;
  int64_t zs;            // row pitch of z
  const float *bias, *lower, *norm;
  float* state;          // [rows, H, D, V]
  const int32_t *q_seq, *q_ctx;
  void* out;             // [T, H V] row-major or packed
  int H, D, V, packed_mt;
  float eps;
};

// seg == null: blockIdx.y is one row of one token (q_ctx 0: a padding row).  seg: [3, nseg] (tok0, ntok, ..)
template <typename T, int VEC>
__global__ __launch_bounds__(256) void hgrn2_scan_kernel(Hgrn2Args a, const int32_t* __restrict__ seg, int nseg) {
  extern __shared__ float sm[];  // q[D], f[D], red[256 * VEC], red16[16]
  const int h = blockIdx.x, D = a.D, V = a.V, tid = threadIdx.x;
  float *sq = sm, *sf = sm + D, *red = sm + 2 * D, *r16 = red + 256 * VEC;
  const int tok0 = seg ? seg[blockIdx.y] : (int)blockIdx.y;
  const int ntok = seg ? seg[nseg + blockIdx.y] : 1;
  const int ctx0 = a.q_ctx[tok0];
  if (ctx0 <= 0) return;
  float* S = a.state + ((int64_t)a.q_seq[tok0] * a.H + h) * D * V;
  const int nv = V / VEC, ng = 256 / nv;
  const int g = tid / nv, c = (tid - g * nv) * VEC;
  const bool act = g < ng;
  for (int t = tok0; t < tok0 + ntok; ++t) {
    const T* z = (const T*)a.z + (int64_t)t * a.zs;
    const bool fresh = t == tok0 && ctx0 == 1;  // a sequence's first token: the slot's old state does not count
    for (int d = tid; d < D; d += 256) {
      const float zq = ld_f(z, h * D + d), zf = ld_f(z, a.H * D + h * D + d);
      const float lo = a.lower[h * D + d];
      sq[d] = zq * sigmoid_f(zq);
      sf[d] = lo + (1.f - lo) * sigmoid_f(zf + a.bias[h * D + d]);
    }
    __syncthreads();
    float o[VEC], v[VEC];
#pragma unroll
    for (int j = 0; j < VEC; ++j) o[j] = 0.f;
    if (act) {
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[j] = ld_f(z, (int64_t)2 * a.H * D + h * V + c + j);
#pragma unroll 8
      for (int d = g; d < D; d += ng) {
        float s[VEC];
        ld_vec<VEC>(S + (int64_t)d * V + c, s);
        const float f = sf[d], k = 1.f - f, qd = sq[d];
#pragma unroll
        for (int j = 0; j < VEC; ++j) {
          s[j] = (fresh ? 0.f : f * s[j]) + k * v[j];
          o[j] += qd * s[j];
        }
        st_vec<VEC>(S + (int64_t)d * V + c, s);
      }
#pragma unroll
      for (int j = 0; j < VEC; ++j) red[g * V + c + j] = o[j];
    }
    __syncthreads();
    float ss = 0.f;
    for (int e = tid; e < V; e += 256) {
      float x = 0.f;
      for (int i = 0; i < ng; ++i) x += red[i * V + e];
      red[e] = x;  // (only this thread reads column e)
      ss += x * x;
    }
    const float sc = 1.f / sqrtf(block_sum(ss, r16) / (float)V + a.eps);
    for (int e = tid; e < V; e += 256)
      st_act((T*)a.out, t, h * V + e, a.H * V, a.packed_mt, red[e] * sc * a.norm[e]);
    __syncthreads();
  }
}

template <typename T>
static int launch_scan(const Hgrn2Args& a, const int32_t* seg, int nseg, int n, hipStream_t stream) {
  const int vec = a.V % 4 == 0 ? 4 : 1;
  if (a.V / vec > 256) return -1;
  const size_t lds = (2 * a.D + 256 * vec + 16) * sizeof(float);
  if (lds > 60000) return -1;
  if (vec == 4) hipLaunchKernelGGL((hgrn2_scan_kernel<T, 4>), dim3(a.H, n), dim3(256), lds, stream, a, seg, nseg);
  else hipLaunchKernelGGL((hgrn2_scan_kernel<T, 1>), dim3(a.H, n), dim3(256), lds, stream, a, seg, nseg);
  return (int)hipGetLastError();
}

}  // namespace mp

extern "C" int mp_hgrn2_scan(const void* z, int64_t zs, const float* bias, const float* lower, const float* norm,
                             float* state, const int32_t* q_seq, const int32_t* q_ctx, void* out, int H, int D, int V,
                             float eps, const int32_t* seg, int nseg, int n, int packed_mt, int f32,
                             hipStream_t stream) {
  using namespace mp;
  (void)hipGetLastError();
  if (n == 0) return 0;
  if (n > 65535) return -1;
  const Hgrn2Args a{z, zs, bias, lower, norm, state, q_seq, q_ctx, out, H, D, V, packed_mt, eps};
  return f32 ? launch_scan<float>(a, seg, nseg, n, stream) : launch_scan<bf16_t>(a, seg, nseg, n, stream);
}
