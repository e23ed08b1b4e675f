// Linear attention with one scalar decay per head and token, gfx950: retention and the mLSTM matrix memory.
//
//   S_t = a_t S_{t-1} + b_t k_t v_t^T      o_t = S_t^T q_t
//   retention  a_t = decay_h, b_t = 1; q and k turned by their position, k scaled
//   mLSTM      m_t = max(f_t + m_{t-1}, i_t), a_t = exp(f_t + m_{t-1} - m_t), b_t = exp(i_t - m_t), a normalizer
//              n_t = a_t n_{t-1} + b_t k_t, and o_t divided by max(|n_t . q_t|, exp(-m_t)) + 1e-6;
//              i = cap tanh((z_i + b_i) / cap), f = log sigmoid(cap tanh((z_f + b_f) / cap))
//   y_t = o_t / rms(o_t) (per head) [* w] * gate(g_t)      gate: silu (retention), sigmoid (mLSTM)
//
// z rows are [q (H D) | k (H D) | v (H V) | g (H V) | i (H) | f (H)], the fused input projection.  The state S [D, V]
// of a (session, head) lives in fp32 and everything between z and y is fp32.
//
//   linear_scan_kernel   one workgroup per (sequence, head), the state streamed through registers once a token: the
//                        decode step (one token per row), both element types and any shape
#include "common.h"
#include "act_io.h"

namespace mp {

enum { RETENTION = 0, MLSTM = 1 };

struct LinArgs {
  const void* z;           // [T, zs] projected rows
  int64_t zs;
  const float* rope;       // retention: [positions, rot], cosines then sines
  const float* decay;      // retention: [H] log2 of the decay
  const float* bias;       // mLSTM: [2, H] input and forget gate
  const float* norm;       // mLSTM: [H V]
  float* state;            // [rows, H, D, V]
  float* aux;              // mLSTM: [rows, H, D + 1] normalizer, running maximum
  const int32_t *q_seq, *q_ctx;
  void* out;               // [T, H V] row-major or packed
  int H, D, V, rot, packed_mt;
  float cap, eps, qs, ks;  // qs, ks: factors of q and k
};

__device__ __forceinline__ float soft_cap(float x, float cap) { return cap * tanhf(x / cap); }
__device__ __forceinline__ float log_sigmoid(float x) { return fminf(x, 0.f) - log1pf(expf(-fabsf(x))); }

// element d of head vector ``x`` (position's table row ``cs``), turned
template <typename T>
__device__ __forceinline__ float turned(const T* x, int d, int rot, const float* cs) {
  const float v = to_f(x[d]);
  if (d >= rot) return v;
  const int half = rot >> 1;
  return d < half ? v * cs[d] - to_f(x[d + half]) * cs[half + d] : v * cs[d - half] + to_f(x[d - half]) * cs[d];
}

// seg == null: blockIdx.y is one row of one token (q_ctx 0: a padding row).  seg: [2+, nseg] (tok0, ntok, ..)
template <typename T, int VEC, int KIND>
__global__ __launch_bounds__(256) void linear_scan_kernel(LinArgs a, const int32_t* __restrict__ seg, int nseg) {
  constexpr int PRE = 16;
  extern __shared__ float sm[];  // q[D], k[D], red[256 * VEC], red16[16]
  const int h = blockIdx.x, H = a.H, D = a.D, V = a.V, tid = threadIdx.x;
  float *sq = sm, *sk = sm + D, *red = sm + 2 * D, *r16 = red + 256 * VEC;
  const int tok0 = seg ? seg[blockIdx.y] : (int)blockIdx.y;
  const int ntok = seg ? seg[nseg + blockIdx.y] : 1;
  const int ctx0 = a.q_ctx[tok0];
  if (ctx0 <= 0) return;
  const int64_t sh = (int64_t)a.q_seq[tok0] * H + h;
  float* S = a.state + sh * D * V;
  float* nm = KIND == MLSTM ? a.aux + sh * (D + 1) : nullptr;
  const int nv = V / VEC, ng = 256 / nv;
  const int g = tid / nv, c = (tid - g * nv) * VEC;
  const bool act = g < ng;
  float m = KIND == MLSTM && ctx0 > 1 ? nm[D] : 0.f;
  for (int t = tok0; t < tok0 + ntok; ++t) {
    const T* z = (const T*)a.z + (int64_t)t * a.zs;
    // the first PRE state rows of this thread are on their way while q, k and the gates are made
    float pre[PRE][VEC];
    if (act) {
#pragma unroll
      for (int i = 0; i < PRE; ++i) ld_vec<VEC>(S + (int64_t)min(g + i * ng, D - 1) * V + c, pre[i]);
    }
    const bool fresh = t == tok0 && ctx0 == 1;  // a sequence's first token: the slot's old state does not count
    float fa, fb;                               // a_t, b_t
    if constexpr (KIND == MLSTM) {
      const T* zg = z + 2 * H * (D + V);
      const float li = soft_cap(to_f(zg[h]) + a.bias[h], a.cap);
      const float lf = log_sigmoid(soft_cap(to_f(zg[H + h]) + a.bias[H + h], a.cap));
      const float m1 = fmaxf(lf + m, li);
      fa = expf(lf + m - m1);
      fb = expf(li - m1);
      m = m1;
    } else {
      fa = exp2f(a.decay[h]);
      fb = 1.f;
    }
    float nq = 0.f;
    for (int d = tid; d < D; d += 256) {
      float q, k;
      if constexpr (KIND == MLSTM) {
        q = to_f(z[h * D + d]) * a.qs;
        k = to_f(z[(H + h) * D + d]) * a.ks * fb;
        const float n = (fresh ? 0.f : fa * nm[d]) + k;
        nm[d] = n;
        nq += n * q;
      } else {
        const float* cs = a.rope + (int64_t)(ctx0 - 1 + t - tok0) * a.rot;
        q = turned(z + h * D, d, a.rot, cs) * a.qs;
        k = turned(z + (H + h) * D, d, a.rot, cs) * a.ks;
      }
      sq[d] = q;
      sk[d] = k;
    }
    float den = 1.f;
    if constexpr (KIND == MLSTM) den = 1.f / (fmaxf(fabsf(block_sum(nq, r16)), expf(-m)) + 1e-6f);
    __syncthreads();
    float o[VEC], v[VEC];
#pragma unroll
    for (int j = 0; j < VEC; ++j) o[j] = 0.f;
    if (act) {
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[j] = ld_f(z, (int64_t)2 * H * D + h * V + c + j);
      auto row = [&](int d, float (&s)[VEC]) {
        const float k = sk[d], qd = sq[d];
#pragma unroll
        for (int j = 0; j < VEC; ++j) {
          s[j] = (fresh ? 0.f : fa * s[j]) + k * v[j];
          o[j] += qd * s[j];
        }
        st_vec<VEC>(S + (int64_t)d * V + c, s);
      };
#pragma unroll
      for (int i = 0; i < PRE; ++i)
        if (g + i * ng < D) row(g + i * ng, pre[i]);
#pragma unroll 4
      for (int d = g + PRE * ng; d < D; d += ng) {
        float s[VEC];
        ld_vec<VEC>(S + (int64_t)d * V + c, s);
        row(d, s);
      }
#pragma unroll
      for (int j = 0; j < VEC; ++j) red[g * V + c + j] = o[j];
    }
    __syncthreads();
    float ss = 0.f;
    for (int e = tid; e < V; e += 256) {
      float x = 0.f;
      for (int i = 0; i < ng; ++i) x += red[i * V + e];
      x *= den;
      red[e] = x;  // (only this thread reads column e)
      ss += x * x;
    }
    const float sc = 1.f / sqrtf(block_sum(ss, r16) / (float)V + a.eps);
    const T* zg = z + 2 * H * D + H * V + h * V;
    for (int e = tid; e < V; e += 256) {
      const float gz = to_f(zg[e]), s = 1.f / (1.f + expf(-gz));
      const float w = KIND == MLSTM ? a.norm[h * V + e] * s : gz * s;
      st_act((T*)a.out, t, h * V + e, H * V, a.packed_mt, red[e] * sc * w);
    }
    __syncthreads();
  }
  if (KIND == MLSTM && tid == 0) nm[D] = m;
}

template <typename T, int KIND>
static int launch_scan(const LinArgs& a, const int32_t* seg, int nseg, int n, hipStream_t stream) {
  const int vec = a.V % 4 == 0 ? 4 : 1;
  if (a.V / vec > 256) return -1;
  const size_t lds = (2 * a.D + 256 * vec + 16) * sizeof(float);
  if (lds > 60000) return -1;
#define MP_LS(VEC_) \
  hipLaunchKernelGGL((linear_scan_kernel<T, VEC_, KIND>), dim3(a.H, n), dim3(256), lds, stream, a, seg, nseg)
  if (vec == 4) MP_LS(4); else MP_LS(1);
#undef MP_LS
  return (int)hipGetLastError();
}

}  // namespace mp

extern "C" int mp_linear_scan(int kind, const void* z, int64_t zs, const float* rope, int rot, const float* decay,
                              const float* bias, const float* norm, float* state, float* aux, const int32_t* q_seq,
                              const int32_t* q_ctx, void* out, int H, int D, int V, float cap, float eps, float qs,
                              float ks, const int32_t* seg, int nseg, int n, int packed_mt, int f32,
                              hipStream_t stream) {
  using namespace mp;
  (void)hipGetLastError();
  if (n == 0) return 0;
  if (n > 65535) return -1;
  const LinArgs a{z, zs, rope, decay, bias, norm, state, aux, q_seq, q_ctx, out, H, D, V, rot, packed_mt, cap, eps, qs, ks};
  if (kind == MLSTM)
    return f32 ? launch_scan<float, MLSTM>(a, seg, nseg, n, stream) : launch_scan<bf16_t, MLSTM>(a, seg, nseg, n, stream);
  return f32 ? launch_scan<float, RETENTION>(a, seg, nseg, n, stream)
             : launch_scan<bf16_t, RETENTION>(a, seg, nseg, n, stream);
}
