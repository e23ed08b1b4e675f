// Grouped-query attention with rotated keys and values, soft-capped scores, a sink, and heads mixed after the softmax.
//
//   s_g(i, j) = cap tanh(scale q_g(i) . k_c(j) / cap)           c = g's kv head, j <= i
//   p_g(i, j) = exp(s_g) / (1 + sum_j exp(s_g))                  (a sink of score 0 without a value)
//   a_h(i, j) = sum_g T[h, g] p_g(i, j)
//   o_h(i)    = R(-i) sum_j a_h(i, j) R(j) v_c(j)                R(p): all pairs (m, m + V / 2) turned by p f_m
//   out_h(i)  = sigmoid(gate_h(i)) o_h(i)
//
// q and k are normed per head (root mean square, one gain for all heads) and turned on their first ``rot`` entries.
//
// Cache: a page holds for every kv head its key rows [page][D] and then its turned values [page / B][V][B], B =
// min(32, page) keys side by side, so that 16-byte loads along the keys are MFMA operands of the value product.  Pair
// m of a value lies in columns 2 m, 2 m + 1.
//
//   mixed_prep_kernel   projected row [q (H D) | k (G D) | v (G V) | gate (H)] -> q', cache; and the feed-forward's
//                       activation where its projection lies in the same row
//   mixed_prep_vec_kernel  the same for whole 8-column vectors
//   mixed_any_kernel    any shape and both element types: one workgroup per query token
#include "attn_mixed.h"

namespace mp {

struct FfArgs {          // feed-forward activation of the row's columns from ``col`` on
  int kind;              // 0: none, 1: gelu, 2: clamped gated form, 3: the same times a gate per token
  int F, block, col, out_col;
  float limit;
};

constexpr int MIX_HEAD = 512;  // largest head size of the prep kernel
constexpr float MIX_GLU_ALPHA = 1.702f;

template <typename T, int VEC>
__device__ __forceinline__ void ff_columns(const T* __restrict__ zr, const FfArgs& f, T* out, int t, int64_t os, int mt,
                                           int first, int step) {
  float tg = 1.f;
  if (f.kind == 3) tg = 1.f / (1.f + expf(-to_f(zr[f.col + 2 * f.F])));
  for (int c = first * VEC; c < f.F; c += step * VEC) {
    float g[VEC], u[VEC];
    if (f.kind == 1) {
      ld_vec<VEC>(zr + f.col + c, g);
#pragma unroll
      for (int j = 0; j < VEC; ++j) g[j] = 0.5f * g[j] * (1.f + erff(g[j] * 0.70710678118654752f));
    } else {
      const T* p = zr + f.col + (int64_t)(c / f.block) * 2 * f.block + c % f.block;
      ld_vec<VEC>(p, g);
      ld_vec<VEC>(p + f.block, u);
#pragma unroll
      for (int j = 0; j < VEC; ++j) {
        const float a = fminf(g[j], f.limit), b = fminf(fmaxf(u[j], -f.limit), f.limit);
        g[j] = tg * (a / (1.f + expf(-MIX_GLU_ALPHA * a)) * (b + 1.f));
      }
    }
    st_act_vec<VEC>(out, t, f.out_col + c, (int)os, mt, g);
  }
}

// grid (T, nh + nf): the first nh blocks take four heads each (queries, keys, values), the others the feed-forward
template <typename T, int VEC>
__global__ __launch_bounds__(256) void mixed_prep_kernel(MixedArgs a, FfArgs f, int nh) {
  __shared__ float sh[4][MIX_HEAD];
  const int t = blockIdx.x, lane = threadIdx.x & 63, wv = threadIdx.x >> 6;
  const T* z = (const T*)a.z + (int64_t)t * a.zs;
  if ((int)blockIdx.y >= nh) {
    ff_columns<T, VEC>(z, f, (T*)a.out, t, a.os, a.packed_mt, ((int)blockIdx.y - nh) * 256 + threadIdx.x,
                       ((int)gridDim.y - nh) * 256);
    return;
  }
  const int64_t slot = a.slots[t];
  if (slot < 0) return;  // (uniform: a padding row)
  const int job = blockIdx.y * 4 + wv, H = a.H, G = a.G, D = a.D, V = a.V;
  const bool on = job < H + 2 * G, val = job >= H + G;
  const int n = val ? V : D, c0 = job < H + G ? job * D : (H + G) * D + (job - H - G) * V;
  const int pos = a.q_ctx[t] - 1;
  float x[MIX_HEAD / 64], ss = 0.f;
#pragma unroll
  for (int k = 0; k < MIX_HEAD / 64; ++k) {
    const int i = lane + 64 * k;
    x[k] = on && i < n ? to_f(z[c0 + i]) : 0.f;
    ss += x[k] * x[k];
  }
  if (!val) {
    const float r = 1.f / sqrtf(wave_sum(ss) / (float)D + a.eps);
    const float* g = job < H ? a.qg : a.kg;
#pragma unroll
    for (int k = 0; k < MIX_HEAD / 64; ++k) {
      const int i = lane + 64 * k;
      if (i < n) x[k] *= r * g[i];
    }
  }
#pragma unroll
  for (int k = 0; k < MIX_HEAD / 64; ++k)
    if (lane + 64 * k < n) sh[wv][lane + 64 * k] = x[k];
  __syncthreads();
  if (!on) return;
  const int dims = val ? V : a.rot, half = dims >> 1;
  const float* cs = val ? a.vrope + (int64_t)pos * V : a.rope + (int64_t)pos * a.rot;
  const int64_t pg = slot >> a.page_log2, off = slot & ((1 << a.page_log2) - 1), page = 1 << a.page_log2;
  const int kv = job < H ? 0 : (job - H) % G;
  T* pb = (T*)a.cache + (pg * G + kv) * page * (D + V);
#pragma unroll
  for (int k = 0; k < MIX_HEAD / 64; ++k) {
    const int i = lane + 64 * k;
    if (i >= n) continue;
    float y = x[k];
    if (i < dims) {
      const int m = i < half ? i : i - half;
      const float c = cs[m], s = cs[half + m], o = sh[wv][i < half ? i + half : i - half];
      y = i < half ? y * c - o * s : y * c + o * s;
    }
    if (job < H) from_f(y, ((T*)a.qn)[((int64_t)t * H + job) * D + i]);
    else if (!val) from_f(y, pb[off * D + i]);
    else from_f(y, pb[page * D + val_at((int)off, i < half ? 2 * i : 2 * (i - half) + 1, V, val_block_log2(a.page_log2))]);
  }
}

// The same for whole 8-column vectors: a workgroup of blockIdx.y 0 takes all of a row's heads.  Pass 1 brings the row to LDS
// with a sum of squares per vector; pass 2 makes a vector from it and its rotation partner, half the turned entries away.
constexpr int PREP_VECS = 2048;  // vectors of a row at most (LDS: 20 bytes each)

__global__ __launch_bounds__(256) void mixed_prep_vec_kernel(MixedArgs a, FfArgs f) {
  extern __shared__ __attribute__((aligned(16))) bf16_t row[];
  const int t = blockIdx.x, tid = threadIdx.x;
  const bf16_t* z = (const bf16_t*)a.z + (int64_t)t * a.zs;
  if (blockIdx.y > 0) {
    ff_columns<bf16_t, 8>(z, f, (bf16_t*)a.out, t, a.os, a.packed_mt, ((int)blockIdx.y - 1) * 256 + tid,
                          ((int)gridDim.y - 1) * 256);
    return;
  }
  const int64_t slot = a.slots[t];
  if (slot < 0) return;  // (uniform: a padding row)
  const int H = a.H, G = a.G, D = a.D, V = a.V, dv = D >> 3, vv = V >> 3, nk = (H + G) * dv, n = nk + G * vv;
  float* sq = reinterpret_cast<float*>(row + n * 8);
  for (int i = tid; i < n; i += 256) {
    const u16x8 x = *reinterpret_cast<const u16x8*>(z + i * 8);
    *reinterpret_cast<u16x8*>(row + i * 8) = x;
    float s = 0.f;
#pragma unroll
    for (int j = 0; j < 8; ++j) s += bf2f(x[j]) * bf2f(x[j]);
    sq[i] = s;
  }
  __syncthreads();
  const int pos = a.q_ctx[t] - 1, bl = val_block_log2(a.page_log2);
  const int64_t pg = slot >> a.page_log2, page = 1 << a.page_log2;
  const int off = (int)(slot & (page - 1));
  for (int i = tid; i < n; i += 256) {
    const bool val = i >= nk;
    const int head = val ? (i - nk) / vv : i / dv, c = val ? (i - nk) - head * vv : i - head * dv;
    const int half = (val ? V : a.rot) >> 1, base = i - c, e0 = 8 * c;  // (whole vectors: half is a multiple of 8)
    float x[8], p[8];
    ld_vec<8>(row + i * 8, x);
    const bool turn = e0 < 2 * half;
    const bool up = e0 >= half;  // the pair's second entry
    const float* cs = (val ? a.vrope + (int64_t)pos * V : a.rope + (int64_t)pos * a.rot) + (turn ? e0 - (up ? half : 0) : 0);
    if (turn) ld_vec<8>(row + (base + ((up ? e0 - half : e0 + half) >> 3)) * 8, p);
    if (!val) {
      float ss = 0.f;
      for (int k = 0; k < dv; ++k) ss += sq[base + k];
      const float r = 1.f / sqrtf(ss / (float)D + a.eps);
      const float* g = head < H ? a.qg : a.kg;
      float gx[8], gp[8];
      ld_vec<8>(g + e0, gx);
      if (turn) ld_vec<8>(g + (up ? e0 - half : e0 + half), gp);
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        x[j] *= r * gx[j];
        if (turn) p[j] *= r * gp[j];
      }
    }
    if (turn) {
      float c8[8], s8[8];
      ld_vec<8>(cs, c8);
      ld_vec<8>(cs + half, s8);
#pragma unroll
      for (int j = 0; j < 8; ++j) x[j] = up ? x[j] * c8[j] + p[j] * s8[j] : x[j] * c8[j] - p[j] * s8[j];
    }
    if (!val && head < H) {
      st_vec<8>((bf16_t*)a.qn + (int64_t)t * H * D + i * 8, x);
      continue;
    }
    bf16_t* pb = (bf16_t*)a.cache + (pg * G + (val ? head : head - H)) * page * (D + V);
    if (!val) {
      st_vec<8>(pb + (int64_t)off * D + e0, x);
    } else {
      pb += page * D + val_at(off, 2 * (up ? e0 - half : e0) + up, V, bl);
#pragma unroll
      for (int j = 0; j < 8; ++j) pb[(int64_t)j << (bl + 1)] = f2bf(x[j]);
    }
  }
}

template <typename T, int VEC>
__global__ __launch_bounds__(256) void ffn_act_kernel(const T* __restrict__ z, int64_t zs, T* out, int64_t os, int mt,
                                                      FfArgs f) {
  ff_columns<T, VEC>(z + (int64_t)blockIdx.x * zs, f, out, blockIdx.x, os, mt, blockIdx.y * 256 + threadIdx.x,
                     gridDim.y * 256);
}

constexpr int MX_TILE = 64;

__device__ __forceinline__ float soft_cap(float s, float cap) { return cap > 0.f ? cap * tanhf(s / cap) : s; }

// NE: accumulators per thread, H V <= 256 NE
template <typename T, int NE>
__global__ __launch_bounds__(256) void mixed_any_kernel(MixedArgs a) {
  extern __shared__ float sm[];
  const int t = blockIdx.x, tid = threadIdx.x, H = a.H, G = a.G, D = a.D, V = a.V, HD = H * D, HV = H * V, rep = H / G;
  const int ctx = a.q_ctx[t];
  if (ctx <= 0) return;
  float *sq = sm, *raw = sq + HD, *mix = raw + H * MX_TILE, *m = mix + H * MX_TILE, *l = m + H;
  int* spg = (int*)(l + H);   // page and place of every key of the tile
  int* soff = spg + MX_TILE;
  for (int i = tid; i < HD; i += 256) sq[i] = ld_f((const T*)a.qn, (int64_t)t * HD + i);
  for (int h = tid; h < H; h += 256) {
    m[h] = 0.f;  // the sink
    l[h] = 1.f;
  }
  float o[NE];
#pragma unroll
  for (int n = 0; n < NE; ++n) o[n] = 0.f;
  const int32_t* bt = a.bt + (int64_t)a.q_seq[t] * a.bt_stride;
  const int pmask = (1 << a.page_log2) - 1, bl = val_block_log2(a.page_log2);
  const int64_t page = 1 << a.page_log2, prow = page * (D + V);
  for (int pass = 0; pass < 2; ++pass)
    for (int j0 = 0; j0 < ctx; j0 += MX_TILE) {
      const int n = min(MX_TILE, ctx - j0);
      __syncthreads();
      for (int j = tid; j < n; j += 256) {
        spg[j] = bt[(j0 + j) >> a.page_log2];
        soff[j] = (j0 + j) & pmask;
      }
      __syncthreads();
      for (int e = tid; e < H * n; e += 256) {
        const int g = e / n, j = e - g * n;
        const T* kp = (const T*)a.cache + ((int64_t)spg[j] * G + g / rep) * prow + (int64_t)soff[j] * D;
        float s = 0.f;
        for (int d = 0; d < D; ++d) s += sq[g * D + d] * to_f(kp[d]);
        raw[g * MX_TILE + j] = soft_cap(s * a.scale, a.cap);
      }
      __syncthreads();
      if (pass == 0) {
        for (int h = tid; h < H; h += 256) {
          float mx = m[h];
          for (int j = 0; j < n; ++j) mx = fmaxf(mx, raw[h * MX_TILE + j]);
          float s = 0.f;
          for (int j = 0; j < n; ++j) s += expf(raw[h * MX_TILE + j] - mx);
          l[h] = l[h] * expf(m[h] - mx) + s;
          m[h] = mx;
        }
        continue;
      }
      for (int e = tid; e < H * n; e += 256) {
        const int g = e / n, at = g * MX_TILE + e - g * n;
        raw[at] = expf(raw[at] - m[g]) / l[g];
      }
      __syncthreads();
      for (int e = tid; e < H * n; e += 256) {
        const int h = e / n, j = e - h * n;
        float s = 0.f;
        for (int g = 0; g < H; ++g) s += a.talk[h * H + g] * raw[g * MX_TILE + j];
        mix[h * MX_TILE + j] = s;
      }
      __syncthreads();
#pragma unroll
      for (int k = 0; k < NE; ++k) {
        const int e = tid + 256 * k;
        if (e < HV) {
          const int h = e / V, v = e - h * V;
          const T* vp = (const T*)a.cache + (h / rep) * prow + page * D;
          float s = o[k];
          for (int j = 0; j < n; ++j)
            s += mix[h * MX_TILE + j] * to_f(vp[(int64_t)spg[j] * G * prow + val_at(soff[j], v, V, bl)]);
          o[k] = s;
        }
      }
    }
  const T* gate = (const T*)a.z + (int64_t)t * a.zs + HD + G * (D + V);
  const float* cs = a.vrope + (int64_t)(ctx - 1) * V;
#pragma unroll
  for (int k = 0; k < NE; ++k) {  // (a pair lies in neighbouring lanes)
    const int e = tid + 256 * k, h = min(e / V, H - 1), v = e % V, mm = v >> 1;
    const float other = __shfl_xor(o[k], 1, 64);
    if (e < HV) {
      const float c = cs[mm], s = cs[V / 2 + mm];
      const float y = v & 1 ? o[k] * c - other * s : o[k] * c + other * s;
      st_act((T*)a.out, t, h * V + mm + (v & 1) * (V / 2), (int)a.os, a.packed_mt, y / (1.f + expf(-ld_f(gate, h))));
    }
  }
}

template <typename T>
static int launch_mixed_any(const MixedArgs& a, int n, hipStream_t stream) {
  const int HV = a.H * a.V;
  const size_t lds = (a.H * a.D + 2 * a.H * MX_TILE + 2 * a.H + 2 * MX_TILE) * sizeof(float);
  if (lds > 160 * 1024) return -1;
#define MP_MA(NE_)                                                                                                 \
  {                                                                                                                \
    if (lds > 65536) /* above the default limit of dynamic LDS */                                                  \
      (void)hipFuncSetAttribute((const void*)mixed_any_kernel<T, NE_>, hipFuncAttributeMaxDynamicSharedMemorySize, \
                                (int)lds);                                                                         \
    hipLaunchKernelGGL((mixed_any_kernel<T, NE_>), dim3(n), dim3(256), lds, stream, a);                            \
  }
  if (HV <= 1024) MP_MA(4)
  else if (HV <= 4096) MP_MA(16)
  else if (HV <= 8192) MP_MA(32)
  else if (HV <= 16384) MP_MA(64)
  else return -1;
#undef MP_MA
  return (int)hipGetLastError();
}

template <typename T>
static int launch_prep(const MixedArgs& a, const FfArgs& f, int n, hipStream_t stream) {
  const int nh = (a.H + 2 * a.G + 3) / 4;
  const bool vec = f.F % 8 == 0 && (f.kind < 2 || f.block % 8 == 0) && f.col % 8 == 0 && f.out_col % 8 == 0 &&
                   a.zs % 8 == 0 && a.os % 8 == 0;
  int nf = f.kind ? (f.F + 256 * (vec ? 8 : 1) - 1) / (256 * (vec ? 8 : 1)) : 0;
  if (nf > 64) nf = 64;
  if constexpr (sizeof(T) == 2) {
    const int vecs = ((a.H + a.G) * a.D + a.G * a.V) / 8;
    if (vec && a.D % 8 == 0 && a.V % 16 == 0 && a.rot % 16 == 0 && vecs <= PREP_VECS) {
      hipLaunchKernelGGL(mixed_prep_vec_kernel, dim3(n, 1 + nf), dim3(256), vecs * 20, stream, a, f);
      return (int)hipGetLastError();
    }
  }
  if (vec) hipLaunchKernelGGL((mixed_prep_kernel<T, 8>), dim3(n, nh + nf), dim3(256), 0, stream, a, f, nh);
  else hipLaunchKernelGGL((mixed_prep_kernel<T, 1>), dim3(n, nh + nf), dim3(256), 0, stream, a, f, nh);
  return (int)hipGetLastError();
}

template <typename T>
static int launch_ffn(const T* z, int64_t zs, T* out, int64_t os, int mt, const FfArgs& f, int n, hipStream_t stream) {
  const bool vec = f.F % 8 == 0 && (f.kind < 2 || f.block % 8 == 0) && zs % 8 == 0 && os % 8 == 0;
  int nf = (f.F + 256 * (vec ? 8 : 1) - 1) / (256 * (vec ? 8 : 1));
  if (nf > 64) nf = 64;
  if (vec) hipLaunchKernelGGL((ffn_act_kernel<T, 8>), dim3(n, nf), dim3(256), 0, stream, z, zs, out, os, mt, f);
  else hipLaunchKernelGGL((ffn_act_kernel<T, 1>), dim3(n, nf), dim3(256), 0, stream, z, zs, out, os, mt, f);
  return (int)hipGetLastError();
}

}  // namespace mp

extern "C" int mp_mixed_prep(const void* z, int64_t zs, const float* qg, const float* kg, void* qn, void* cache,
                             const int64_t* slots, const int32_t* q_ctx, const float* rope, int rot, const float* vrope,
                             void* out, int64_t os, int packed_mt, int kind, int F, int block, int col, int out_col,
                             float limit, int n, int H, int G, int D, int V, int page_log2, float eps, int f32,
                             hipStream_t stream) {
  using namespace mp;
  (void)hipGetLastError();
  if (n == 0) return 0;
  if (D > MIX_HEAD || V > MIX_HEAD || rot > D || rot % 2 || V % 2) return -1;
  MixedArgs a{};
  a.z = z, a.zs = zs, a.qg = qg, a.kg = kg, a.qn = qn, a.cache = cache, a.slots = slots, a.q_ctx = q_ctx;
  a.rope = rope, a.rot = rot, a.vrope = vrope, a.out = out, a.os = os, a.packed_mt = packed_mt;
  a.H = H, a.G = G, a.D = D, a.V = V, a.page_log2 = page_log2, a.eps = eps;
  const FfArgs f{kind, F, block > 0 ? block : 8, col, out_col, limit};
  return f32 ? launch_prep<float>(a, f, n, stream) : launch_prep<bf16_t>(a, f, n, stream);
}

extern "C" int mp_ffn_act(const void* z, int64_t zs, void* out, int64_t os, int packed_mt, int kind, int F, int block,
                          float limit, int n, int f32, hipStream_t stream) {
  using namespace mp;
  (void)hipGetLastError();
  if (n == 0) return 0;
  const FfArgs f{kind, F, block > 0 ? block : 8, 0, 0, limit};
  return f32 ? launch_ffn<float>((const float*)z, zs, (float*)out, os, packed_mt, f, n, stream)
             : launch_ffn<bf16_t>((const bf16_t*)z, zs, (bf16_t*)out, os, packed_mt, f, n, stream);
}

extern "C" int mp_mixed_any(const void* z, int64_t zs, const void* qn, const float* talk, const void* cache,
                            const int32_t* bt, int bt_stride, const int32_t* q_seq, const int32_t* q_ctx,
                            const float* vrope, void* out, int64_t os, int packed_mt, int n, int H, int G, int D, int V,
                            int page_log2, float scale, float cap, int f32, hipStream_t stream) {
  using namespace mp;
  (void)hipGetLastError();
  if (n == 0) return 0;
  MixedArgs a{};
  a.z = z, a.zs = zs, a.qn = (void*)qn, a.talk = talk, a.cache = (void*)cache, a.bt = bt, a.bt_stride = bt_stride;
  a.q_seq = q_seq, a.q_ctx = q_ctx, a.vrope = vrope, a.out = out, a.os = os, a.packed_mt = packed_mt;
  a.H = H, a.G = G, a.D = D, a.V = V, a.page_log2 = page_log2, a.scale = scale, a.cap = cap;
  return f32 ? launch_mixed_any<float>(a, n, stream) : launch_mixed_any<bf16_t>(a, n, stream);
}
