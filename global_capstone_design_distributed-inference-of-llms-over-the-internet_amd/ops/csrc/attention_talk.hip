// Chunked talking-heads attention over a shared key/value cache, gfx950.
//
// A key and its value are the same projected row: the cache holds the raw row once per kv head plus
// one fp32 number per token, the reciprocal root mean square r_j of the whole row (all kv heads at once).
// The key norm's weight is folded into the query, so the raw score of query head g is
//   s_g(i, j) = scale r_j (q'_g(i) . c_{kv(g)}(j)) - slope_g (i - j),   slope_g = 2^(-8 (g + 1) / H)
// with q' = rms(q) * wq * wk; the heads' scores are mixed, m_h = sum_g T[h, g] s_g, and
//   o_h(i) = softmax_j(m_h)(i) c_{kv(h)}(j) * sigmoid(gate_h(i))
// over the keys j <= i of i's own chunk (floor(j / size) = floor(i / size)).  Scores and softmax are fp32.
//
//   talk_prep_kernel    norms of a projected row [q (H D) | k (G D) | gate (H D)], cache write, q'
//   talk_attn_kernel    any shape and both element types: one workgroup per query token
#include "common.h"
#include "act_io.h"

namespace mp {

struct TalkArgs {
  const void* z;         // [T, zs] projected rows
  int64_t zs;
  void* qn;              // [T, H D] q'
  const float* wqk;      // [H D] query norm weight x the kv head's key norm weight
  const float* talk;     // [H, H]
  void* cache;           // [pages, G, page, D]
  float* rk;             // [pages, page]
  const int64_t* slots;
  const int32_t* bt;
  int bt_stride;
  const int32_t *q_seq, *q_ctx;
  void* out;             // [T, H D] row-major or packed
  int H, G, D, page_log2, chunk, packed_mt;
  float scale, eps;
};

template <typename T>
__global__ __launch_bounds__(256) void talk_prep_kernel(TalkArgs a) {
  __shared__ float red[16];
  const int t = blockIdx.x, HD = a.H * a.D, GD = a.G * a.D;
  const int64_t slot = a.slots[t];
  if (slot < 0) return;
  const T* z = (const T*)a.z + (int64_t)t * a.zs;
  float sq = 0.f, sk = 0.f;
  for (int i = threadIdx.x; i < HD; i += 256) {
    const float x = ld_f(z, i);
    sq += x * x;
  }
  for (int i = threadIdx.x; i < GD; i += 256) {
    const float x = ld_f(z, HD + i);
    sk += x * x;
  }
  sq = block_sum(sq, red);
  sk = block_sum(sk, red);
  const float rq = 1.f / sqrtf(sq / (float)HD + a.eps);
  for (int i = threadIdx.x; i < HD; i += 256)
    from_f(ld_f(z, i) * rq * a.wqk[i], ((T*)a.qn)[(int64_t)t * HD + i]);
  const int64_t pg = slot >> a.page_log2, off = slot & ((1 << a.page_log2) - 1);
  for (int i = threadIdx.x; i < GD; i += 256) {
    const int c = i / a.D, d = i - c * a.D;
    ((T*)a.cache)[(((pg * a.G + c) << a.page_log2) + off) * a.D + d] = z[HD + i];
  }
  if (threadIdx.x == 0) a.rk[slot] = 1.f / sqrtf(sk / (float)GD + a.eps);
}

constexpr int TK_TILE = 64;

// NE: accumulators per thread, H D <= 256 NE
template <typename T, int NE>
__global__ __launch_bounds__(256) void talk_attn_kernel(TalkArgs a) {
  extern __shared__ float sm[];
  const int t = blockIdx.x, tid = threadIdx.x, H = a.H, G = a.G, D = a.D, HD = H * D, rep = H / G;
  const int ctx = a.q_ctx[t];
  if (ctx <= 0) return;
  float *sq = sm, *raw = sq + HD, *mix = raw + H * TK_TILE, *sl = mix + H * TK_TILE, *m = sl + H, *l = m + H,
        *al = l + H;
  int* srow = (int*)(al + H);  // key row base of every key of the tile (in rows of D, head 0), r_j beside it
  float* srk = (float*)(srow + TK_TILE);
  for (int i = tid; i < HD; i += 256) sq[i] = ld_f((const T*)a.qn, (int64_t)t * HD + i);
  for (int h = tid; h < H; h += 256) {
    sl[h] = exp2f(-8.f * (float)(h + 1) / (float)H);
    m[h] = -INFINITY;
    l[h] = 0.f;
  }
  float o[NE];
#pragma unroll
  for (int n = 0; n < NE; ++n) o[n] = 0.f;
  const int i = ctx - 1, lo = i / a.chunk * a.chunk;
  const int32_t* bt = a.bt + (int64_t)a.q_seq[t] * a.bt_stride;
  const int pmask = (1 << a.page_log2) - 1;
  for (int j0 = lo; j0 < ctx; j0 += TK_TILE) {
    const int n = min(TK_TILE, ctx - j0);
    __syncthreads();
    for (int j = tid; j < n; j += 256) {
      const int64_t pg = bt[(j0 + j) >> a.page_log2];
      const int off = (j0 + j) & pmask;
      srow[j] = (int)(((pg * G) << a.page_log2) + off);
      srk[j] = a.rk[(pg << a.page_log2) + off];
    }
    __syncthreads();
    for (int e = tid; e < H * n; e += 256) {
      const int g = e / n, j = e - g * n;
      const T* kp = (const T*)a.cache + ((int64_t)srow[j] + ((int64_t)(g / rep) << a.page_log2)) * D;
      float s = 0.f;
      for (int d = 0; d < D; ++d) s += sq[g * D + d] * to_f(kp[d]);
      raw[g * TK_TILE + j] = s * srk[j] * a.scale - sl[g] * (float)(i - j0 - j);
    }
    __syncthreads();
    for (int e = tid; e < H * n; e += 256) {
      const int h = e / n, j = e - h * n;
      float s = 0.f;
      for (int g = 0; g < H; ++g) s += a.talk[h * H + g] * raw[g * TK_TILE + j];
      mix[h * TK_TILE + j] = s;
    }
    __syncthreads();
    for (int h = tid; h < H; h += 256) {
      float mx = m[h];
      for (int j = 0; j < n; ++j) mx = fmaxf(mx, mix[h * TK_TILE + j]);
      const float f = expf(m[h] - mx);
      float s = 0.f;
      for (int j = 0; j < n; ++j) {
        const float p = expf(mix[h * TK_TILE + j] - mx);
        mix[h * TK_TILE + j] = p;
        s += p;
      }
      al[h] = f;
      l[h] = l[h] * f + s;
      m[h] = mx;
    }
    __syncthreads();
#pragma unroll
    for (int k = 0; k < NE; ++k) {
      const int e = tid + 256 * k;
      if (e < HD) {
        const int h = e / D, d = e - h * D;
        const T* vp = (const T*)a.cache + ((int64_t)(h / rep) << a.page_log2) * D + d;
        float s = o[k] * al[h];
        for (int j = 0; j < n; ++j) s += mix[h * TK_TILE + j] * to_f(vp[(int64_t)srow[j] * D]);
        o[k] = s;
      }
    }
  }
  __syncthreads();
  const T* gate = (const T*)a.z + (int64_t)t * a.zs + HD + G * D;
#pragma unroll
  for (int k = 0; k < NE; ++k) {
    const int e = tid + 256 * k;
    if (e < HD) {
      const float gz = ld_f(gate, e);
      st_act((T*)a.out, t, e, HD, a.packed_mt, o[k] / l[e / D] / (1.f + expf(-gz)));
    }
  }
}

template <typename T>
static int launch_talk(const TalkArgs& a, int n, hipStream_t stream) {
  const int HD = a.H * a.D;
  const size_t lds = (HD + 2 * a.H * TK_TILE + 4 * a.H + 2 * TK_TILE) * sizeof(float);
  if (lds > 64000) return -1;
#define MP_TA(NE_) hipLaunchKernelGGL((talk_attn_kernel<T, NE_>), dim3(n), dim3(256), lds, stream, a)
  if (HD <= 1024) MP_TA(4);
  else if (HD <= 4096) MP_TA(16);
  else if (HD <= 8192) MP_TA(32);
  else return -1;
#undef MP_TA
  return (int)hipGetLastError();
}

}  // namespace mp

extern "C" int mp_talk_prep(const void* z, int64_t zs, void* qn, const float* wqk, void* cache, float* rk,
                            const int64_t* slots, int n, int H, int G, int D, int page_log2, float eps, int f32,
                            hipStream_t stream) {
  using namespace mp;
  (void)hipGetLastError();
  if (n == 0) return 0;
  TalkArgs a{};
  a.z = z, a.zs = zs, a.qn = qn, a.wqk = wqk, a.cache = cache, a.rk = rk, a.slots = slots;
  a.H = H, a.G = G, a.D = D, a.page_log2 = page_log2, a.eps = eps;
  if (f32) hipLaunchKernelGGL(talk_prep_kernel<float>, dim3(n), dim3(256), 0, stream, a);
  else hipLaunchKernelGGL(talk_prep_kernel<bf16_t>, dim3(n), dim3(256), 0, stream, a);
  return (int)hipGetLastError();
}

extern "C" int mp_talk_attention(const void* z, int64_t zs, const void* qn, const float* talk, const void* cache,
                                 const float* rk, const int32_t* bt, int bt_stride, const int32_t* q_seq,
                                 const int32_t* q_ctx, void* out, int n, int H, int G, int D, int page_log2, int chunk,
                                 float scale, int packed_mt, int f32, hipStream_t stream) {
  using namespace mp;
  (void)hipGetLastError();
  if (n == 0) return 0;
  TalkArgs a{};
  a.z = z, a.zs = zs, a.qn = (void*)qn, a.talk = talk, a.cache = (void*)cache, a.rk = (float*)rk, a.bt = bt;
  a.bt_stride = bt_stride, a.q_seq = q_seq, a.q_ctx = q_ctx, a.out = out;
  a.H = H, a.G = G, a.D = D, a.page_log2 = page_log2, a.chunk = chunk, a.packed_mt = packed_mt, a.scale = scale;
  return f32 ? launch_talk<float>(a, n, stream) : launch_talk<bf16_t>(a, n, stream);
}
