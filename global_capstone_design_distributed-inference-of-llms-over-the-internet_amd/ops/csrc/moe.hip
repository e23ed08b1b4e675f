// Routed experts of the hybrid decoders: router, choice, and the experts' gated feed-forwards as grouped products.
//
//   moe_router       logits[t, e] = x[t] . router[e] in 32-bit, over K slices
//   moe_choose       softmax over all experts; a group of neighbouring experts counts as its best one; the ``top``
//                    experts with the largest scores among the ``keep`` best groups; weights = scores / (sum + 1e-20)
//                    * scale.  Every choice also gets its place among its expert's rows
//   moe_place        rows sorted by expert: first row of every expert, the token of every row, the row of every choice
//   moe_gemm_any     any shape and both element types
//   moe_gemm_rows    bf16, few rows per expert: weights stream once through registers in fragment order
//   moe_gemm_tile    bf16, many rows per expert: 128 x 128 or 256 x 256 tiles through LDS
//
// The products come in two kinds: gathered rows x gate/up weights with the clamped gated form as epilogue
// (GLU: out = g sigmoid(1.702 g) (u + 1), g <= limit, |u| <= limit), and sorted rows x down weights.
#include "common.h"
#include "act_io.h"

namespace mp {

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8_t;
__device__ __forceinline__ f32x4 mfma_bf(const u16x8& a, const u16x8& b, const f32x4& c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, a), __builtin_bit_cast(bf16x8_t, b), c, 0,
                                                 0, 0);
}

constexpr float MOE_ALPHA = 1.702f;
constexpr int MOE_EXPERTS = 512;
// int32 scratch of a step: [counts E][first row E + 1][active experts E][number of active experts]
struct MoeLists {
  int32_t *cnt, *off, *act, *nact;
};
__host__ __device__ __forceinline__ MoeLists moe_lists(int32_t* p, int E) {
  return MoeLists{p, p + E, p + 2 * E + 1, p + 3 * E + 1};
}

// element offset of x[row, col], row-major (pitch xs) or packed (mt row tiles)
__device__ __forceinline__ int64_t act_at(int row, int col, int64_t xs, int mt) {
  return mt > 0 ? apk_off(row, col, mt) : (int64_t)row * xs + col;
}

__device__ __forceinline__ float moe_glu(float g, float u, float limit) {
  const float a = fminf(g, limit), b = fminf(fmaxf(u, -limit), limit);
  return a / (1.f + __expf(-MOE_ALPHA * a)) * (b + 1.f);
}
__device__ __forceinline__ float moe_glu_exact(float g, float u, float limit) {
  const float a = fminf(g, limit), b = fminf(fmaxf(u, -limit), limit);
  return a / (1.f + expf(-MOE_ALPHA * a)) * (b + 1.f);
}

// ------------------------------------------------------------------------------------ router
// part[s][t][e].  A workgroup: one token, four experts (a wave each), slice s of K.
template <typename T>
__global__ __launch_bounds__(256) void moe_router_any_kernel(const T* __restrict__ x, int64_t xs, int mt,
                                                             const T* __restrict__ w, float* __restrict__ part, int T_,
                                                             int E, int W, int ks, int32_t* __restrict__ cnt) {
  const int t = blockIdx.x, e = blockIdx.y * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63, s = blockIdx.z;
  if (t == 0 && s == 0 && e < E && lane == 0) cnt[e] = 0;
  if (e >= E) return;
  const int k1 = min(W, (s + 1) * ks);
  float a = 0.f;
  for (int k = s * ks + lane; k < k1; k += 64) a += to_f(x[act_at(t, k, xs, mt)]) * to_f(w[(int64_t)e * W + k]);
  a = wave_sum(a);
  if (lane == 0) part[((int64_t)s * T_ + t) * E + e] = a;
}

// 16 tokens x 16 NT experts a workgroup; the slice's 32-column steps go round the waves, U of them in flight
template <int NT, int U>
__global__ __launch_bounds__(256) void moe_router_mfma_kernel(const bf16_t* __restrict__ x, int64_t xs, int mt,
                                                              const bf16_t* __restrict__ w, float* __restrict__ part,
                                                              int T, int E, int W, int ks, int32_t* __restrict__ cnt) {
  __shared__ float red[4][16 * NT * 17];
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, c16 = lane & 15, g4 = lane >> 4;
  const int t0 = blockIdx.x * 16, e0 = blockIdx.y * 16 * NT, s = blockIdx.z;
  if (blockIdx.x == 0 && s == 0 && tid < 16 * NT && e0 + tid < E) cnt[e0 + tid] = 0;
  const int row = min(t0 + c16, T - 1), k1 = min(W, (s + 1) * ks);
  f32x4 acc[NT];
  const bf16_t* wp[NT];
#pragma unroll
  for (int n = 0; n < NT; ++n) {
    acc[n] = (f32x4)(0.f);
    wp[n] = w + (int64_t)min(e0 + 16 * n + c16, E - 1) * W + 8 * g4;
  }
  for (int k = s * ks + 32 * wv; k < k1; k += 128 * U) {
    u16x8 b[U], a[U][NT];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int kk = min(k + 128 * u, W - 32);  // (past the slice: loaded, not used)
      b[u] = *reinterpret_cast<const u16x8*>(x + act_at(row, kk + 8 * g4, xs, mt));
#pragma unroll
      for (int n = 0; n < NT; ++n) a[u][n] = *reinterpret_cast<const u16x8*>(wp[n] + kk);
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (k + 128 * u < k1)  // (uniform)
#pragma unroll
        for (int n = 0; n < NT; ++n) acc[n] = mfma_bf(a[u][n], b[u], acc[n]);  // rows: experts, columns: tokens
  }
#pragma unroll
  for (int n = 0; n < NT; ++n)
#pragma unroll
    for (int r = 0; r < 4; ++r) red[wv][(16 * n + 4 * g4 + r) * 17 + c16] = acc[n][r];
  __syncthreads();
  for (int i = tid; i < 256 * NT; i += 256) {
    const int t = i / (16 * NT), e = i % (16 * NT), at = e * 17 + t;
    if (t0 + t < T && e0 + e < E)
      part[((int64_t)s * T + t0 + t) * E + e0 + e] = red[0][at] + red[1][at] + red[2][at] + red[3][at];
  }
}

// ------------------------------------------------------------------------------------ choice
struct ChooseArgs {
  const float* part;  // [S][T][E]
  const int32_t* ctx;  // [T]; <= 0: a padding row, no choice
  int S, T, E, top, groups, keep;
  float scale;
  float* ew;          // [T, top]
  int32_t* idx;       // [T, top] expert, -1: none
  int32_t* slot;      // [T, top] place among its expert's rows, then (moe_place) the row
  int32_t* lists;     // moe_lists
  int32_t* tok;       // [T top] token of every row
};

constexpr int CH_WAVES = 16, CH_PER = MOE_EXPERTS / 64;

// exclusive prefix of n <= MOE_EXPERTS counts by one wave; returns the total
__device__ __forceinline__ int moe_prefix(const int32_t* cnt, int32_t* off, int n, int lane) {
  int base = 0;
  for (int i = 0; i < n; i += 64) {
    const int v = i + lane < n ? cnt[i + lane] : 0;
    int x = v;
#pragma unroll
    for (int d = 1; d < 64; d <<= 1) {
      const int y = __shfl_up(x, d, 64);
      if (lane >= d) x += y;
    }
    if (i + lane < n) off[i + lane] = base + x - v;
    base += __shfl(x, 63, 64);
  }
  if (lane == 0) off[n] = base;
  return base;
}
// the experts that have rows, in order
__device__ __forceinline__ void moe_active(const int32_t* cnt, const MoeLists& l, int n, int lane) {
  int base = 0;
  for (int i = 0; i < n; i += 64) {
    const bool on = i + lane < n && cnt[i + lane] > 0;
    const unsigned long long m = __ballot(on);
    if (on) l.act[base + __popcll(m & ((1ull << lane) - 1))] = i + lane;
    base += __popcll(m);
  }
  if (lane == 0) *l.nact = base;
}

// ``per`` tokens a wave; one workgroup (gridDim.x == 1): places the rows as well
__global__ __launch_bounds__(CH_WAVES * 64) void moe_choose_kernel(ChooseArgs a, int per) {
  extern __shared__ float sm[];
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, E = a.E, gs = E / a.groups;
  const int nw = blockDim.x >> 6;
  int32_t* hist = (int32_t*)sm;                // [E]
  int32_t* base = hist + E;                    // [E + 1]
  float* z = sm + 2 * E + 1 + wv * 2 * E;      // this wave's logits
  float* gz = z + E;                           // and its groups' best
  const MoeLists l = moe_lists(a.lists, E);
  for (int e = tid; e < E; e += blockDim.x) hist[e] = 0;
  __syncthreads();
  const int t0 = (blockIdx.x * nw + wv) * per;
  // the next token's logits are on their way while this one's experts are ranked
  float nx[CH_PER];
  auto fetch = [&](int t) {
#pragma unroll
    for (int j = 0; j < CH_PER; ++j) {
      const int e = lane + 64 * j;
      nx[j] = 0.f;
      if (64 * j < E) {  // (uniform)
        for (int s = 0; s < a.S; s += 8) {  // eight slices' loads in flight, added in order
          float p[8];
#pragma unroll
          for (int i = 0; i < 8; ++i)
            p[i] = a.part[((int64_t)min(s + i, a.S - 1) * a.T + min(t, a.T - 1)) * E + min(e, E - 1)];
#pragma unroll
          for (int i = 0; i < 8; ++i) nx[j] += s + i < a.S ? p[i] : 0.f;
        }
      }
    }
  };
  fetch(t0);
  for (int i = 0; i < per; ++i) {
    const int t = t0 + i;
    const bool live = t < a.T && a.ctx[t] > 0;
    float cur[CH_PER];
#pragma unroll
    for (int j = 0; j < CH_PER; ++j) cur[j] = nx[j];
    if (i + 1 < per) fetch(t + 1);
    if (t < a.T && !live)
      for (int k = lane; k < a.top; k += 64) a.idx[t * a.top + k] = a.slot[t * a.top + k] = -1, a.ew[t * a.top + k] = 0.f;
    if (live) {
      float v[CH_PER], mx = -INFINITY;
#pragma unroll
      for (int j = 0; j < CH_PER; ++j) {
        const int e = lane + 64 * j;
        v[j] = -INFINITY;
        if (e < E) {
          v[j] = fmaxf(cur[j], -3e38f);  // (not a number: last, so that every rank is taken once)
          z[e] = v[j];
          mx = fmaxf(mx, v[j]);
        }
      }
      mx = wave_max(mx);
      float sum = 0.f;
#pragma unroll
      for (int j = 0; j < CH_PER; ++j) sum += lane + 64 * j < E ? expf(v[j] - mx) : 0.f;
      sum = wave_sum(sum);
      __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
      __builtin_amdgcn_wave_barrier();
      for (int g = lane; g < a.groups; g += 64) {
        float b = z[g * gs];
#pragma unroll 8
        for (int j = 1; j < gs; ++j) b = fmaxf(b, z[g * gs + j]);
        gz[g] = b;
      }
      __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
      __builtin_amdgcn_wave_barrier();
      // an expert of a group that is not kept leaves the contest (a group's rank: how many are better)
      bool in[CH_PER];
#pragma unroll
      for (int j = 0; j < CH_PER; ++j) {
        const int e = lane + 64 * j, g = min(e, E - 1) / gs;
        int better = 0;
        if (e < E)
#pragma unroll 8
          for (int q = 0; q < a.groups; ++q) better += gz[q] > gz[g] || (gz[q] == gz[g] && q < g);
        in[j] = e < E && better < a.keep;
      }
      __builtin_amdgcn_wave_barrier();
#pragma unroll
      for (int j = 0; j < CH_PER; ++j)
        if (lane + 64 * j < E && !in[j]) z[lane + 64 * j] = -INFINITY;
      __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
      __builtin_amdgcn_wave_barrier();
      float s[CH_PER], cs = 0.f;
      int rank[CH_PER];
#pragma unroll
      for (int j = 0; j < CH_PER; ++j) {
        const int e = lane + 64 * j;
        rank[j] = a.top;
        s[j] = 0.f;
        if (in[j]) {
          int better = 0;
#pragma unroll 8
          for (int q = 0; q < E; ++q) better += z[q] > v[j] || (z[q] == v[j] && q < e);
          rank[j] = better;
          if (better < a.top) s[j] = expf(v[j] - mx) / sum;
        }
        cs += s[j];
      }
      cs = wave_sum(cs);
#pragma unroll
      for (int j = 0; j < CH_PER; ++j)
        if (rank[j] < a.top) {
          const int e = lane + 64 * j, at = t * a.top + rank[j];
          a.ew[at] = s[j] / (cs + 1e-20f) * a.scale;
          a.idx[at] = e;
          a.slot[at] = atomicAdd(&hist[e], 1);
        }
    }
  }
  __syncthreads();
  if (gridDim.x > 1) {  // places become places among all workgroups' rows
    for (int e = tid; e < E; e += blockDim.x) base[e] = hist[e] > 0 ? atomicAdd(&l.cnt[e], hist[e]) : 0;
    __syncthreads();
    for (int i = lane; i < per * a.top; i += 64) {
      const int t = t0 + i / a.top, at = t0 * a.top + i;
      if (t < a.T && a.idx[at] >= 0) a.slot[at] += base[a.idx[at]];
    }
    return;
  }
  if (wv == 0) {
    moe_prefix(hist, base, E, lane);
    moe_active(hist, l, E, lane);
  }
  __syncthreads();
  for (int e = tid; e < E; e += blockDim.x) l.cnt[e] = hist[e];
  for (int e = tid; e <= E; e += blockDim.x) l.off[e] = base[e];
  for (int i = lane; i < per * a.top; i += 64) {
    const int t = t0 + i / a.top, at = t0 * a.top + i;
    if (t < a.T && a.idx[at] >= 0) {
      const int r = base[a.idx[at]] + a.slot[at];
      a.slot[at] = r;
      a.tok[r] = t;
    }
  }
}

__global__ __launch_bounds__(256) void moe_place_kernel(ChooseArgs a) {
  __shared__ int32_t off[MOE_EXPERTS + 1];
  const MoeLists l = moe_lists(a.lists, a.E);
  if (threadIdx.x < 64) {
    moe_prefix(l.cnt, off, a.E, threadIdx.x);
    if (blockIdx.x == 0) moe_active(l.cnt, l, a.E, threadIdx.x);
  }
  __syncthreads();
  if (blockIdx.x == 0)
    for (int e = threadIdx.x; e <= a.E; e += 256) l.off[e] = off[e];
  const int i = blockIdx.x * 256 + threadIdx.x;
  if (i < a.T * a.top && a.idx[i] >= 0) {
    const int r = off[a.idx[i]] + a.slot[i];
    a.slot[i] = r;
    a.tok[r] = i / a.top;
  }
}

// ------------------------------------------------------------------------------------ products
struct MoeGemm {
  const void* x;       // rows: x[tok[r]] (gathered; row-major or packed) or x[r]
  int64_t xs;
  int mt;
  const int32_t* tok;  // null: sorted rows
  const int32_t* lists;
  const void* w;       // [E, N, K] row-major, or fragment order [E, N / 16, K / 32, 64, 8]
  void* out;           // [rows, N] or (GLU) [rows, N / 2]
  int E, N, K, block;  // block: rows of a gate / up block
  float limit;
};

// 32 rows x 32 outputs a workgroup
template <typename T, bool GLU>
__global__ __launch_bounds__(256) void moe_gemm_any_kernel(MoeGemm a) {
  __shared__ float xa[32][33], wa[2][32][33];
  const MoeLists l = moe_lists(const_cast<int32_t*>(a.lists), a.E);
  if ((int)blockIdx.y >= *l.nact) return;
  const int e = l.act[blockIdx.y], r0 = l.off[e], n = l.cnt[e], O = GLU ? a.N / 2 : a.N, o0 = blockIdx.x * 32;
  const int tid = threadIdx.x, tr = tid >> 3, tc = tid & 7;
  const T* w = (const T*)a.w + (int64_t)e * a.N * a.K;
  for (int m0 = 0; m0 < n; m0 += 32) {
    float acc[2][4] = {};
    for (int k0 = 0; k0 < a.K; k0 += 32) {
      __syncthreads();
      for (int i = tid; i < 1024; i += 256) {
        const int r = i >> 5, k = k0 + (i & 31);
        const int m = r0 + min(m0 + r, n - 1), row = a.tok ? a.tok[m] : m;
        xa[r][i & 31] = k < a.K ? to_f(((const T*)a.x)[act_at(row, k, a.xs, a.mt)]) : 0.f;
        const int o = min(o0 + r, O - 1);
#pragma unroll
        for (int h = 0; h < (GLU ? 2 : 1); ++h) {
          const int wr = GLU ? o / a.block * 2 * a.block + h * a.block + o % a.block : o;
          wa[h][r][i & 31] = k < a.K ? to_f(w[(int64_t)wr * a.K + k]) : 0.f;
        }
      }
      __syncthreads();
      for (int k = 0; k < 32; ++k)
#pragma unroll
        for (int c = 0; c < 4; ++c) {
          acc[0][c] += xa[tr][k] * wa[0][tc + 8 * c][k];
          if (GLU) acc[1][c] += xa[tr][k] * wa[1][tc + 8 * c][k];
        }
    }
    if (m0 + tr < n)
#pragma unroll
      for (int c = 0; c < 4; ++c) {
        const int o = o0 + tc + 8 * c;
        if (o >= O) continue;
        const int64_t at = (int64_t)(r0 + m0 + tr) * O + o;
        if (GLU) from_f(moe_glu_exact(acc[0][c], acc[1][c], a.limit), ((T*)a.out)[at]);
        else ((float*)a.out)[at] = acc[0][c];
      }
  }
}

// Few rows per expert.  A workgroup makes 32 weight rows' outputs (two fragment tiles: one gate / up pair) for up to 64
// rows at a time; its four waves take the 32-column steps in turn, so that together they stream 4 KiB runs of packed
// weights, and their sums meet in LDS.  D = W x^T: a lane owns one row and four neighbouring outputs.
template <bool GLU, int NR, int U>
__device__ __forceinline__ void moe_rows_pass(const MoeGemm& a, const bf16_t* __restrict__ w0, const bf16_t* __restrict__ w1,
                                              int r0, int m0, int n, int o0, int nt1, float* red) {
  const int tid = threadIdx.x, lane = tid & 63, c16 = lane & 15, g4 = lane >> 4;
  const int wv = __builtin_amdgcn_readfirstlane(tid >> 6), ks = a.K >> 5;
  const bf16_t* xp[NR];
  int64_t xstep;  // elements from one 32-column step to the next
  {
    xstep = a.mt > 0 ? (int64_t)a.mt * 512 : 32;
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      const int m = r0 + min(m0 + 16 * i + c16, n - 1), row = a.tok ? a.tok[m] : m;
      xp[i] = (const bf16_t*)a.x + act_at(row, 8 * g4, a.xs, a.mt);
    }
  }
  f32x4 acc[NR][2];
#pragma unroll
  for (int i = 0; i < NR; ++i) acc[i][0] = acc[i][1] = (f32x4)(0.f);
  for (int s0 = wv; s0 < ks; s0 += 4 * U) {
    u16x8 wf[U][2], xf[U][NR];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int64_t st = min(s0 + 4 * u, ks - 1);
      wf[u][0] = *reinterpret_cast<const u16x8*>(w0 + st * 512 + lane * 8);
      wf[u][1] = *reinterpret_cast<const u16x8*>(w1 + st * 512 + lane * 8);
#pragma unroll
      for (int i = 0; i < NR; ++i) xf[u][i] = *reinterpret_cast<const u16x8*>(xp[i] + st * xstep);
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (s0 + 4 * u < ks)  // (uniform)
#pragma unroll
        for (int i = 0; i < NR; ++i)
#pragma unroll
          for (int h = 0; h < 2; ++h) acc[i][h] = mfma_bf(wf[u][h], xf[u][i], acc[i][h]);
  }
  __syncthreads();  // (the previous pass has read its sums)
#pragma unroll
  for (int i = 0; i < NR; ++i)
#pragma unroll
    for (int h = 0; h < 2; ++h) *reinterpret_cast<f32x4*>(red + ((((wv * NR + i) * 2 + h) * 64) + lane) * 4) = acc[i][h];
  __syncthreads();
  for (int q = tid; q < 128 * NR; q += 256) {  // (row tile, half, lane)
    const int i = q >> 7, h = (q >> 6) & 1, ln = q & 63, m = m0 + 16 * i + (ln & 15);
    if (GLU && h) continue;
    f32x4 v[2];
#pragma unroll
    for (int k = 0; k < 2; ++k) {
      v[k] = (f32x4)(0.f);
      if (GLU || k == h)
#pragma unroll
        for (int w = 0; w < 4; ++w) v[k] += *reinterpret_cast<const f32x4*>(red + ((((w * NR + i) * 2 + k) * 64) + ln) * 4);
    }
    if (m >= n) continue;
    if (GLU) {
      float y[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) y[r] = moe_glu(v[0][r], v[1][r], a.limit);
      st_vec<4>((bf16_t*)a.out + (int64_t)(r0 + m) * (a.N / 2) + o0 / 2 + 4 * (ln >> 4), y);
    } else if (h == 0 || nt1) {
      *reinterpret_cast<f32x4*>((float*)a.out + (int64_t)(r0 + m) * a.N + o0 + 16 * h + 4 * (ln >> 4)) = v[h];
    }
  }
}

template <bool GLU>
__global__ __launch_bounds__(256) void moe_gemm_rows_kernel(MoeGemm a) {
  __shared__ __attribute__((aligned(16))) float red[4 * 4 * 2 * 64 * 4];
  const MoeLists l = moe_lists(const_cast<int32_t*>(a.lists), a.E);
  if ((int)blockIdx.y >= *l.nact) return;
  const int e = l.act[blockIdx.y], r0 = l.off[e], n = l.cnt[e], nt = a.N / 16, t0 = 2 * blockIdx.x, t1 = min(t0 + 1, nt - 1);
  const int64_t tile = (int64_t)a.K * 16;
  const bf16_t* w = (const bf16_t*)a.w + (int64_t)e * a.N * a.K;
  for (int m0 = 0; m0 < n; m0 += 64) {
    const int left = n - m0;
    if (left <= 16) moe_rows_pass<GLU, 1, 8>(a, w + t0 * tile, w + t1 * tile, r0, m0, n, 16 * t0, t1 > t0, red);
    else if (left <= 32) moe_rows_pass<GLU, 2, 4>(a, w + t0 * tile, w + t1 * tile, r0, m0, n, 16 * t0, t1 > t0, red);
    else moe_rows_pass<GLU, 4, 4>(a, w + t0 * tile, w + t1 * tile, r0, m0, n, 16 * t0, t1 > t0, red);
  }
}

// Many rows per expert: WM x WN waves of MW x NW fragment tiles (rows x weight rows), 32 columns a stage.  Both operands
// arrive in LDS in fragment order (global_load_lds, 1 KiB a wave: packed weights as they lie, rows gathered by lane)
// through a ring of MG_P slots, MG_P - 1 of them in flight.
constexpr int MG_P = 4;

__device__ __forceinline__ int moe_tile_count(const MoeLists& l, int E, int i, int lane, int bm) {
  return i + lane < E ? (l.cnt[i + lane] + bm - 1) / bm : 0;
}

template <bool GLU, typename TO, int MW, int NW, int WM, int WN>
__global__ __launch_bounds__(WM * WN * 64) void moe_gemm_tile_kernel(MoeGemm a) {
  constexpr int BM = 16 * MW * WM, BN = 16 * NW * WN, FX = BM / 16, J = (BM + BN) / 16 / (WM * WN), SLOT = (BM + BN) * 64;
  static_assert((BM + BN) / 16 % (WM * WN) == 0, "whole fragments a wave");
  extern __shared__ __attribute__((aligned(1024))) char smem[];
  __shared__ int pick[4];
  const MoeLists l = moe_lists(const_cast<int32_t*>(a.lists), a.E);
  const int tid = threadIdx.x, lane = tid & 63, c16 = lane & 15, g4 = lane >> 4;
  const int wv = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int ntn = (a.N + BN - 1) / BN;
  if (wv == 0) {  // which tile: experts' row tiles in order, an expert's tiles by weight rows, then rows
    int total = 0;
    for (int i = 0; i < a.E; i += 64) total += moe_tile_count(l, a.E, i, lane, BM);
#pragma unroll
    for (int d = 32; d > 0; d >>= 1) total += __shfl_xor(total, d, 64);
    const int all = total * ntn, per = (all + 7) / 8;  // a contiguous run of tiles per XCD
    const int id = ((int)blockIdx.x & 7) * per + ((int)blockIdx.x >> 3);
    const bool on = ((int)blockIdx.x >> 3) < per && id < all;
    if (lane == 0) pick[0] = -1;
    int base = 0;
    for (int i = 0; i < a.E && on; i += 64) {
      const int c = moe_tile_count(l, a.E, i, lane, BM);
      int x = c;
#pragma unroll
      for (int d = 1; d < 64; d <<= 1) {
        const int y = __shfl_up(x, d, 64);
        if (lane >= d) x += y;
      }
      const int lo = (base + x - c) * ntn, hi = (base + x) * ntn;
      if (id >= lo && id < hi) {
        pick[0] = i + lane;
        pick[1] = (id - lo) / c;
        pick[2] = (id - lo) % c;
      }
      base += __shfl(x, 63, 64);
    }
  }
  __syncthreads();
  const int e = pick[0];
  if (e < 0) return;
  const int n0 = pick[1] * BN, m0 = pick[2] * BM, r0 = l.off[e], n = l.cnt[e], nt = a.N / 16, ks = a.K / 32;
  const bf16_t* w = (const bf16_t*)a.w + (int64_t)e * a.N * a.K;
  const bf16_t* fp[J];  // this wave's fragments of a stage, and their step to the next one
  int fs[J];
#pragma unroll
  for (int j = 0; j < J; ++j) {
    const int f = wv * J + j;
    if (f < FX) {
      const int m = r0 + min(m0 + 16 * f + c16, n - 1), row = a.tok ? a.tok[m] : m;
      fp[j] = (const bf16_t*)a.x + (int64_t)row * a.xs + 8 * g4;
      fs[j] = 32;
    } else {
      fp[j] = w + (int64_t)min(n0 / 16 + f - FX, nt - 1) * a.K * 16 + lane * 8;
      fs[j] = 512;
    }
  }
  typedef __attribute__((address_space(3))) void* lptr_t;
  typedef __attribute__((address_space(1))) const void* gptr_t;
  auto issue = [&](int st) {
    char* b = smem + (st & (MG_P - 1)) * SLOT + wv * J * 1024;
    const int k = min(st, ks - 1);  // (past the end: a slot that is not read)
#pragma unroll
    for (int j = 0; j < J; ++j)
      __builtin_amdgcn_global_load_lds((gptr_t)(fp[j] + (int64_t)k * fs[j]), (lptr_t)(b + j * 1024), 16, 0, 0);
  };
  const int wm = wv % WM, wn = wv / WM;
  f32x4 acc[NW][MW];
#pragma unroll
  for (int i = 0; i < NW; ++i)
#pragma unroll
    for (int j = 0; j < MW; ++j) acc[i][j] = (f32x4)(0.f);
#pragma unroll
  for (int p = 0; p < MG_P - 1; ++p) issue(p);
  for (int st = 0; st < ks; ++st) {
    asm volatile("s_waitcnt vmcnt(%0)" ::"n"(J * (MG_P - 2)) : "memory");
    lds_wait_barrier();  // stage st has landed for all waves, and all have read stage st - 1
    issue(st + MG_P - 1);
    const char* b = smem + (st & (MG_P - 1)) * SLOT + lane * 16;
    u16x8 xf[MW], wf[NW];
#pragma unroll
    for (int j = 0; j < MW; ++j) xf[j] = *reinterpret_cast<const u16x8*>(b + (MW * wm + j) * 1024);
#pragma unroll
    for (int i = 0; i < NW; ++i) wf[i] = *reinterpret_cast<const u16x8*>(b + (FX + NW * wn + i) * 1024);
#pragma unroll
    for (int i = 0; i < NW; ++i)
#pragma unroll
      for (int j = 0; j < MW; ++j) acc[i][j] = mfma_bf(wf[i], xf[j], acc[i][j]);
  }
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");  // (the ring's last loads end before the workgroup does)
#pragma unroll
  for (int j = 0; j < MW; ++j) {
    const int m = m0 + 16 * (MW * wm + j) + c16;
    if (m >= n) continue;
#pragma unroll
    for (int i = 0; i < NW; i += GLU ? 2 : 1) {
      const int o = n0 + 16 * (NW * wn + i);
      if (o >= a.N) continue;
      float y[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) y[r] = GLU ? moe_glu(acc[i][j][r], acc[GLU ? i + 1 : i][j][r], a.limit) : acc[i][j][r];
      st_vec<4>((TO*)a.out + (int64_t)(r0 + m) * (GLU ? a.N / 2 : a.N) + (GLU ? o / 2 : o) + 4 * g4, y);
    }
  }
}

template <bool GLU, typename TO, int MW, int NW, int WM, int WN>
static int launch_moe_tile(const MoeGemm& a, int rows, int act, hipStream_t stream) {
  constexpr int BM = 16 * MW * WM, BN = 16 * NW * WN, LDS = MG_P * (BM + BN) * 64;
  // (row tiles: at most one more than full ones per expert that has rows)
  const int tiles = (rows / BM + act) * ((a.N + BN - 1) / BN);
  (void)hipFuncSetAttribute((const void*)moe_gemm_tile_kernel<GLU, TO, MW, NW, WM, WN>,
                            hipFuncAttributeMaxDynamicSharedMemorySize, LDS);
  hipLaunchKernelGGL((moe_gemm_tile_kernel<GLU, TO, MW, NW, WM, WN>), dim3((tiles + 7) / 8 * 8), dim3(WM * WN * 64), LDS,
                     stream, a);
  return (int)hipGetLastError();
}

}  // namespace mp

// int32 elements of ``lists``
extern "C" int64_t mp_moe_lists(int E) { return 3 * (int64_t)E + 2; }

// K slices of the router's product over T rows
extern "C" int mp_moe_router_splits(int T, int W, int E, int f32) {
  if (f32) return 1;
  const int tiles = ((T + 15) / 16) * ((E + 63) / 64);
  int s = 256 / (tiles > 0 ? tiles : 1);
  if (s > W / 256) s = W / 256;
  return s < 1 ? 1 : s > 16 ? 16 : s;
}

extern "C" int mp_moe_route(const void* x, int64_t xs, int mt, const void* w, const int32_t* ctx, float* part, int S,
                            float* ew, int32_t* idx, int32_t* slot, int32_t* lists, int32_t* tok, int T, int E, int W,
                            int top, int groups, int keep, float scale, int f32, hipStream_t stream) {
  using namespace mp;
  (void)hipGetLastError();
  if (T == 0) return 0;
  if (E > MOE_EXPERTS || E < 1 || groups < 1 || E % groups || keep > groups || top > E) return -1;
  const MoeLists l = moe_lists(lists, E);
  int ks = (W + S - 1) / S;
  ks = (ks + 31) / 32 * 32;
  if (!f32 && W % 32 == 0 && (mt > 0 || xs % 8 == 0)) {
#define MP_RT(NT_, U_)                                                                                                  \
  hipLaunchKernelGGL((moe_router_mfma_kernel<NT_, U_>), dim3((T + 15) / 16, (E + 16 * NT_ - 1) / (16 * NT_), S),        \
                     dim3(256), 0, stream, (const bf16_t*)x, xs, mt, (const bf16_t*)w, part, T, E, W, ks, l.cnt)
    if (E <= 16) MP_RT(1, 8);
    else if (E <= 32) MP_RT(2, 8);
    else MP_RT(4, 4);
#undef MP_RT
  } else {
    const dim3 grid(T, (E + 3) / 4, S);
    if (f32)
      hipLaunchKernelGGL(moe_router_any_kernel<float>, grid, dim3(256), 0, stream, (const float*)x, xs, mt,
                         (const float*)w, part, T, E, W, ks, l.cnt);
    else
      hipLaunchKernelGGL(moe_router_any_kernel<bf16_t>, grid, dim3(256), 0, stream, (const bf16_t*)x, xs, mt,
                         (const bf16_t*)w, part, T, E, W, ks, l.cnt);
  }
  const ChooseArgs a{part, ctx, S, T, E, top, groups, keep, scale, ew, idx, slot, lists, tok};
  const int nw = E <= 256 ? CH_WAVES : CH_WAVES / 2;  // (LDS: 8 E bytes a wave)
  const size_t lds = (2 * E + 1 + nw * 2 * E) * sizeof(float);
  // one token a wave as long as that fills no more than the chip; a single workgroup also places the rows
  const int per = (T + 256 * nw - 1) / (256 * nw), nb = (T + nw * per - 1) / (nw * per);
  hipLaunchKernelGGL(moe_choose_kernel, dim3(nb), dim3(nw * 64), lds, stream, a, per);
  if (nb > 1) hipLaunchKernelGGL(moe_place_kernel, dim3((T * top + 255) / 256), dim3(256), 0, stream, a);
  return (int)hipGetLastError();
}

// form 0: any shape, 1: few rows per expert, 2: many, 3: very many
extern "C" int mp_moe_gemm(int form, int glu, const void* x, int64_t xs, int mt, const int32_t* tok,
                           const int32_t* lists, const void* w, void* out, int out_f32, int rows, int E, int N, int K,
                           int block, float limit, int f32, hipStream_t stream) {
  using namespace mp;
  (void)hipGetLastError();
  if (rows == 0) return 0;
  const MoeGemm a{x, xs, mt, tok, lists, w, out, E, N, K, block, limit};
  const int act = rows < E ? rows : E, O = glu ? N / 2 : N;
  const dim3 grid((O + 31) / 32, act);
  if (form) {
    if (f32 || N % 16 || K % 32 || (glu && (N % 32 || block != 16))) return -1;
    if (form == 1) {
      if (!glu && !out_f32) return -1;
      const dim3 g((N / 16 + 1) / 2, act);
      if (glu) hipLaunchKernelGGL((moe_gemm_rows_kernel<true>), g, dim3(256), 0, stream, a);
      else hipLaunchKernelGGL((moe_gemm_rows_kernel<false>), g, dim3(256), 0, stream, a);
      return (int)hipGetLastError();
    }
    if (mt > 0) return -1;
    // 256 x 256 tiles where an expert's rows fill them, else 128 x 128
    const bool big = form == 3;
#define MP_MT(GLU_, TO_)                                                       \
  return big ? launch_moe_tile<GLU_, TO_, 4, 8, 4, 2>(a, rows, act, stream) \
             : launch_moe_tile<GLU_, TO_, 4, 4, 2, 2>(a, rows, act, stream);
    if (glu) MP_MT(true, bf16_t)
    if (out_f32) MP_MT(false, float)
    MP_MT(false, bf16_t)
#undef MP_MT
  }
  if (!glu && !out_f32) return -1;
  if (f32) {
    if (glu) hipLaunchKernelGGL((moe_gemm_any_kernel<float, true>), grid, dim3(256), 0, stream, a);
    else hipLaunchKernelGGL((moe_gemm_any_kernel<float, false>), grid, dim3(256), 0, stream, a);
  } else {
    if (glu) hipLaunchKernelGGL((moe_gemm_any_kernel<bf16_t, true>), grid, dim3(256), 0, stream, a);
    else hipLaunchKernelGGL((moe_gemm_any_kernel<bf16_t, false>), grid, dim3(256), 0, stream, a);
  }
  return (int)hipGetLastError();
}
