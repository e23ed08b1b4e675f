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
//   talk_mfma_kernel    bf16, head size <= 128: prompts and decode on MFMA, the head mixing folded into
//                       the queries
//   talk_merge_kernel   merges the context splits of a decode step, applies the gate
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

// ---------------------------------------------------------------------------------------
// MFMA form.  The mixing is linear in the scores, so it moves to the queries: over the concatenation of all
// kv heads' rows (the "wide key", G Dp columns, Dp = D rounded up to 32)
//   m_h(i, j) = scale r_j (u_h(i) . c(j)) - sigma_h (i - j)
//   u_h[kv head c] = sum_{g in c's group} T[h, g] q'_g      sigma_h = sum_g T[h, g] slope_g
// and every query head reads the same wide key: K and V come from LDS once for all heads of a token block,
// and one cached row serves as key (all columns) and value (its head's columns).
//
// A workgroup owns ``ntok`` consecutive query tokens of one sequence.  A unit is (kv head c, 16 rows), row =
// token x the group's query heads; each wave holds UPW units: u in registers as the B operand of
// S^T = K u^T (v_mfma_f32_16x16x32_bf16), so a lane owns one query row and the softmax is lane-local plus
// two shuffles; P^T is the B operand of O^T += V^T P^T straight from the accumulators.  The weights stay
// 32-bit in effect: P = hi + lo in two bf16 MFMAs.  V^T comes from the row-major tile by transposed LDS
// reads.  Tiles of 32 keys, aligned to 32 (so within a page), double-buffered through registers.
typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8_t;
typedef short s16x4_t __attribute__((ext_vector_type(4)));

__device__ __forceinline__ f32x4 mfma_bf(const u16x8& a, const u16x8& b, const f32x4& c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, a), __builtin_bit_cast(bf16x8_t, b), c, 0,
                                                 0, 0);
}
__device__ __forceinline__ u16x4 lds_tr4(const bf16_t* p) {
  const s16x4_t v = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4_t*)(p));
  return __builtin_bit_cast(u16x4, v);
}

typedef __attribute__((ext_vector_type(4))) unsigned u32x4_t;
typedef __attribute__((ext_vector_type(2))) float f32x2_t;
typedef __attribute__((ext_vector_type(2))) __bf16 bf16x2_t;
__device__ __forceinline__ unsigned pk2_bf(float a, float b) {
  return __builtin_bit_cast(unsigned, __builtin_convertvector((f32x2_t){a, b}, bf16x2_t));
}

constexpr int TM_KEYS = 32;

// DH: 32-column slices per head (Dp = 32 DH); KF: slices of the wide key the kernel is built for
// (G DH <= KF, the rest zero); NW waves; UPW units per wave
template <int DH, int KF, int UPW, int NW>
__global__ __launch_bounds__(NW * 64, KF * UPW > 32 ? 1 : 2) void talk_mfma_kernel(TalkArgs a,
                                                                                 const int32_t* __restrict__ blk,
                                                                                 int nblk, int PS,
                                                                                 float* __restrict__ part,
                                                                                 int T) {
  constexpr int DP = 32 * DH, WC = 32 * KF, STR = WC + 8, NT = NW * 64;
  constexpr int CPT = (TM_KEYS * WC / 8 + NT - 1) / NT;
  __shared__ __attribute__((aligned(16))) bf16_t kt[2][TM_KEYS * STR];
  __shared__ __attribute__((aligned(16))) float rks[2][TM_KEYS];

  const int tid = threadIdx.x, lane = tid & 63, c16 = lane & 15, g4 = lane >> 4;
  const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int H = a.H, G = a.G, D = a.D, HD = H * D, rep = H / G;
  const int bx = blk ? nblk - 1 - (int)blockIdx.x : (int)blockIdx.x;  // (later tokens see more keys: first)
  const int tok0 = blk ? blk[bx] : bx, ntok = blk ? blk[nblk + bx] : 1;
  const int hi = a.q_ctx[tok0 + ntok - 1];
  if (hi <= 0) return;
  const int lo = (a.q_ctx[tok0] - 1) / a.chunk * a.chunk;
  const int nrb = (ntok * rep + 15) >> 4, units = G * nrb;
  const int p = blockIdx.z, s_lo = (lo & ~(TM_KEYS - 1)) + p * PS, s_hi = PS > 0 ? min(hi, s_lo + PS) : hi;
  const int32_t* bt = a.bt + (int64_t)a.q_seq[tok0] * a.bt_stride;
  const int pmask = (1 << a.page_log2) - 1;
  constexpr float LOG2E = 1.44269504088896340736f;

  int row_t[UPW], row_h[UPW], klo[UPW], khi[UPW], uc[UPW];
  float sig[UPW];
  u16x8 q[UPW][KF];
  f32x4 o[UPW][2 * DH];
  float m[UPW], l[UPW];
#pragma unroll
  for (int u = 0; u < UPW; ++u) {
    const int unit = ((int)blockIdx.y * NW + w) * UPW + u;
    const int c = unit < units ? unit / nrb : 0;
    const int row = (unit < units ? unit - c * nrb : 0) * 16 + c16;
    const bool ok = unit < units && row < ntok * rep;
    uc[u] = c;
    row_t[u] = ok ? tok0 + row / rep : -1;
    row_h[u] = c * rep + row % rep;
    khi[u] = ok ? a.q_ctx[row_t[u]] : 0;
    klo[u] = ok ? (khi[u] - 1) / a.chunk * a.chunk : 0;
    m[u] = -INFINITY;
    l[u] = 0.f;
#pragma unroll
    for (int t = 0; t < 2 * DH; ++t) o[u][t] = (f32x4)(0.f);
    const float* tr = a.talk + row_h[u] * H;
    float sg = 0.f;
    for (int g = 0; g < H; ++g) sg += tr[g] * exp2f(-8.f * (float)(g + 1) / (float)H);
    sig[u] = sg * LOG2E;
#pragma unroll
    for (int f = 0; f < KF; ++f) {
      const int cc = f / DH, d = (f % DH) * 32 + 8 * g4;
      float x[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
      if (ok && cc < G && d < D) {
        const bf16_t* qp = (const bf16_t*)a.qn + (int64_t)row_t[u] * HD + cc * rep * D + d;
        for (int g = 0; g < rep; ++g) {
          const u16x8 v = *reinterpret_cast<const u16x8*>(qp + g * D);
          const float t = tr[cc * rep + g];
#pragma unroll
          for (int j = 0; j < 8; ++j) x[j] += t * bf2f(v[j]);
        }
      }
      u32x4_t pk;
#pragma unroll
      for (int j = 0; j < 4; ++j) pk[j] = pk2_bf(x[2 * j], x[2 * j + 1]);
      asm volatile("" : "+v"(pk));  // packed here: four registers a slice stay live, not eight
      q[u][f] = __builtin_bit_cast(u16x8, pk);
    }
  }

  u16x8 kreg[CPT];
  float rreg = 0.f;
  auto fetch = [&](int s0) {
    const int64_t pg = bt[s0 >> a.page_log2];
    const bf16_t* base = (const bf16_t*)a.cache + ((pg * G) << a.page_log2) * D + (int64_t)(s0 & pmask) * D;
#pragma unroll
    for (int k = 0; k < CPT; ++k) {
      const int x = tid + NT * k, key = x / (WC / 8), col = (x % (WC / 8)) * 8;
      const int c = col / DP, d = col % DP;
      const bool ok = key < TM_KEYS && c < G && d < D && s0 + key < s_hi;
      kreg[k] = ok ? *reinterpret_cast<const u16x8*>(base + (((int64_t)c << a.page_log2) + key) * D + d) : (u16x8)(0);
    }
    if (tid < TM_KEYS) rreg = s0 + tid < s_hi ? a.rk[(pg << a.page_log2) + (s0 & pmask) + tid] : 0.f;
  };
  auto stash = [&](int buf) {
#pragma unroll
    for (int k = 0; k < CPT; ++k) {
      const int x = tid + NT * k, key = x / (WC / 8), col = (x % (WC / 8)) * 8;
      if (key < TM_KEYS) *reinterpret_cast<u16x8*>(&kt[buf][key * STR + col]) = kreg[k];
    }
    if (tid < TM_KEYS) rks[buf][tid] = rreg * a.scale * LOG2E;
  };

  if (s_lo < s_hi) {
    fetch(s_lo);
    stash(0);
  }
  __syncthreads();
  int cur = 0;
  for (int s0 = s_lo; s0 < s_hi; s0 += TM_KEYS, cur ^= 1) {
    const bool more = s0 + TM_KEYS < s_hi;
    if (more) fetch(s0 + TM_KEYS);
    const bf16_t* tb = kt[cur];
    f32x4 st[UPW][2];
#pragma unroll
    for (int u = 0; u < UPW; ++u) st[u][0] = st[u][1] = (f32x4)(0.f);
#pragma unroll
    for (int f = 0; f < KF; ++f)
#pragma unroll
      for (int sub = 0; sub < 2; ++sub) {
        const u16x8 ka = *reinterpret_cast<const u16x8*>(tb + (16 * sub + c16) * STR + 32 * f + 8 * g4);
#pragma unroll
        for (int u = 0; u < UPW; ++u) st[u][sub] = mfma_bf(ka, q[u][f], st[u][sub]);
      }
    f32x4 rr[2];
#pragma unroll
    for (int sub = 0; sub < 2; ++sub) rr[sub] = *reinterpret_cast<const f32x4*>(&rks[cur][16 * sub + 4 * g4]);
#pragma unroll
    for (int u = 0; u < UPW; ++u) {
      float lm = -INFINITY;
#pragma unroll
      for (int sub = 0; sub < 2; ++sub)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int j = s0 + 16 * sub + 4 * g4 + r;
          const float x = st[u][sub][r] * rr[sub][r] - sig[u] * (float)(khi[u] - 1 - j);
          st[u][sub][r] = j >= klo[u] && j < khi[u] && j < s_hi ? x : -INFINITY;
          lm = fmaxf(lm, st[u][sub][r]);
        }
      lm = fmaxf(lm, __shfl_xor(lm, 16, 64));
      lm = fmaxf(lm, __shfl_xor(lm, 32, 64));
      if (__any(lm > m[u])) {
        const float mn = fmaxf(m[u], lm);
        const float al = mn == -INFINITY ? 1.f : __builtin_amdgcn_exp2f(m[u] - mn);
        l[u] *= al;
#pragma unroll
        for (int t = 0; t < 2 * DH; ++t) o[u][t] *= al;
        m[u] = mn;
      }
      const float mu = m[u] == -INFINITY ? 0.f : m[u];
      u16x8 ph, pl;
#pragma unroll
      for (int sub = 0; sub < 2; ++sub)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float x = __builtin_amdgcn_exp2f(st[u][sub][r] - mu);
          l[u] += x;
          ph[4 * sub + r] = f2bf(x);
          pl[4 * sub + r] = f2bf(x - bf2f(ph[4 * sub + r]));
        }
      // V^T: lane c16 of group g4 needs column d = 16 t + c16 of keys 4 g4 .. + 3 (+ 16)
      const bf16_t* vb = tb + (4 * g4 + (c16 >> 2)) * STR + uc[u] * DP + 4 * (c16 & 3);
#pragma unroll
      for (int t = 0; t < 2 * DH; ++t) {
        const u16x4 v0 = lds_tr4(vb + 16 * t), v1 = lds_tr4(vb + 16 * STR + 16 * t);
        const u16x8 va = {v0[0], v0[1], v0[2], v0[3], v1[0], v1[1], v1[2], v1[3]};
        o[u][t] = mfma_bf(va, ph, o[u][t]);
        o[u][t] = mfma_bf(va, pl, o[u][t]);
      }
    }
    if (more) stash(cur ^ 1);
    __syncthreads();
  }
#pragma unroll
  for (int u = 0; u < UPW; ++u) {
    float ls = l[u];
    ls += __shfl_xor(ls, 16, 64);
    ls += __shfl_xor(ls, 32, 64);
    if (row_t[u] < 0) continue;
    const int t = row_t[u], h = row_h[u];
    if (part != nullptr) {  // split context: [NP][T][H][D] sums, then [NP][T][H][2] (max, sum)
      const int64_t pr = ((int64_t)p * T + t) * H + h;
      float* po = part + pr * D;
#pragma unroll
      for (int k = 0; k < 2 * DH; ++k)
        if (16 * k + 4 * g4 < D) *reinterpret_cast<f32x4*>(po + 16 * k + 4 * g4) = o[u][k];
      if (g4 == 0) {
        float* ml = part + (int64_t)gridDim.z * T * HD + pr * 2;
        ml[0] = m[u];
        ml[1] = ls;
      }
      continue;
    }
    const float inv = 1.f / ls;
    const bf16_t* gate = (const bf16_t*)a.z + (int64_t)t * a.zs + HD + G * D + h * D;
#pragma unroll
    for (int k = 0; k < 2 * DH; ++k) {
      const int d = 16 * k + 4 * g4;
      if (d < D) {
        float x[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) x[r] = o[u][k][r] * inv / (1.f + __expf(-bf2f(gate[d + r])));
        st_act_vec<4>((bf16_t*)a.out, t, h * D + d, HD, a.packed_mt, x);
      }
    }
  }
}

__global__ __launch_bounds__(256) void talk_merge_kernel(TalkArgs a, const float* __restrict__ part, int T, int NP) {
  const int t = blockIdx.x, HD = a.H * a.D;
  if (a.q_ctx[t] <= 0) return;
  const float* ml = part + (int64_t)NP * T * HD;
  const bf16_t* gate = (const bf16_t*)a.z + (int64_t)t * a.zs + HD + a.G * a.D;
  for (int e = (blockIdx.y * 256 + threadIdx.x) * 4; e < HD; e += gridDim.y * 1024) {
    const int h = e / a.D;
    float mx = -INFINITY;
    for (int p = 0; p < NP; ++p) mx = fmaxf(mx, ml[(((int64_t)p * T + t) * a.H + h) * 2]);
    f32x4 acc = (f32x4)(0.f);
    float l = 0.f;
    for (int p = 0; p < NP; ++p) {
      const int64_t pr = ((int64_t)p * T + t) * a.H + h;
      const float f = __builtin_amdgcn_exp2f(ml[pr * 2] - mx);  // (an empty split: exp2(-inf) = 0)
      l += f * ml[pr * 2 + 1];
      acc += f * *reinterpret_cast<const f32x4*>(part + pr * a.D + (e - h * a.D));
    }
    float x[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) x[r] = acc[r] / l / (1.f + __expf(-bf2f(gate[e + r])));
    st_act_vec<4>((bf16_t*)a.out, t, e, HD, a.packed_mt, x);
  }
}

// Geometry of the MFMA form for (H, G, D): slices built for, units per workgroup; false: not covered
static bool talk_geometry(int H, int G, int D, int& dh, int& kf, int& upw, int& nw) {
  if (D % 8 || D > 128 || G < 1 || H % G) return false;
  dh = D <= 32 ? 1 : D <= 64 ? 2 : 4;
  kf = G * dh <= 4 ? 4 : G * dh <= 8 ? 8 : G * dh <= 16 ? 16 : 32;
  if (G * dh > kf) return false;
  // (the widest keys: one wave per SIMD with two units' queries in its 512 registers)
  nw = kf == 16 ? 8 : 4;
  upw = kf == 16 ? 1 : 2;
  return true;
}

template <int DH>
static int launch_talk_mfma(const TalkArgs& a, const int32_t* blk, int nblk, int grid_x, int tokens, int PS, int NP,
                            float* part, int T, int kf, hipStream_t stream) {
  const int nw = kf == 16 ? 8 : 4, upw = kf == 16 ? 1 : 2;
  const int units = a.G * ((tokens * (a.H / a.G) + 15) / 16);
  const dim3 grid(grid_x, (units + nw * upw - 1) / (nw * upw), NP);
#define MP_TM(KF_, UPW_, NW_)                                                                                     \
  hipLaunchKernelGGL((talk_mfma_kernel<DH, KF_, UPW_, NW_>), grid, dim3(NW_ * 64), 0, stream, a, blk, nblk, PS, part, T)
  if (kf == 4) MP_TM(4, 2, 4);
  else if (kf == 8) MP_TM(8, 2, 4);
  else if (kf == 16) MP_TM(16, 1, 8);
  else MP_TM(32, 2, 4);
#undef MP_TM
  return (int)hipGetLastError();
}

template <typename T>
static int launch_talk(const TalkArgs& a, int n, hipStream_t stream) {
  const int HD = a.H * a.D;
  const size_t lds = (HD + 2 * a.H * TK_TILE + 4 * a.H + 2 * TK_TILE) * sizeof(float);
  if (lds > 160 * 1024) return -1;
#define MP_TA(NE_)                                                                                            \
  {                                                                                                           \
    if (lds > 65536) /* above the default limit of dynamic LDS */                                             \
      (void)hipFuncSetAttribute((const void*)talk_attn_kernel<T, NE_>, hipFuncAttributeMaxDynamicSharedMemorySize, \
                                (int)lds);                                                                    \
    hipLaunchKernelGGL((talk_attn_kernel<T, NE_>), dim3(n), dim3(256), lds, stream, a);                       \
  }
  if (HD <= 1024) MP_TA(4)
  else if (HD <= 4096) MP_TA(16)
  else if (HD <= 8192) MP_TA(32)
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

// Tokens of a prompt's query block (0: the MFMA form does not cover the shape)
extern "C" int mp_talk_block(int H, int G, int D) {
  using namespace mp;
  int dh, kf, upw, nw;
  if (!talk_geometry(H, G, D, dh, kf, upw, nw)) return 0;
  const int rep = H / G, nrb = nw * upw / G > 1 ? nw * upw / G : 1;
  const int tb = 16 * nrb / rep;
  return tb < 1 ? 1 : tb > 64 ? 64 : tb;
}

// blk [2, nblk] (first token, tokens; tokens <= mp_talk_block): a prompt step; blk == null: n one-token rows, the
// context in NP splits of PS keys (part: NP n (H D + 2 H) floats when NP > 1)
extern "C" int mp_talk_mfma(const void* z, int64_t zs, const void* qn, const float* talk, const void* cache,
                            const float* rk, const int32_t* bt, int bt_stride, const int32_t* q_seq,
                            const int32_t* q_ctx, void* out, int n, int H, int G, int D, int page_log2, int chunk,
                            float scale, const int32_t* blk, int nblk, int PS, int NP, float* part, int packed_mt,
                            hipStream_t stream) {
  using namespace mp;
  (void)hipGetLastError();
  if (n == 0) return 0;
  int dh, kf, upw, nw;
  if (!talk_geometry(H, G, D, dh, kf, upw, nw) || page_log2 < 5) return -1;
  if (NP > 1 && (PS <= 0 || PS % TM_KEYS || part == nullptr || blk != nullptr)) return -2;
  if (NP < 1 || NP > 65535) return -2;
  TalkArgs a{};
  a.z = z, a.zs = zs, a.qn = (void*)qn, a.talk = talk, a.cache = (void*)cache, a.rk = (float*)rk, a.bt = bt;
  a.bt_stride = bt_stride, a.q_seq = q_seq, a.q_ctx = q_ctx, a.out = out;
  a.H = H, a.G = G, a.D = D, a.page_log2 = page_log2, a.chunk = chunk, a.packed_mt = packed_mt, a.scale = scale;
  const int gx = blk ? nblk : n, tokens = blk ? mp_talk_block(H, G, D) : 1;
  float* pp = NP > 1 ? part : nullptr;
  const int ps = NP > 1 ? PS : 0;
  int rc;
  if (dh == 1) rc = launch_talk_mfma<1>(a, blk, nblk, gx, tokens, ps, NP, pp, n, kf, stream);
  else if (dh == 2) rc = launch_talk_mfma<2>(a, blk, nblk, gx, tokens, ps, NP, pp, n, kf, stream);
  else rc = launch_talk_mfma<4>(a, blk, nblk, gx, tokens, ps, NP, pp, n, kf, stream);
  if (rc || NP == 1) return rc;
  const int gy = (H * D / 4 + 255) / 256;
  hipLaunchKernelGGL(talk_merge_kernel, dim3(n, gy), dim3(256), 0, stream, a, part, n, NP);
  return (int)hipGetLastError();
}
