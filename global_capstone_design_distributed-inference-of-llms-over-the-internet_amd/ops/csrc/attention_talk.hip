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
//   talk_xchg_kernel    the same for many heads: raw scores exchanged through LDS, mixed by another MFMA
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
  const float* sigma;    // [H] the mixed slopes, talk @ slope
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

// VEC columns a thread and step; NT threads (decode rows are few: more threads, one round of loads)
template <typename T, int VEC, int NT>
__global__ __launch_bounds__(NT) void talk_prep_kernel(TalkArgs a) {
  __shared__ float red[16];
  const int t = blockIdx.x, HD = a.H * a.D, GD = a.G * a.D;
  const int64_t slot = a.slots[t];
  if (slot < 0) return;
  const T* z = (const T*)a.z + (int64_t)t * a.zs;
  float sq = 0.f, sk = 0.f;
  for (int i = threadIdx.x * VEC; i < HD + GD; i += NT * VEC) {
    float x[VEC], s = 0.f;
    ld_vec<VEC>(z + i, x);
#pragma unroll
    for (int j = 0; j < VEC; ++j) s += x[j] * x[j];
    if (i < HD) sq += s;
    else sk += s;
  }
  sq = block_sum(sq, red);
  sk = block_sum(sk, red);
  const float rq = 1.f / sqrtf(sq / (float)HD + a.eps);
  const int64_t pg = slot >> a.page_log2, off = slot & ((1 << a.page_log2) - 1);
  for (int i = threadIdx.x * VEC; i < HD + GD; i += NT * VEC) {
    float x[VEC];
    ld_vec<VEC>(z + i, x);
    if (i < HD) {
      float g[VEC];
      ld_vec<VEC>(a.wqk + i, g);
#pragma unroll
      for (int j = 0; j < VEC; ++j) x[j] *= rq * g[j];
      st_vec<VEC>((T*)a.qn + (int64_t)t * HD + i, x);
    } else {
      const int c = (i - HD) / a.D, d = i - HD - c * a.D;
      st_vec<VEC>((T*)a.cache + (((pg * a.G + c) << a.page_log2) + off) * a.D + d, x);
    }
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
// log2 units a row's maximum may grow before its sums are rescaled (weights reach 2^8, their sums are fp32)
constexpr float TM_GROW = 8.f;

// first of the 4 head columns in accumulator tile t of lane group g4 (the key tile's column order)
__device__ __forceinline__ int tm_col(int t, int g4) {
  return 32 * (t >> 1) + 16 * (g4 & 1) + 8 * (t & 1) + 4 * (g4 >> 1);
}

// A query row's result: normalised, gated and stored, or left as this split's (maximum, sum, sums).
// PERM: accumulator tile t holds the columns tm_col(t, g4), else 16 t + 4 g4.
template <int DH, bool PERM>
__device__ __forceinline__ void talk_store(const TalkArgs& a, float* __restrict__ part, int T, int p, int t, int h, int g4,
                                           float m, float ls, const f32x4 (&o)[2 * DH]) {
  const int D = a.D, HD = a.H * D;
  if (part != nullptr) {  // split context: [NP][T][H][D] sums, then [NP][T][H][2] (max, sum)
    const int64_t pr = ((int64_t)p * T + t) * a.H + h;
#pragma unroll
    for (int k = 0; k < 2 * DH; ++k) {
      const int d = PERM ? tm_col(k, g4) : 16 * k + 4 * g4;
      if (d < D) *reinterpret_cast<f32x4*>(part + pr * D + d) = o[k];
    }
    if (g4 == 0) {
      float* ml = part + (int64_t)gridDim.z * T * HD + pr * 2;
      ml[0] = m;
      ml[1] = ls;
    }
    return;
  }
  const float inv = 1.f / ls;
  const bf16_t* gate = (const bf16_t*)a.z + (int64_t)t * a.zs + HD + a.G * D + h * D;
#pragma unroll
  for (int k = 0; k < 2 * DH; ++k) {
    const int d = PERM ? tm_col(k, g4) : 16 * k + 4 * g4;
    if (d < D) {
      float x[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) x[r] = o[k][r] * inv / (1.f + __expf(-bf2f(gate[d + r])));
      st_act_vec<4>((bf16_t*)a.out, t, h * D + d, HD, a.packed_mt, x);
    }
  }
}

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
#pragma unroll
    for (int f = 0; f < KF; ++f) q[u][f] = (u16x8)(0);
    const int c = unit < units ? unit / nrb : 0;
    const int row = (unit < units ? unit - c * nrb : 0) * 16 + c16;
    const bool ok = unit < units && row < ntok * rep;
    uc[u] = c;
    row_t[u] = ok ? tok0 + row / rep : -1;
    row_h[u] = c * rep + row % rep;
    const int ctx = a.q_ctx[ok ? row_t[u] : tok0];
    khi[u] = ok ? ctx : 0;
    klo[u] = ok ? (khi[u] - 1) / a.chunk * a.chunk : 0;
    m[u] = -INFINITY;
    l[u] = 0.f;
#pragma unroll
    for (int t = 0; t < 2 * DH; ++t) o[u][t] = (f32x4)(0.f);
    sig[u] = a.sigma[row_h[u]] * LOG2E;
  }

  // The mixed queries: per row block, its tokens' query rows go to LDS as a [32][wide] tile (row = token x group
  // member g, column = kv head c, d) and u^T = Q^T T^T runs on MFMA, T^T block-diagonal over the tokens.  The
  // accumulator leaves lane group g4 with d = 4 g4 + r of both 16-column halves of a slice, so that is the
  // order in which the key tile keeps a slice's columns.
  {
    bf16_t* qt = kt[1];
    for (int rb = 0; rb < nrb; ++rb) {
      const int t0 = rb * 16 / rep, t1 = min((rb * 16 + 15) / rep, ntok - 1), nr = (t1 - t0 + 1) * rep;
      if (rb > 0) __syncthreads();
      // (clamped, unconditional loads: all in flight together)
      u16x8 qreg[CPT];
#pragma unroll
      for (int k = 0; k < CPT; ++k) {
        const int x = tid + NT * k, kr = min(x / (WC / 8), nr - 1), col = (x % (WC / 8)) * 8;
        const int c = min(col / DP, G - 1), d = min(col % DP, D - 8);
        qreg[k] = *reinterpret_cast<const u16x8*>((const bf16_t*)a.qn + (int64_t)(tok0 + t0 + kr / rep) * HD +
                                                  (c * rep + kr % rep) * D + d);
      }
#pragma unroll
      for (int k = 0; k < CPT; ++k) {
        const int x = tid + NT * k, kr = x / (WC / 8), col = (x % (WC / 8)) * 8;
        if (kr < TM_KEYS)
          *reinterpret_cast<u16x8*>(qt + kr * STR + col) =
              kr < nr && col / DP < G && col % DP < D ? qreg[k] : (u16x8)(0);
      }
      __syncthreads();
#pragma unroll
      for (int u = 0; u < UPW; ++u) {
        const int unit = ((int)blockIdx.y * NW + w) * UPW + u;
        if (unit >= units || unit % nrb != rb) continue;  // (uniform over the wave)
        const float* tr = a.talk + row_h[u] * H;
        const int mt = row_t[u] - tok0 - t0;  // this lane's token within the block
        const bf16_t* qb = qt + (8 * g4 + (c16 >> 2)) * STR + 4 * (c16 & 3);
#pragma unroll
        for (int c = 0; c < KF / DH; ++c) {
          u16x8 tb;
#pragma unroll
          for (int j = 0; j < 8; ++j) {
            const int g = 8 * g4 + j - mt * rep;
            const float t = tr[min(c, G - 1) * rep + min(max(g, 0), rep - 1)];
            tb[j] = c < G && row_t[u] >= 0 && g >= 0 && g < rep ? f2bf(t) : (bf16_t)0;
          }
#pragma unroll
          for (int f = c * DH; f < (c + 1) * DH; ++f) {
            f32x4 x[2];
#pragma unroll
            for (int half = 0; half < 2; ++half) {
              const bf16_t* p0 = qb + 32 * f + 16 * half;
              const u16x4 v0 = lds_tr4(p0), v1 = lds_tr4(p0 + 4 * STR);
              const u16x8 va = {v0[0], v0[1], v0[2], v0[3], v1[0], v1[1], v1[2], v1[3]};
              x[half] = mfma_bf(va, tb, (f32x4)(0.f));
            }
            u32x4_t pk = {pk2_bf(x[0][0], x[0][1]), pk2_bf(x[0][2], x[0][3]), pk2_bf(x[1][0], x[1][1]),
                          pk2_bf(x[1][2], x[1][3])};
            asm volatile("" : "+v"(pk));  // packed here: four registers a slice stay live, not eight
            q[u][f] = __builtin_bit_cast(u16x8, pk);
          }
        }
      }
    }
  }

  u16x8 kreg[CPT];
  float rreg = 0.f;
  auto fetch = [&](int s0) {
    const int64_t pg = bt[s0 >> a.page_log2];
    const bf16_t* base = (const bf16_t*)a.cache + ((pg * G) << a.page_log2) * D + (int64_t)(s0 & pmask) * D;
#pragma unroll
    for (int k = 0; k < CPT; ++k) {
      // clamped, unconditional: a column past the head meets a 0 in u, a row past the context is masked
      const int x = tid + NT * k, key = min(x / (WC / 8), s_hi - 1 - s0), col = (x % (WC / 8)) * 8;
      const int c = min(col / DP, G - 1), d = min(col % DP, D - 8);
      kreg[k] = *reinterpret_cast<const u16x8*>(base + (((int64_t)c << a.page_log2) + min(key, TM_KEYS - 1)) * D + d);
    }
    rreg = a.rk[(pg << a.page_log2) + (s0 & pmask) + min(min(tid, TM_KEYS - 1), s_hi - 1 - s0)];
  };
  auto stash = [&](int buf) {
#pragma unroll
    for (int k = 0; k < CPT; ++k) {
      const int x = tid + NT * k, key = x / (WC / 8), col = (x % (WC / 8)) * 8;
      if (key < TM_KEYS) {  // column d of a slice at 8 (d % 16 / 4) + 4 (d / 16) + d % 4
        const int i = (col >> 3) & 3;
        bf16_t* kp = &kt[buf][key * STR + (col & ~31) + 16 * (i & 1) + 4 * (i >> 1)];
        *reinterpret_cast<u16x4*>(kp) = (u16x4){kreg[k][0], kreg[k][1], kreg[k][2], kreg[k][3]};
        *reinterpret_cast<u16x4*>(kp + 8) = (u16x4){kreg[k][4], kreg[k][5], kreg[k][6], kreg[k][7]};
      }
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
      if (__any(lm > m[u] + TM_GROW)) {
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
      // V^T: lane c16 of group g4 needs tile column 16 t + c16 of keys 4 g4 .. + 3 (+ 16)
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
    f32x4 y[2 * DH];
#pragma unroll
    for (int k = 0; k < 2 * DH; ++k) y[k] = o[u][k];
    talk_store<DH, true>(a, part, T, p, row_t[u], row_h[u], g4, m[u], ls, y);
  }
}

// ---------------------------------------------------------------------------------------
// MFMA form for many heads (up to 8 kv heads, 32 query heads): the fold above multiplies the QK work by G, so
// here the raw scores are made once, exchanged through LDS and mixed by another MFMA:
//
//   wave w streams kv head c = w / (8 / G) alone: K fragments go from global memory to registers (the A operand
//   of S^T = K q'^T) and from there to a wave-private LDS tile, which the PV product reads transposed;
//   raw scores, r_j applied, go to LDS as fp32 S[token][key][head];
//   M^T[key, h] = sum_g S^T[key, g] T[h, g] per (token, 16 keys): S splits exactly into three bf16 terms
//   (24 bits), T is bf16 as it comes from the checkpoint;
//   mixed scores return through LDS M[token, head][key]; softmax and O^T += V^T P^T as above.
//
// Two barriers per 32 keys; everything else is private to a wave.
constexpr int TX_NW = 8;

__device__ __forceinline__ u16x8 split_bf(float (&x)[8]) {  // leading bf16 of every x, x <- the remainder (exact)
  u16x8 h;
#pragma unroll
  for (int j = 0; j < 8; ++j) {
    h[j] = f2bf(x[j]);
    x[j] -= bf2f(h[j]);
  }
  return h;
}

struct TalkXchg {  // LDS layout (floats): S at 0, M at m_off, the waves' key tiles (bf16) at k_off
  int hp, s_tok, m_tok, m_off, k_off, nwc, tb;  // (s_tok, m_tok: pitch of a token, padded against bank conflicts)
};

template <int DH, int UPW>
__global__ __launch_bounds__(TX_NW * 64, 2) void talk_xchg_kernel(TalkArgs a, TalkXchg x, const int32_t* __restrict__ blk,
                                                                  int nblk, int PS, float* __restrict__ part, int T) {
  constexpr int STR = 32 * DH + 8, MS = TM_KEYS + 4;
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int tid = threadIdx.x, lane = tid & 63, c16 = lane & 15, g4 = lane >> 4;
  const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int H = a.H, G = a.G, D = a.D, HD = H * D, rep = H / G;
  const int bx = blk ? nblk - 1 - (int)blockIdx.x : (int)blockIdx.x;
  const int tok0 = blk ? blk[bx] : bx, ntok = blk ? blk[nblk + bx] : 1;
  const int hi = a.q_ctx[tok0 + ntok - 1];
  if (hi <= 0) return;
  const int lo = (a.q_ctx[tok0] - 1) / a.chunk * a.chunk;
  const int p = blockIdx.z, s_lo = (lo & ~(TM_KEYS - 1)) + p * PS, s_hi = PS > 0 ? min(hi, s_lo + PS) : hi;
  const int32_t* bt = a.bt + (int64_t)a.q_seq[tok0] * a.bt_stride;
  const int pmask = (1 << a.page_log2) - 1;
  constexpr float LOG2E = 1.44269504088896340736f;
  const float sl2 = a.scale * LOG2E;
  float* sS = sm;
  float* sM = sm + x.m_off;
  bf16_t* kt = reinterpret_cast<bf16_t*>(sm + x.k_off) + w * TM_KEYS * STR;
  const int c = min(w / x.nwc, G - 1);
  const bool streams = w / x.nwc < G && ((w % x.nwc) * UPW) * 16 < ntok * rep;  // this wave has rows

  int khi[UPW], klo[UPW], row_t[UPW], row_h[UPW];
  float sig[UPW], m[UPW], l[UPW];
  u16x8 q[UPW][DH];
  f32x4 o[UPW][2 * DH];
#pragma unroll
  for (int u = 0; u < UPW; ++u) {
    const int row = ((w % x.nwc) * UPW + u) * 16 + c16;
    const bool ok = streams && row < ntok * rep;
    row_t[u] = ok ? row / rep : -1;
    row_h[u] = c * rep + row % rep;
    const int ctx = a.q_ctx[tok0 + max(row_t[u], 0)];
    khi[u] = ok ? ctx : 0;
    klo[u] = ok ? (khi[u] - 1) / a.chunk * a.chunk : 0;
    sig[u] = a.sigma[row_h[u]] * LOG2E;
    m[u] = -INFINITY;
    l[u] = 0.f;
#pragma unroll
    for (int t = 0; t < 2 * DH; ++t) o[u][t] = (f32x4)(0.f);
#pragma unroll
    for (int f = 0; f < DH; ++f) {
      const int d = 32 * f + 8 * g4;
      const u16x8 v = *reinterpret_cast<const u16x8*>((const bf16_t*)a.qn + (int64_t)(tok0 + max(row_t[u], 0)) * HD +
                                                      row_h[u] * D + min(d, D - 8));
      q[u][f] = ok && d < D ? v : (u16x8)(0);
    }
  }
  u16x8 tb[2];  // T^T: column h = 16 hb + c16, k = g = 8 g4 + j
#pragma unroll
  for (int hb = 0; hb < 2; ++hb)
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int h = 16 * hb + c16, g = 8 * g4 + j;
      const float t = a.talk[min(h, H - 1) * H + min(g, H - 1)];
      tb[hb][j] = h < H && g < H ? f2bf(t) : (bf16_t)0;
    }

  u16x8 kf[2][DH];
  f32x4 rr[2];
  auto fetch = [&](int64_t pg, int s0) {
    const int off = s0 & pmask;
    const bf16_t* base = (const bf16_t*)a.cache + (((pg * G + c) << a.page_log2) + off) * D;
    const float* rp = a.rk + (pg << a.page_log2) + off + 4 * g4;
#pragma unroll
    for (int sub = 0; sub < 2; ++sub) {
      rr[sub] = *reinterpret_cast<const f32x4*>(rp + 16 * sub);
#pragma unroll
      for (int f = 0; f < DH; ++f)
        // clamped: a column past the head meets a 0 in q', a row past the context is masked
        kf[sub][f] = *reinterpret_cast<const u16x8*>(base + min(16 * sub + c16, s_hi - 1 - s0) * D +
                                                     min(32 * f + 8 * g4, D - 8));
    }
  };
  int64_t pg1 = 0;
  if (s_lo < s_hi) {
    if (streams) fetch(bt[s_lo >> a.page_log2], s_lo);
    pg1 = bt[min(s_lo + TM_KEYS, s_hi - 1) >> a.page_log2];
  }
  for (int s0 = s_lo; s0 < s_hi; s0 += TM_KEYS) {
    const int64_t pg2 = bt[min(s0 + 2 * TM_KEYS, s_hi - 1) >> a.page_log2];  // a tile ahead of its use
    if (streams) {
#pragma unroll
      for (int sub = 0; sub < 2; ++sub) {
#pragma unroll
        for (int f = 0; f < DH; ++f)
          *reinterpret_cast<u16x8*>(kt + (16 * sub + c16) * STR + 32 * f + 8 * g4) = kf[sub][f];
#pragma unroll
        for (int u = 0; u < UPW; ++u) {
          f32x4 s = (f32x4)(0.f);
#pragma unroll
          for (int f = 0; f < DH; ++f) s = mfma_bf(kf[sub][f], q[u][f], s);
          if (row_t[u] >= 0) {
            float* sp = sS + row_t[u] * x.s_tok + (16 * sub + 4 * g4) * (x.hp + 4) + row_h[u];
#pragma unroll
            for (int r = 0; r < 4; ++r) sp[r * (x.hp + 4)] = s[r] * (rr[sub][r] * sl2);
          }
        }
      }
      if (s0 + TM_KEYS < s_hi) fetch(pg1, s0 + TM_KEYS);
      pg1 = pg2;
    }
    __syncthreads();
    for (int f0 = w; f0 < 2 * ntok; f0 += 2 * TX_NW) {  // (token, 16 keys), two at a time
      float v[2][8];
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        const int fr = min(f0 + i * TX_NW, 2 * ntok - 1);
        ld_vec<8>(sS + (fr >> 1) * x.s_tok + (16 * (fr & 1) + c16) * (x.hp + 4) + min(8 * g4, x.hp - 8), v[i]);
      }
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < 8; ++j) v[i][j] = 8 * g4 + j < H ? v[i][j] : 0.f;  // (columns past H are never written)
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        const int fr = f0 + i * TX_NW;
        const u16x8 v1 = split_bf(v[i]), v2 = split_bf(v[i]), v3 = split_bf(v[i]);
#pragma unroll
        for (int hb = 0; hb < 2; ++hb) {
          f32x4 y = mfma_bf(v3, tb[hb], (f32x4)(0.f));
          y = mfma_bf(v2, tb[hb], y);
          y = mfma_bf(v1, tb[hb], y);
          if (16 * hb + c16 < H && fr < 2 * ntok)
            *reinterpret_cast<f32x4*>(sM + (fr >> 1) * x.m_tok + (16 * hb + c16) * MS + 16 * (fr & 1) + 4 * g4) = y;
        }
      }
    }
    __syncthreads();
    if (!streams) continue;
    u16x8 ph[UPW], pl[UPW];
    f32x4 sc[UPW][2];
#pragma unroll
    for (int u = 0; u < UPW; ++u)
#pragma unroll
      for (int sub = 0; sub < 2; ++sub)
        sc[u][sub] = *reinterpret_cast<const f32x4*>(sM + max(row_t[u], 0) * x.m_tok + row_h[u] * MS + 16 * sub + 4 * g4);
#pragma unroll
    for (int u = 0; u < UPW; ++u) {
      f32x4 (&st)[2] = sc[u];
      float lm = -INFINITY;
      const float dj = (float)(s0 + 4 * g4 - (khi[u] - 1));  // key - query of this lane's first key
      const int k0 = klo[u] - s0 - 4 * g4, k1 = min(khi[u], s_hi) - s0 - 4 * g4;
#pragma unroll
      for (int sub = 0; sub < 2; ++sub)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float y = __builtin_fmaf(dj + (float)(16 * sub + r), sig[u], st[sub][r]);
          st[sub][r] = 16 * sub + r >= k0 && 16 * sub + r < k1 ? y : -INFINITY;
          lm = fmaxf(lm, st[sub][r]);
        }
      lm = fmaxf(lm, __shfl_xor(lm, 16, 64));
      lm = fmaxf(lm, __shfl_xor(lm, 32, 64));
      if (__any(lm > m[u] + TM_GROW)) {
        const float mn = fmaxf(m[u], lm);
        const float al = mn == -INFINITY ? 1.f : __builtin_amdgcn_exp2f(m[u] - mn);
        l[u] *= al;
#pragma unroll
        for (int t = 0; t < 2 * DH; ++t) o[u][t] *= al;
        m[u] = mn;
      }
      const float mu = m[u] == -INFINITY ? 0.f : m[u];
#pragma unroll
      for (int sub = 0; sub < 2; ++sub)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float e = __builtin_amdgcn_exp2f(st[sub][r] - mu);
          l[u] += e;
          ph[u][4 * sub + r] = f2bf(e);
          pl[u][4 * sub + r] = f2bf(e - bf2f(ph[u][4 * sub + r]));
        }
    }
    const bf16_t* vb = kt + (4 * g4 + (c16 >> 2)) * STR + 4 * (c16 & 3);
#pragma unroll
    for (int t = 0; t < 2 * DH; ++t) {
      const u16x4 v0 = lds_tr4(vb + 16 * t), v1 = lds_tr4(vb + 16 * STR + 16 * t);
      const u16x8 va = {v0[0], v0[1], v0[2], v0[3], v1[0], v1[1], v1[2], v1[3]};
#pragma unroll
      for (int u = 0; u < UPW; ++u) {
        o[u][t] = mfma_bf(va, ph[u], o[u][t]);
        o[u][t] = mfma_bf(va, pl[u], o[u][t]);
      }
    }
  }
  if (!streams) return;
#pragma unroll
  for (int u = 0; u < UPW; ++u) {
    float ls = l[u];
    ls += __shfl_xor(ls, 16, 64);
    ls += __shfl_xor(ls, 32, 64);
    if (row_t[u] < 0) continue;
    f32x4 y[2 * DH];
#pragma unroll
    for (int k = 0; k < 2 * DH; ++k) y[k] = o[u][k];
    talk_store<DH, false>(a, part, T, p, tok0 + row_t[u], row_h[u], g4, m[u], ls, y);
  }
}

static bool talk_xchg_geometry(int H, int G, int D, int upw, TalkXchg& x, size_t& lds) {
  const int dh = D <= 32 ? 1 : D <= 64 ? 2 : 4;
  if (D % 8 || D > 128 || H > 32 || G < 1 || G > TX_NW || TX_NW % G || H % G) return false;
  const int rep = H / G;
  x.nwc = TX_NW / G;
  x.tb = 16 * x.nwc * upw / rep;
  if (x.tb < 1) return false;
  if (upw == 1) x.tb = 1;  // decode: one token a workgroup
  x.hp = (H + 7) / 8 * 8;
  x.s_tok = TM_KEYS * (x.hp + 4) + 4;
  x.m_off = x.tb * x.s_tok;
  x.m_tok = H * (TM_KEYS + 4) + 16;
  x.k_off = x.m_off + x.tb * x.m_tok;
  lds = (size_t)x.k_off * 4 + (size_t)TX_NW * TM_KEYS * (32 * dh + 8) * 2;
  return lds <= 160 * 1024;
}

__global__ __launch_bounds__(256) void talk_merge_kernel(TalkArgs a, const float* __restrict__ part, int T, int NP) {
  const int t = blockIdx.x, HD = a.H * a.D;
  if (a.q_ctx[t] <= 0) return;
  const float* ml = part + (int64_t)NP * T * HD;
  const bf16_t* gate = (const bf16_t*)a.z + (int64_t)t * a.zs + HD + a.G * a.D;
  for (int e = (blockIdx.y * 256 + threadIdx.x) * 4; e < HD; e += gridDim.y * 1024) {
    const int h = e / a.D;
    float mx = -INFINITY;
#pragma unroll 8
    for (int p = 0; p < NP; ++p) mx = fmaxf(mx, ml[(((int64_t)p * T + t) * a.H + h) * 2]);
    f32x4 acc = (f32x4)(0.f);
    float l = 0.f;
#pragma unroll 4
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
  const int rep = H / G;
  for (int rb = 0; rb < 16; ++rb)  // a row block's tokens must fit the 32-row query tile
    if (((rb * 16 + 15) / rep - rb * 16 / rep + 1) * rep > TM_KEYS) return false;
  // (the widest keys: one wave per SIMD with two units' queries in its 512 registers)
  nw = kf >= 16 ? 8 : 4;
  upw = kf >= 16 ? 1 : 2;
  return true;
}

template <int DH>
static int launch_talk_mfma(const TalkArgs& a, const int32_t* blk, int nblk, int grid_x, int tokens, int PS, int NP,
                            float* part, int T, int kf, hipStream_t stream) {
  const int nw = kf >= 16 ? 8 : 4, upw = kf >= 16 ? 1 : 2;
  const int units = a.G * ((tokens * (a.H / a.G) + 15) / 16);
  const dim3 grid(grid_x, (units + nw * upw - 1) / (nw * upw), NP);
#define MP_TM(KF_, UPW_, NW_)                                                                                     \
  hipLaunchKernelGGL((talk_mfma_kernel<DH, KF_, UPW_, NW_>), grid, dim3(NW_ * 64), 0, stream, a, blk, nblk, PS, part, T)
  if (kf == 4) MP_TM(4, 2, 4);
  else if (kf == 8) MP_TM(8, 2, 4);
  else if (kf == 16) MP_TM(16, 1, 8);
  else MP_TM(32, 1, 8);
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
  const bool vec = D % 8 == 0 && zs % 8 == 0;
  if (f32) {
    if (vec) hipLaunchKernelGGL((talk_prep_kernel<float, 8, 256>), dim3(n), dim3(256), 0, stream, a);
    else hipLaunchKernelGGL((talk_prep_kernel<float, 1, 256>), dim3(n), dim3(256), 0, stream, a);
  } else if (!vec) {
    hipLaunchKernelGGL((talk_prep_kernel<bf16_t, 1, 256>), dim3(n), dim3(256), 0, stream, a);
  } else if (n <= 256 && (H + G) * D > 2048) {
    hipLaunchKernelGGL((talk_prep_kernel<bf16_t, 8, 1024>), dim3(n), dim3(1024), 0, stream, a);
  } else {
    hipLaunchKernelGGL((talk_prep_kernel<bf16_t, 8, 256>), dim3(n), dim3(256), 0, stream, a);
  }
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

namespace mp {
constexpr int TX_UPW = 2;  // prompts: two 16-row blocks per wave (one in decode)
static bool use_xchg(int H, int G, int D, int form, int upw, TalkXchg& x, size_t& lds) {
  // the fold costs G x the QK work: it is kept where G is small and for the shapes the exchange does not take
  const int work = H * G * (D <= 32 ? 1 : D <= 64 ? 2 : 4);
  return form != 1 && (form == 2 || work >= (upw == 1 ? 256 : 512)) && talk_xchg_geometry(H, G, D, upw, x, lds);
}
}  // namespace mp

// Tokens of a prompt's query block (0: the MFMA forms do not cover the shape).  form 0: by shape, 1: the folded
// form, 2: the exchange form where it applies
extern "C" int mp_talk_block(int H, int G, int D, int form) {
  using namespace mp;
  TalkXchg x;
  size_t lds;
  if (use_xchg(H, G, D, form, TX_UPW, x, lds)) return x.tb;
  int dh, kf, upw, nw;
  if (!talk_geometry(H, G, D, dh, kf, upw, nw)) return 0;
  const int rep = H / G;
  int nrb = nw * upw / G > 1 ? nw * upw / G : 1;
  nrb = nrb > 16 ? 16 : nrb;
  const int tb = 16 * nrb / rep;
  return tb < 1 ? 1 : tb > 64 ? 64 : tb;
}

// blk [2, nblk] (first token, tokens; tokens <= mp_talk_block): a prompt step; blk == null: n one-token rows, the
// context in NP splits of PS keys (part: NP n (H D + 2 H) floats when NP > 1)
extern "C" int mp_talk_mfma(const void* z, int64_t zs, const void* qn, const float* talk, const float* sigma,
                            const void* cache,
                            const float* rk, const int32_t* bt, int bt_stride, const int32_t* q_seq,
                            const int32_t* q_ctx, void* out, int n, int H, int G, int D, int page_log2, int chunk,
                            float scale, const int32_t* blk, int nblk, int PS, int NP, float* part, int packed_mt,
                            int form, hipStream_t stream) {
  using namespace mp;
  (void)hipGetLastError();
  if (n == 0) return 0;
  int dh, kf, upw, nw;
  TalkXchg x;
  size_t lds;
  // (decode rows: one row block per wave, so all of a kv head's query heads must fit it)
  const bool xchg = use_xchg(H, G, D, form, blk ? TX_UPW : 1, x, lds) && mp_talk_block(H, G, D, form) > 0;
  if (page_log2 < 5 || (!xchg && !talk_geometry(H, G, D, dh, kf, upw, nw))) return -1;
  if (NP > 1 && (PS <= 0 || PS % TM_KEYS || part == nullptr || blk != nullptr)) return -2;
  if (NP < 1 || NP > 65535) return -2;
  TalkArgs a{};
  a.z = z, a.zs = zs, a.qn = (void*)qn, a.talk = talk, a.sigma = sigma, a.cache = (void*)cache, a.rk = (float*)rk, a.bt = bt;
  a.bt_stride = bt_stride, a.q_seq = q_seq, a.q_ctx = q_ctx, a.out = out;
  a.H = H, a.G = G, a.D = D, a.page_log2 = page_log2, a.chunk = chunk, a.packed_mt = packed_mt, a.scale = scale;
  const int gx = blk ? nblk : n, tokens = blk ? mp_talk_block(H, G, D, form) : 1;
  float* pp = NP > 1 ? part : nullptr;
  const int ps = NP > 1 ? PS : 0;
  int rc;
  if (xchg) {
    const dim3 grid(gx, 1, NP);
#define MP_TX(DH_, UPW_)                                                                                              \
  {                                                                                                                   \
    (void)hipFuncSetAttribute((const void*)talk_xchg_kernel<DH_, UPW_>, hipFuncAttributeMaxDynamicSharedMemorySize,  \
                              (int)lds);                                                                             \
    hipLaunchKernelGGL((talk_xchg_kernel<DH_, UPW_>), grid, dim3(TX_NW * 64), lds, stream, a, x, blk, nblk, ps, pp, n); \
  }
    if (D <= 32) {
      if (blk) MP_TX(1, TX_UPW) else MP_TX(1, 1)
    } else if (D <= 64) {
      if (blk) MP_TX(2, TX_UPW) else MP_TX(2, 1)
    } else {
      if (blk) MP_TX(4, TX_UPW) else MP_TX(4, 1)
    }
#undef MP_TX
    rc = (int)hipGetLastError();
  } else if (dh == 1) rc = launch_talk_mfma<1>(a, blk, nblk, gx, tokens, ps, NP, pp, n, kf, stream);
  else if (dh == 2) rc = launch_talk_mfma<2>(a, blk, nblk, gx, tokens, ps, NP, pp, n, kf, stream);
  else rc = launch_talk_mfma<4>(a, blk, nblk, gx, tokens, ps, NP, pp, n, kf, stream);
  if (rc || NP == 1) return rc;
  const int gy = (H * D / 4 + 255) / 256;
  hipLaunchKernelGGL(talk_merge_kernel, dim3(n, gy), dim3(256), 0, stream, a, part, n, NP);
  return (int)hipGetLastError();
}
