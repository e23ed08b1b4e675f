// Latent attention over a paged cache of latents, gfx950.
//
// A token's cache row is its latent c (C values, RMS-normed) and one rotated key part r (R values) that all heads
// share.  Head h's key is [U_h c | r], its value W_h c, its query [a | b] (a: D unrotated, b: R rotated values):
//   s(i, j) = (a_i . U_h c_j + b_i . r_j) scale          p = exp(s) / (exp(sink_h) + sum_j exp(s))
// over all j <= i.  Both products move to the query side, a . U c = (U^T a) . c and sum_j p_j W c_j = W sum_j p_j c_j,
// so every head reads the same cached row, as key (all of it) and as value (its first C columns):
//   u_i = [U_h^T a_i | b_i]  (C + R)      s = (u_i . row_j) scale      o_i = W_h sum_j p_j c_j
// Scores and weights are fp32.
//
//   latent_prep_kernel    norms of a projected row [q latent | c | r], r turned, cache write
//   latent_any_kernel     any shape and both element types: one workgroup per (query token, head)
//   latent_query_kernel   u, by MFMA: 16 rows of a head at a time
//   latent_attn_kernel    the core on MFMA: rows = (token, head) against 64-key tiles of the cache, split contexts
//   latent_value_kernel   merges the splits, applies the sink, W_h by MFMA
//   latent_gather_kernel, latent_wide_kernel   long portions of prompts: the context's latents in one piece (a library
//                         GEMM makes every head's keys and values of them), then attention over those, whose scores
//                         have D + R terms where the shared row's have C + R
#include "common.h"
#include "act_io.h"

namespace mp {

struct LatentArgs {
  const void* z;          // prep: [T, zs] projected rows
  int64_t zs;
  const float *qw, *cw;   // norm weights of the q latent [Q] and of c [C]
  void* cq;               // [T, Q] row-major or packed
  int Q, packed_q;
  const void* q;          // [T, qs] queries, head by head [D | R]
  int64_t qs;
  const void *uk, *uv;    // [H, C, D], [H, V, C]
  const float* sink;      // [H]
  const float* rope;      // [positions, R], cosines then sines
  void* cache;            // [pages, page, C + R]
  const int64_t* slots;
  const int32_t* bt;
  int bt_stride;
  const int32_t *q_seq, *q_ctx;
  const int32_t* rows;    // token rows to work on (null: all)
  void* u;                // [T, H, C + R]
  void* oc;               // [T, H, C]
  void* out;              // [T, H V] row-major or packed
  int T, H, D, R, V, C, page_log2, packed_mt;
  float scale, eps;
};

constexpr float LOG2E_F = 1.44269504088896340736f;

// VEC columns a thread and step; NT threads (decode rows are few: more threads, one round of loads)
template <typename T, int VEC, int NT>
__global__ __launch_bounds__(NT) void latent_prep_kernel(LatentArgs a) {
  __shared__ float red[16];
  const int t = blockIdx.x, tid = threadIdx.x, Q = a.Q, QC = a.Q + a.C;
  const int64_t slot = a.slots[t];
  if (slot < 0) return;
  const T* z = (const T*)a.z + (int64_t)t * a.zs;
  float sq = 0.f, sc = 0.f;
  for (int i = tid * VEC; i < QC; i += NT * VEC) {
    float x[VEC], s = 0.f;
    ld_vec<VEC>(z + i, x);
#pragma unroll
    for (int j = 0; j < VEC; ++j) s += x[j] * x[j];
    if (i < Q) sq += s;
    else sc += s;
  }
  sq = 1.f / sqrtf(block_sum(sq, red) / (float)Q + a.eps);
  sc = 1.f / sqrtf(block_sum(sc, red) / (float)a.C + a.eps);
  T* row = (T*)a.cache + slot * (a.C + a.R);
  for (int i = tid * VEC; i < QC; i += NT * VEC) {
    float x[VEC], g[VEC];
    ld_vec<VEC>(z + i, x);
    ld_vec<VEC>(i < Q ? a.qw + i : a.cw + i - Q, g);
    const float s = i < Q ? sq : sc;
#pragma unroll
    for (int j = 0; j < VEC; ++j) x[j] *= s * g[j];
    if (i < Q) st_act_vec<VEC>((T*)a.cq, t, i, Q, a.packed_q, x);
    else st_vec<VEC>(row + i - Q, x);
  }
  const float* cs = a.rope + (int64_t)(a.q_ctx[t] - 1) * a.R;
  const int half = a.R >> 1;
  const T* zr = z + QC;
  for (int i = tid; i < half; i += NT) {
    const float x = to_f(zr[i]), y = to_f(zr[i + half]), c = cs[i], s = cs[half + i];
    from_f(x * c - y * s, row[a.C + i]);
    from_f(y * c + x * s, row[a.C + half + i]);
  }
}

// dynamic LDS: u [C + R], acc [C], p [256], row ids [256] (as int), red [16]
template <typename T>
__global__ __launch_bounds__(256) void latent_any_kernel(LatentArgs a) {
  extern __shared__ float sm[];
  const int t = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int ctx = a.q_ctx[t];
  if (ctx <= 0) return;
  const int D = a.D, R = a.R, C = a.C, V = a.V, KW = C + R, half = R >> 1;
  float *u = sm, *acc = u + KW, *p = acc + C, *red = p + 512;
  int* rid = (int*)(p + 256);
  const T* q = (const T*)a.q + (int64_t)t * a.qs + (int64_t)h * (D + R);
  const T* uk = (const T*)a.uk + (int64_t)h * C * D;
  for (int c = tid; c < C; c += 256) {
    float s = 0.f;
    for (int d = 0; d < D; ++d) s += to_f(q[d]) * to_f(uk[(int64_t)c * D + d]);
    u[c] = s;
  }
  const float* cs = a.rope + (int64_t)(ctx - 1) * R;
  for (int i = tid; i < half; i += 256) {
    const float x = to_f(q[D + i]), y = to_f(q[D + half + i]), c = cs[i], s = cs[half + i];
    u[C + i] = x * c - y * s;
    u[C + half + i] = y * c + x * s;
  }
  __syncthreads();
  for (int c = tid; c < C; c += 256) acc[c] = 0.f;
  const int32_t* bt = a.bt + (int64_t)a.q_seq[t] * a.bt_stride;
  const int pmask = (1 << a.page_log2) - 1;
  float m = fmaxf(a.sink[h], -1e30f), l = 1.f;  // the sink's own term
  for (int j0 = 0; j0 < ctx; j0 += 256) {
    const int n = min(256, ctx - j0), j = j0 + tid;
    float s = -INFINITY;
    if (tid < n) {
      const int64_t r = ((int64_t)bt[j >> a.page_log2] << a.page_log2) + (j & pmask);
      rid[tid] = (int)r;
      const T* kp = (const T*)a.cache + r * KW;
      s = 0.f;
      for (int d = 0; d < KW; ++d) s += u[d] * to_f(kp[d]);
      s *= a.scale;
    }
    const float mx = fmaxf(m, block_max(s, red)), f = expf(m - mx), e = tid < n ? expf(s - mx) : 0.f;
    p[tid] = e;
    l = l * f + block_sum(e, red);
    m = mx;
    __syncthreads();
    for (int c = tid; c < C; c += 256) {
      float x = acc[c] * f;
      for (int k = 0; k < n; ++k) x += p[k] * to_f(((const T*)a.cache)[(int64_t)rid[k] * KW + c]);
      acc[c] = x;
    }
    __syncthreads();
  }
  const float inv = 1.f / l;
  const T* uv = (const T*)a.uv + (int64_t)h * V * C;
  const int lane = tid & 63;
  for (int v = tid >> 6; v < V; v += 4) {
    float x = 0.f;
    for (int c = lane; c < C; c += 64) x += acc[c] * inv * to_f(uv[(int64_t)v * C + c]);
    x = wave_sum(x);
    if (lane == 0) st_act((T*)a.out, t, h * V + v, a.H * V, a.packed_mt, x);
  }
}

// ---------------------------------------------------------------------------------------
// MFMA forms (bf16): C a multiple of 32 up to 512, D and R of 8, V of 4, pages of 64 tokens or more.
typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8_l;
typedef short s16x4_l __attribute__((ext_vector_type(4)));
__device__ __forceinline__ f32x4 mfma_l(const u16x8& a, const u16x8& b, const f32x4& c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_l, a), __builtin_bit_cast(bf16x8_l, b), c, 0,
                                                 0, 0);
}
__device__ __forceinline__ u16x4 lds_tr(const bf16_t* p) {
  const s16x4_l v = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4_l*)(p));
  return __builtin_bit_cast(u16x4, v);
}
__device__ __forceinline__ u16x4 pack4(float a, float b, float c, float d) { return (u16x4){f2bf(a), f2bf(b), f2bf(c), f2bf(d)}; }

// u rows of head blockIdx.y for 16 token rows; the four waves take 16-column tiles of C, blockIdx.z splits them.
// NF: 32-wide slices of D (past D the query fragment is 0 and the weight's last columns repeat: no branch)
template <int NF>
__global__ __launch_bounds__(256) void latent_query_kernel(LatentArgs a, int n) {
  const int tid = threadIdx.x, lane = tid & 63, c16 = lane & 15, g4 = lane >> 4;
  const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int h = blockIdx.y, D = a.D, R = a.R, C = a.C, KW = C + R;
  const int i = blockIdx.x * 16 + c16;
  const int t = i < n ? (a.rows ? a.rows[i] : i) : -1;
  const bf16_t* q = (const bf16_t*)a.q + (int64_t)max(t, 0) * a.qs + (int64_t)h * (D + R);
  u16x8 qf[NF];
#pragma unroll
  for (int f = 0; f < NF; ++f) {
    const int d = 32 * f + 8 * g4;
    const u16x8 x = *reinterpret_cast<const u16x8*>(q + min(d, D - 8));
    qf[f] = t >= 0 && d < D ? x : (u16x8)(0);
  }
  bf16_t* u = (bf16_t*)a.u + ((int64_t)max(t, 0) * a.H + h) * KW;
  for (int ct = blockIdx.z * 4 + w; ct * 16 < C; ct += 4 * gridDim.z) {
    const bf16_t* wk = (const bf16_t*)a.uk + ((int64_t)h * C + ct * 16 + c16) * D;
    u16x8 wf[NF];
#pragma unroll
    for (int f = 0; f < NF; ++f) wf[f] = *reinterpret_cast<const u16x8*>(wk + min(32 * f + 8 * g4, D - 8));
    f32x4 x = (f32x4)(0.f);
#pragma unroll
    for (int f = 0; f < NF; ++f) x = mfma_l(wf[f], qf[f], x);
    if (t >= 0) *reinterpret_cast<u16x4*>(u + ct * 16 + 4 * g4) = pack4(x[0], x[1], x[2], x[3]);
  }
  if (blockIdx.z == 0 && t >= 0 && a.q_ctx[t] > 0) {
    const float* cs = a.rope + (int64_t)(a.q_ctx[t] - 1) * R;
    const int half = R >> 1;
    for (int k = w * 4 + g4; k < half; k += 16) {
      const float x = bf2f(q[D + k]), y = bf2f(q[D + half + k]), c = cs[k], s = cs[half + k];
      u[C + k] = f2bf(x * c - y * s);
      u[C + half + k] = f2bf(y * c + x * s);
    }
  }
}

constexpr int LT_KEYS = 64, LT_PS = LT_KEYS + 8;
constexpr float LT_GROW = 8.f;  // log2 units a row's maximum may grow before its sums are rescaled

// A workgroup of NW waves owns up to 16 RT query rows (token-major x heads) of one sequence.  Per 64-key tile wave w
// makes the scores of keys 16 (w % 4) .. + 15 for RW of the row tiles (S^T = rows u^T: a lane owns one query row), the
// row maxima meet in LDS, the weights go to LDS as hi + lo bf16 (32-bit in effect), and wave w adds them into its
// 16 CW of the C value columns (O^T += c^T P^T, c^T by transposed reads of the same tile).  The next two tiles are in
// flight in registers.
template <int RT, int CW, int NW>
__global__ __launch_bounds__(NW * 64) void latent_attn_kernel(LatentArgs a, const int32_t* __restrict__ blk, int nblk,
                                                              int PS, float* __restrict__ part) {
  constexpr int NT = NW * 64, KPT = 2 * CW + 8 / NW;  // 16-B chunks of a tile per thread: C + R <= 16 CW NW + 64
  constexpr int RG = NW / 4, RW = RT / RG;
  static_assert(RT % RG == 0, "row tiles split evenly over the waves");
  extern __shared__ __attribute__((aligned(16))) bf16_t ls[];
  const int tid = threadIdx.x, lane = tid & 63, c16 = lane & 15, g4 = lane >> 4;
  const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int ws = w & 3, rg = w >> 2;
  const int H = a.H, C = a.C, KW = C + a.R, KF = (KW + 31) >> 5, STR = 32 * KF + 8;
  bf16_t *kt = ls, *qt = kt + LT_KEYS * STR, *ph = qt + 16 * RT * STR, *pl = ph + 16 * RT * LT_PS;
  float* wred = (float*)(pl + 16 * RT * LT_PS);  // [4][16 RT]

  const int bx = blk ? nblk - 1 - (int)blockIdx.x : (int)blockIdx.x;  // (later tokens see more keys: first)
  const int tok0 = blk ? blk[bx] : bx, ntok = blk ? blk[nblk + bx] : 1;
  const int hi = a.q_ctx[tok0 + ntok - 1];
  if (hi <= 0) return;
  const int h0 = blockIdx.y * 16 * RT, hg = min(H - h0, 16 * RT), nrow = ntok * hg;
  const int p = blockIdx.z, s_lo = p * PS, s_hi = PS > 0 ? min(hi, s_lo + PS) : hi;
  const int32_t* bt = a.bt + (int64_t)a.q_seq[tok0] * a.bt_stride;
  const int pmask = (1 << a.page_log2) - 1;
  const int cpr = KW >> 3;  // chunks per cache row
  const float rcp = 1.f / (float)cpr, sl2 = a.scale * LOG2E_F;

  float m[RT], l[RT];
  f32x4 o[RT][CW];
#pragma unroll
  for (int r = 0; r < RT; ++r) {
    m[r] = -INFINITY;
    l[r] = 0.f;
#pragma unroll
    for (int t = 0; t < CW; ++t) o[r][t] = (f32x4)(0.f);
  }

  int khi[RW];
#pragma unroll
  for (int r = 0; r < RW; ++r) {
    const int row = 16 * (rg * RW + r) + c16;
    khi[r] = row < nrow ? min(a.q_ctx[tok0 + row / hg], s_hi) : 0;
  }
  u16x8 ka_reg[KPT], kb_reg[KPT];  // the next two tiles, in flight
  auto fetch = [&](u16x8 (&kreg)[KPT], int s0) {  // a tile's rows are consecutive in the page; past the context the last row repeats
    const bf16_t* base = (const bf16_t*)a.cache + (((int64_t)bt[s0 >> a.page_log2] << a.page_log2) + (s0 & pmask)) * KW;
    const int lastc = min(LT_KEYS, s_hi - s0) * cpr - 1;
#pragma unroll
    for (int k = 0; k < KPT; ++k) kreg[k] = *reinterpret_cast<const u16x8*>(base + min(tid + NT * k, lastc) * 8);
  };
  auto stash = [&](const u16x8 (&kreg)[KPT]) {
#pragma unroll
    for (int k = 0; k < KPT; ++k) {
      const int x = tid + NT * k, key = (int)(((float)x + 0.5f) * rcp);
      if (key < LT_KEYS) *reinterpret_cast<u16x8*>(kt + key * STR + (x - key * cpr) * 8) = kreg[k];
    }
  };

  auto tile = [&](u16x8 (&kreg)[KPT], int s0) {
    stash(kreg);
    if (s0 + 2 * LT_KEYS < s_hi) fetch(kreg, s0 + 2 * LT_KEYS);
    __syncthreads();
    f32x4 st[RW];
#pragma unroll
    for (int r = 0; r < RW; ++r) st[r] = (f32x4)(0.f);
    const bf16_t *kp = kt + (16 * ws + c16) * STR + 8 * g4, *qp = qt + (16 * rg * RW + c16) * STR + 8 * g4;
#pragma unroll 6
    for (int f = 0; f < KF; ++f) {
      const u16x8 ka = *reinterpret_cast<const u16x8*>(kp + 32 * f);
#pragma unroll
      for (int r = 0; r < RW; ++r) st[r] = mfma_l(ka, *reinterpret_cast<const u16x8*>(qp + 16 * r * STR + 32 * f), st[r]);
    }
#pragma unroll
    for (int r = 0; r < RW; ++r) {
      const int row = 16 * (rg * RW + r) + c16;
      float lm = -INFINITY;
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        st[r][k] = s0 + 16 * ws + 4 * g4 + k < khi[r] ? st[r][k] * sl2 : -INFINITY;
        lm = fmaxf(lm, st[r][k]);
      }
      lm = fmaxf(lm, __shfl_xor(lm, 16, 64));
      lm = fmaxf(lm, __shfl_xor(lm, 32, 64));
      if (g4 == 0) wred[ws * 16 * RT + row] = lm;
    }
    __syncthreads();
#pragma unroll
    for (int r = 0; r < RT; ++r) {
      float lm = wred[16 * r + c16];
#pragma unroll
      for (int k = 1; k < 4; ++k) lm = fmaxf(lm, wred[k * 16 * RT + 16 * r + c16]);
      if (__any(lm > m[r] + LT_GROW)) {  // (every wave sees the same maxima: the same decision)
        const float mn = fmaxf(m[r], lm), al = mn == -INFINITY ? 1.f : __builtin_amdgcn_exp2f(m[r] - mn);
        l[r] *= al;
#pragma unroll
        for (int t = 0; t < CW; ++t) o[r][t] *= al;
        m[r] = mn;
      }
      if (r / RW != rg) continue;  // (uniform over the wave: this wave's scores)
      const float mu = m[r] == -INFINITY ? 0.f : m[r];
      float x[4];
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        x[k] = __builtin_amdgcn_exp2f(st[r % RW][k] - mu);
        l[r] += x[k];
      }
      const u16x4 xh = pack4(x[0], x[1], x[2], x[3]);
      const int off = (16 * r + c16) * LT_PS + 16 * ws + 4 * g4;
      *reinterpret_cast<u16x4*>(ph + off) = xh;
      *reinterpret_cast<u16x4*>(pl + off) =
          pack4(x[0] - bf2f(xh[0]), x[1] - bf2f(xh[1]), x[2] - bf2f(xh[2]), x[3] - bf2f(xh[3]));
    }
    __syncthreads();
#pragma unroll
    for (int kb = 0; kb < 2; ++kb) {
      u16x8 bh[RT], bl[RT];
#pragma unroll
      for (int r = 0; r < RT; ++r) {
        const int off = (16 * r + c16) * LT_PS + 32 * kb + 8 * g4;
        bh[r] = *reinterpret_cast<const u16x8*>(ph + off);
        bl[r] = *reinterpret_cast<const u16x8*>(pl + off);
      }
      // c^T: lane c16 of group g4 needs column 16 tile + c16 of keys 32 kb + 8 g4 .. + 7
      const bf16_t* vb = kt + (32 * kb + 8 * g4 + (c16 >> 2)) * STR + 4 * (c16 & 3);
#pragma unroll
      for (int t = 0; t < CW; ++t) {
        const int ct = min(w * CW + t, (C >> 4) - 1);  // (a tile past C repeats the last one and is not stored)
        const u16x4 v0 = lds_tr(vb + 16 * ct), v1 = lds_tr(vb + 4 * STR + 16 * ct);
        const u16x8 va = {v0[0], v0[1], v0[2], v0[3], v1[0], v1[1], v1[2], v1[3]};
#pragma unroll
        for (int r = 0; r < RT; ++r) {
          o[r][t] = mfma_l(va, bh[r], o[r][t]);
          o[r][t] = mfma_l(va, bl[r], o[r][t]);
        }
      }
    }
    __syncthreads();
  };
  if (s_lo < s_hi) fetch(ka_reg, s_lo);
  if (s_lo + LT_KEYS < s_hi) fetch(kb_reg, s_lo + LT_KEYS);
  // query rows, zero past the row count and past KW; the tile's own columns past KW
  for (int x = tid; x < 16 * RT * 4 * KF; x += NT) {
    const int r = x / (4 * KF), col = (x - r * 4 * KF) * 8;
    const int rr = min(r, nrow - 1);
    const bf16_t* src = (const bf16_t*)a.u + ((int64_t)(tok0 + rr / hg) * H + h0 + rr % hg) * KW;
    const u16x8 v = *reinterpret_cast<const u16x8*>(src + min(col, KW - 8));
    *reinterpret_cast<u16x8*>(qt + r * STR + col) = r < nrow && col < KW ? v : (u16x8)(0);
  }
  if (KW & 31)
    for (int x = tid; x < LT_KEYS * (4 * KF - cpr); x += NT) {
      const int r = x / (4 * KF - cpr), col = KW + (x - r * (4 * KF - cpr)) * 8;
      *reinterpret_cast<u16x8*>(kt + r * STR + col) = (u16x8)(0);
    }
  for (int s0 = s_lo; s0 < s_hi; s0 += 2 * LT_KEYS) {
    tile(ka_reg, s0);
    if (s0 + LT_KEYS < s_hi) tile(kb_reg, s0 + LT_KEYS);
  }
#pragma unroll
  for (int r = 0; r < RT; ++r) {
    float x = l[r];
    x += __shfl_xor(x, 16, 64);
    x += __shfl_xor(x, 32, 64);
    if (g4 == 0 && r / RW == rg) wred[ws * 16 * RT + 16 * r + c16] = x;
  }
  __syncthreads();
#pragma unroll
  for (int r = 0; r < RT; ++r) {
    const int row = 16 * r + c16;
    if (row >= nrow) continue;
    float ll = 0.f;
#pragma unroll
    for (int k = 0; k < 4; ++k) ll += wred[k * 16 * RT + row];
    const int h = h0 + row % hg;
    const int64_t th = (int64_t)(tok0 + row / hg) * H + h;
    if (part != nullptr) {  // split context: [NP][T H][C] sums, then [NP][T H][2] (maximum, sum)
      const int64_t TH = (int64_t)a.T * H;
      float* po = part + ((int64_t)p * TH + th) * C;
#pragma unroll
      for (int t = 0; t < CW; ++t)
        if ((w * CW + t) * 16 < C) *reinterpret_cast<f32x4*>(po + (w * CW + t) * 16 + 4 * g4) = o[r][t];
      if (w == 0 && g4 == 0) {
        float* ml = part + (int64_t)gridDim.z * TH * C + ((int64_t)p * TH + th) * 2;
        ml[0] = m[r];
        ml[1] = ll;
      }
      continue;
    }
    const float sk = fmaxf(a.sink[h] * LOG2E_F, -1e30f), mf = fmaxf(m[r], sk);
    const float f = __builtin_amdgcn_exp2f(m[r] - mf), inv = f / (ll * f + __builtin_amdgcn_exp2f(sk - mf));
    bf16_t* po = (bf16_t*)a.oc + th * C;
#pragma unroll
    for (int t = 0; t < CW; ++t)
      if ((w * CW + t) * 16 < C)
        *reinterpret_cast<u16x4*>(po + (w * CW + t) * 16 + 4 * g4) =
            pack4(o[r][t][0] * inv, o[r][t][1] * inv, o[r][t][2] * inv, o[r][t][3] * inv);
  }
}

// values of head blockIdx.y for 16 token rows: the latent sums go to LDS (merged over NP splits when part is given),
// then each wave makes 16-column tiles of V.  CF: 32-column slices of C the kernel is built for; the first tile's
// weights are in flight during the merge
constexpr int LV_NP = 64;  // splits whose factors fit in LDS (the host gives no more)
template <int CF>
__global__ __launch_bounds__(256) void latent_value_kernel(LatentArgs a, int n, const float* __restrict__ part, int NP) {
  constexpr int STR = 32 * CF + 8;
  __shared__ __attribute__((aligned(16))) bf16_t ls[16 * STR];
  __shared__ float fac[16][LV_NP + 1];
  const int tid = threadIdx.x, lane = tid & 63, c16 = lane & 15, g4 = lane >> 4;
  const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int h = blockIdx.y, H = a.H, C = a.C, V = a.V;
  u16x8 wf[CF];
  auto weights = [&](int vt) {  // (slices past C repeat the last one and meet zeros)
    const bf16_t* wv = (const bf16_t*)a.uv + ((int64_t)h * V + min(vt * 16 + c16, V - 1)) * C + 8 * g4;
#pragma unroll
    for (int f = 0; f < CF; ++f) wf[f] = *reinterpret_cast<const u16x8*>(wv + min(32 * f, C - 32));
  };
  weights(blockIdx.z * 4 + w);
  {
    const int r = tid >> 4, k0 = tid & 15, i = blockIdx.x * 16 + r;  // 16 threads a row
    const int t = i < n ? (a.rows ? a.rows[i] : i) : -1;
    const bool live = t >= 0 && a.q_ctx[max(t, 0)] > 0;
    const int64_t TH = (int64_t)a.T * H, th = (int64_t)max(t, 0) * H + h;
    if (part == nullptr) {
#pragma unroll
      for (int k = 0; k < CF; k += 4) {
        const int c = 32 * k + k0 * 8;
        const u16x8 x = *reinterpret_cast<const u16x8*>((const bf16_t*)a.oc + th * C + min(c, C - 8));
        if (c < 32 * CF) *reinterpret_cast<u16x8*>(ls + r * STR + c) = live && c < C ? x : (u16x8)(0);
      }
    } else {
      const float* ml = part + (int64_t)NP * TH * C + th * 2;
      const float sk = fmaxf(a.sink[h] * LOG2E_F, -1e30f);
      float pm[LV_NP / 16], plv[LV_NP / 16], m = sk;
#pragma unroll
      for (int k = 0; k < LV_NP / 16; ++k) {  // thread k0 has the splits k0, k0 + 16, ..
        const int p = k0 + 16 * k;
        const bool ok = live && p < NP;
        pm[k] = ok ? ml[min(p, NP - 1) * TH * 2] : -INFINITY;
        plv[k] = ok ? ml[min(p, NP - 1) * TH * 2 + 1] : 0.f;
        m = fmaxf(m, pm[k]);
      }
#pragma unroll
      for (int s = 1; s < 16; s <<= 1) m = fmaxf(m, __shfl_xor(m, s, 64));
      float l = k0 == 0 ? __builtin_amdgcn_exp2f(sk - m) : 0.f;
#pragma unroll
      for (int k = 0; k < LV_NP / 16; ++k) {
        pm[k] = __builtin_amdgcn_exp2f(pm[k] - m);
        l += plv[k] * pm[k];
      }
#pragma unroll
      for (int s = 1; s < 16; s <<= 1) l += __shfl_xor(l, s, 64);
      const float inv = 1.f / l;
#pragma unroll
      for (int k = 0; k < LV_NP / 16; ++k) fac[r][k0 + 16 * k] = pm[k] * inv;
      __syncthreads();
      float x[CF / 4][8];
#pragma unroll
      for (int k = 0; k < CF / 4; ++k)
#pragma unroll
        for (int e = 0; e < 8; ++e) x[k][e] = 0.f;
      for (int p = 0; p < NP; p += 2) {  // two splits' rows in flight
        float y[2][CF / 4][8];
#pragma unroll
        for (int q = 0; q < 2; ++q)
#pragma unroll
          for (int k = 0; k < CF / 4; ++k)
            ld_vec<8>(part + ((int64_t)min(p + q, NP - 1) * TH + th) * C + min(128 * k + k0 * 8, C - 8), y[q][k]);
        const float f0 = fac[r][p], f1 = p + 1 < NP ? fac[r][p + 1] : 0.f;
#pragma unroll
        for (int k = 0; k < CF / 4; ++k)
#pragma unroll
          for (int e = 0; e < 8; ++e) x[k][e] += f0 * y[0][k][e] + f1 * y[1][k][e];
      }
#pragma unroll
      for (int k = 0; k < CF / 4; ++k) {
        const int c = 128 * k + k0 * 8;
        if (!live || c >= C)
#pragma unroll
          for (int e = 0; e < 8; ++e) x[k][e] = 0.f;
        st_vec<8>(ls + r * STR + c, x[k]);
      }
    }
  }
  __syncthreads();
  const int i = blockIdx.x * 16 + c16;
  const int t = i < n ? (a.rows ? a.rows[i] : i) : -1;
  for (int vt = blockIdx.z * 4 + w; vt * 16 < V; vt += 4 * gridDim.z) {
    f32x4 x = (f32x4)(0.f);
#pragma unroll
    for (int f = 0; f < CF; ++f)
      x = mfma_l(wf[f], *reinterpret_cast<const u16x8*>(ls + c16 * STR + 32 * f + 8 * g4), x);
    const int v = vt * 16 + 4 * g4;
    if (t >= 0 && v < V) {
      const float y[4] = {x[0], x[1], x[2], x[3]};
      st_act_vec<4>((bf16_t*)a.out, t, h * V + v, H * V, a.packed_mt, y);
    }
    if ((vt + 4 * gridDim.z) * 16 < V) weights(vt + 4 * gridDim.z);
  }
}

// row tiles of a workgroup (0: the MFMA forms do not cover the shape), the value columns the kernels are built for, and
// the LDS; rows: query rows that there are
static int latent_geometry(int H, int D, int R, int V, int C, int page_log2, int rows, int& cw, size_t& lds) {
  if (page_log2 < 6 || D % 8 || R % 8 || V % 4 || C % 32 || C > 512 || D > 256) return 0;
  cw = C <= 128 ? 128 : C <= 256 ? 256 : 512;
  if (C + R > cw + 64) return 0;
  const int str = (C + R + 31) / 32 * 32 + 8;
  for (int rt = rows > 32 ? 4 : rows > 16 ? 2 : 1; rt; rt >>= 1) {
    lds = (size_t)(LT_KEYS + 16 * rt) * str * 2 + 2 * 16 * rt * LT_PS * 2 + 4 * 16 * rt * 4;
    if (lds <= 160 * 1024) return rt;
  }
  return 0;
}

// out[i] = cache row idx[i], 16-B chunks
__global__ __launch_bounds__(256) void latent_gather_kernel(const bf16_t* __restrict__ cache,
                                                            const int64_t* __restrict__ idx, bf16_t* __restrict__ out,
                                                            int64_t n, int KW) {
  const int cpr = KW >> 3;
  const int64_t total = n * cpr;
  for (int64_t i = blockIdx.x * (int64_t)256 + threadIdx.x; i < total; i += (int64_t)gridDim.x * 256) {
    const int64_t r = i / cpr;
    const int c = (int)(i - r * cpr) * 8;
    *reinterpret_cast<u16x8*>(out + r * KW + c) = *reinterpret_cast<const u16x8*>(cache + idx[r] * KW + c);
  }
}

// LDS image of a tile of 32 NS columns (16-B chunks ch): 8-row x 32-column subtiles of 512 B, the chunk XOR-swizzled by
// the row, so that row reads and transposed reads are both free of bank conflicts
template <int NS>
__device__ __forceinline__ int lw_off(int row, int ch) {
  return 512 * NS * (row >> 3) + 512 * (ch >> 2) + 64 * (row & 7) + 16 * ((ch & 3) ^ ((row >> 2) & 3));
}
__device__ __forceinline__ f32x16 mfma_lw(const u16x8& a, const u16x8& b, const f32x16& c) {
  return __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8_l, a), __builtin_bit_cast(bf16x8_l, b), c, 0,
                                                 0, 0);
}
__device__ __forceinline__ u16x4 lw_tr(const unsigned char* p) { return lds_tr(reinterpret_cast<const bf16_t*>(p)); }

struct WideArgs {
  const bf16_t* kv;       // [N, kvs] every context row's keys and values, head by head [D | V]
  int64_t kvs;
  const bf16_t* lat;      // [N, C + R] gathered cache rows (the rotated key part lies behind C)
  const int32_t* blk;     // [3, nblk] first token, tokens, first context row of the sequence
  int nblk;
};

// One workgroup: 32 NW query tokens of one head and sequence against 64-key tiles, double-buffered in LDS.
// S^T = K q^T and O^T += V^T P^T on 32x32x16 MFMA: a lane owns one query row, the softmax is lane-local plus one
// exchange, the weights go as hi + lo bf16 straight from the accumulators.  DF, RF, VF: 32-column slices of D, R, V.
// A long query block and its short mirror are taken by one workgroup, so all stream about the same context.
template <int DF, int RF, int VF, int NW>
__global__ __launch_bounds__(NW * 64) void latent_wide_kernel(LatentArgs a, WideArgs b) {
  constexpr int NSK = DF + RF, KT = 64 * 64 * NSK, VT = 64 * 64 * VF, NT = NW * 64;  // tile bytes
  constexpr int KCH = 64 * 4 * NSK / NT, VCH = 64 * 4 * VF / NT;
  static_assert(64 * 4 * NSK % NT == 0 && 64 * 4 * VF % NT == 0, "tile chunks split evenly over the threads");
  extern __shared__ __attribute__((aligned(16))) unsigned char lw[];
  const int tid = threadIdx.x, lane = tid & 63;
  const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int H = a.H, D = a.D, R = a.R, V = a.V, C = a.C, KW = C + R;
  const int NBP = (b.nblk + 1) / 2, G = gridDim.x;
  int lin = blockIdx.x;
  if ((G & 7) == 0) lin = (lin & 7) * (G >> 3) + (lin >> 3);  // a head's query blocks share an XCD's L2
  const int h = lin / NBP, jb = lin - h * NBP;
  const int r = lane & 31, hh = lane >> 5;
  const float sl2 = a.scale * LOG2E_F;
  const int npass = b.nblk - 1 - jb != jb ? 2 : 1;
  for (int pass = 0; pass < npass; ++pass) {
    const int bx = pass == 0 ? b.nblk - 1 - jb : jb;
    const int tok0 = b.blk[bx], ntok = b.blk[b.nblk + bx];
    const int64_t row0 = b.blk[2 * b.nblk + bx];
    const int end = a.q_ctx[tok0 + ntok - 1];
    const int wt = 32 * w;
    const bool wave_rows = wt < ntok;
    const int wave_ctx = wave_rows ? a.q_ctx[tok0 + min(wt + 31, ntok - 1)] : 0;
    const int wave_lim0 = wave_rows ? a.q_ctx[tok0 + wt] : 0;  // smallest limit of its rows
    const bool row_ok = wt + r < ntok;
    const int tok = tok0 + min(wt + r, ntok - 1);
    const int lim = row_ok ? a.q_ctx[tok] : 0;

    u16x8 qf[2 * NSK];
    {
      const bf16_t* q = (const bf16_t*)a.q + (int64_t)tok * a.qs + (int64_t)h * (D + R);
#pragma unroll
      for (int s = 0; s < 2 * DF; ++s) {
        const int d = 16 * s + 8 * hh;
        const u16x8 x = *reinterpret_cast<const u16x8*>(q + min(d, D - 8));
        qf[s] = row_ok && d < D ? x : (u16x8)(0);
      }
      const int half = R >> 1;
      const float* cs = a.rope + (int64_t)(max(a.q_ctx[tok], 1) - 1) * R;
#pragma unroll
      for (int s = 0; s < 2 * RF; ++s) {
        const int d = min(16 * s + 8 * hh, R - 8), e = d < half ? d + half : d - half, f = d < half ? d : e;
        const u16x8 x = *reinterpret_cast<const u16x8*>(q + D + d), y = *reinterpret_cast<const u16x8*>(q + D + e);
        float c[8], sn[8];
        ld_vec<8>(cs + f, c);
        ld_vec<8>(cs + half + f, sn);
        const float sg = d < half ? -1.f : 1.f;
        u16x8 z;
#pragma unroll
        for (int j = 0; j < 8; ++j) z[j] = f2bf(bf2f(x[j]) * c[j] + sg * bf2f(y[j]) * sn[j]);
        qf[2 * DF + s] = row_ok && 16 * s + 8 * hh < R ? z : (u16x8)(0);
      }
    }
    f32x16 o[VF];
#pragma unroll
    for (int t = 0; t < VF; ++t) o[t] = (f32x16)(0.f);
    float m = -INFINITY, l = 0.f;

    u16x8 kreg[KCH], vreg[VCH];
    auto fetch = [&](int s0) {
#pragma unroll
      for (int j = 0; j < KCH; ++j) {
        const int c = tid + NT * j, row = c / (4 * NSK), ch = c - row * (4 * NSK);
        const int64_t cr = row0 + min(s0 + row, end - 1);
        const bf16_t* p = ch < 4 * DF ? b.kv + cr * b.kvs + h * (D + V) + min(ch * 8, D - 8)
                                      : b.lat + cr * KW + C + min((ch - 4 * DF) * 8, R - 8);
        kreg[j] = *reinterpret_cast<const u16x8*>(p);
      }
#pragma unroll
      for (int j = 0; j < VCH; ++j) {
        const int c = tid + NT * j, row = c / (4 * VF), ch = c - row * (4 * VF);
        vreg[j] = *reinterpret_cast<const u16x8*>(b.kv + (row0 + min(s0 + row, end - 1)) * b.kvs + h * (D + V) + D +
                                                  min(ch * 8, V - 8));
      }
    };
    // (columns past D and R meet a 0 in q, columns past V are not stored, rows past the context repeat the last one
    // and meet a weight of 0)
    auto stash = [&](int buf) {
      unsigned char* kb = lw + buf * (KT + VT);
#pragma unroll
      for (int j = 0; j < KCH; ++j) {
        const int c = tid + NT * j, row = c / (4 * NSK), ch = c - row * (4 * NSK);
        *reinterpret_cast<u16x8*>(kb + lw_off<NSK>(row, ch)) = kreg[j];
      }
#pragma unroll
      for (int j = 0; j < VCH; ++j) {
        const int c = tid + NT * j, row = c / (4 * VF), ch = c - row * (4 * VF);
        *reinterpret_cast<u16x8*>(kb + KT + lw_off<VF>(row, ch)) = vreg[j];
      }
    };
    const int grp = lane >> 4, gi = lane & 15, tq = gi >> 2, tp = gi & 3;
    const int kb0 = lw_off<NSK>(r, hh), kb1 = lw_off<NSK>(r, 2 + hh);
    const int trc = 2 * (grp & 1) + (tp >> 1);
    const int vb0 = KT + lw_off<VF>(4 * hh + tq, trc) + 8 * (tp & 1), vb1 = KT + lw_off<VF>(8 + 4 * hh + tq, trc) + 8 * (tp & 1);

    fetch(0);
    stash(0);
    __syncthreads();
    int cur = 0;
    for (int s0 = 0; s0 < end; s0 += 64, cur ^= 1) {
      const bool more = s0 + 64 < end;
      if (more) fetch(s0 + 64);
      if (s0 < wave_ctx) {
        const unsigned char* tb = lw + cur * (KT + VT);
        f32x16 st[2];
        st[0] = st[1] = (f32x16)(0.f);
#pragma unroll
        for (int s = 0; s < 2 * NSK; ++s)
#pragma unroll
          for (int sub = 0; sub < 2; ++sub)
            st[sub] = mfma_lw(*reinterpret_cast<const u16x8*>(tb + ((s & 1) ? kb1 : kb0) + 2048 * NSK * sub + 512 * (s >> 1)),
                              qf[s], st[sub]);
        if (s0 + 64 > wave_lim0) {  // diagonal and last tiles
#pragma unroll
          for (int sub = 0; sub < 2; ++sub)
#pragma unroll
            for (int j = 0; j < 16; ++j)
              st[sub][j] = s0 + 32 * sub + 4 * hh + (j & 3) + 8 * (j >> 2) < lim ? st[sub][j] : -INFINITY;
        }
        float lm = -INFINITY;
#pragma unroll
        for (int sub = 0; sub < 2; ++sub)
#pragma unroll
          for (int j = 0; j < 16; ++j) lm = fmaxf(lm, st[sub][j]);
        lm = fmaxf(lm, __shfl_xor(lm, 32, 64)) * sl2;
        if (!__all(lm <= m + LT_GROW)) {
          const float mn = fmaxf(m, lm), al = mn == -INFINITY ? 1.f : __builtin_amdgcn_exp2f(m - mn);
          l *= al;
#pragma unroll
          for (int t = 0; t < VF; ++t) o[t] *= al;
          m = mn;
        }
        const float mu = m == -INFINITY ? 0.f : m;
#pragma unroll
        for (int sub = 0; sub < 2; ++sub)
#pragma unroll
          for (int s2 = 0; s2 < 2; ++s2) {
            u16x8 ph, pl;
#pragma unroll
            for (int j = 0; j < 8; ++j) {
              const float x = __builtin_amdgcn_exp2f(__builtin_fmaf(st[sub][8 * s2 + j], sl2, -mu));
              l += x;
              ph[j] = f2bf(x);
              pl[j] = f2bf(x - bf2f(ph[j]));
            }
#pragma unroll
            for (int t = 0; t < VF; ++t) {
              const int imm = 2048 * VF * sub + 1024 * VF * s2 + 512 * t;
              const u16x4 v0 = lw_tr(tb + vb0 + imm), v1 = lw_tr(tb + vb1 + imm);
              const u16x8 va = {v0[0], v0[1], v0[2], v0[3], v1[0], v1[1], v1[2], v1[3]};
              o[t] = mfma_lw(va, ph, o[t]);
              o[t] = mfma_lw(va, pl, o[t]);
            }
          }
      }
      if (more) stash(cur ^ 1);
      __syncthreads();
    }
    l += __shfl_xor(l, 32, 64);
    if (!row_ok) continue;  // (every tile ended in a barrier: the LDS is free)
    const float sk = fmaxf(a.sink[h] * LOG2E_F, -1e30f), mf = fmaxf(m, sk);
    const float f = __builtin_amdgcn_exp2f(m - mf), inv = f / (l * f + __builtin_amdgcn_exp2f(sk - mf));
#pragma unroll
    for (int t = 0; t < VF; ++t)
#pragma unroll
      for (int gq = 0; gq < 4; ++gq) {
        const int v = 32 * t + 8 * gq + 4 * hh;
        if (v >= V) continue;
        const float y[4] = {o[t][4 * gq] * inv, o[t][4 * gq + 1] * inv, o[t][4 * gq + 2] * inv, o[t][4 * gq + 3] * inv};
        st_act_vec<4>((bf16_t*)a.out, tok, h * V + v, H * V, a.packed_mt, y);
      }
  }
}

static int latent_wide_form(int D, int R, int V) {
  if (D % 8 || R % 16 || V % 8) return 0;
  return D <= 64 && R <= 32 && V <= 64 ? 1 : D <= 128 && R <= 64 && V <= 128 ? 2 : 0;
}

}  // namespace mp

extern "C" int mp_latent_prep(const void* z, int64_t zs, const float* qw, const float* cw, void* cq, void* cache,
                              const int64_t* slots, const int32_t* q_ctx, const float* rope, int n, int Q, int C, int R,
                              float eps, int packed_q, int f32, hipStream_t stream) {
  using namespace mp;
  (void)hipGetLastError();
  if (n == 0) return 0;
  LatentArgs a{};
  a.z = z, a.zs = zs, a.qw = qw, a.cw = cw, a.cq = cq, a.cache = cache, a.slots = slots, a.q_ctx = q_ctx, a.rope = rope;
  a.Q = Q, a.C = C, a.R = R, a.eps = eps, a.packed_q = packed_q;
  const bool vec = Q % 8 == 0 && C % 8 == 0 && R % 8 == 0 && zs % 8 == 0;
  if (f32 && vec) hipLaunchKernelGGL((latent_prep_kernel<float, 8, 256>), dim3(n), dim3(256), 0, stream, a);
  else if (f32) hipLaunchKernelGGL((latent_prep_kernel<float, 1, 256>), dim3(n), dim3(256), 0, stream, a);
  else if (vec) hipLaunchKernelGGL((latent_prep_kernel<bf16_t, 8, 256>), dim3(n), dim3(256), 0, stream, a);
  else hipLaunchKernelGGL((latent_prep_kernel<bf16_t, 1, 256>), dim3(n), dim3(256), 0, stream, a);
  return (int)hipGetLastError();
}

// Tokens of a query block of the MFMA form (0: it does not cover the shape)
extern "C" int mp_latent_block(int H, int D, int R, int V, int C, int page_log2) {
  int cw;
  size_t lds;
  const int rt = mp::latent_geometry(H, D, R, V, C, page_log2, 64, cw, lds);
  return rt == 0 ? 0 : 16 * rt / H > 1 ? 16 * rt / H : 1;
}

// form 0: any shape.  form 1: MFMA over the rows ``rows`` (n of them, null: all T rows) in the blocks ``blk`` [2, nblk]
// (null: every row its own block), the context in NP splits of PS keys (part: NP T H (C + 2) floats when NP > 1).
extern "C" int mp_latent_attention(int form, const void* q, int64_t qs, const void* uk, const void* uv, const float* sink,
                                   const float* rope, const void* cache, const int32_t* bt, int bt_stride,
                                   const int32_t* q_seq, const int32_t* q_ctx, void* u, void* oc, void* out, int T, int H,
                                   int D, int R, int V, int C, int page_log2, float scale, const int32_t* rows, int n,
                                   const int32_t* blk, int nblk, int PS, int NP, float* part, int packed_mt, int f32,
                                   hipStream_t stream) {
  using namespace mp;
  (void)hipGetLastError();
  if (T == 0 || n == 0) return 0;
  LatentArgs a{};
  a.q = q, a.qs = qs, a.uk = uk, a.uv = uv, a.sink = sink, a.rope = rope, a.cache = (void*)cache, a.bt = bt;
  a.bt_stride = bt_stride, a.q_seq = q_seq, a.q_ctx = q_ctx, a.u = u, a.oc = oc, a.out = out, a.rows = rows;
  a.T = T, a.H = H, a.D = D, a.R = R, a.V = V, a.C = C, a.page_log2 = page_log2, a.packed_mt = packed_mt;
  a.scale = scale;
  if (form == 0) {
    const size_t lds = (size_t)(C + R + C + 512 + 16) * sizeof(float);
    if (lds > 60000 || H > 65535) return -1;
    if (f32) hipLaunchKernelGGL(latent_any_kernel<float>, dim3(T, H), dim3(256), lds, stream, a);
    else hipLaunchKernelGGL(latent_any_kernel<bf16_t>, dim3(T, H), dim3(256), lds, stream, a);
    return (int)hipGetLastError();
  }
  int cw;
  size_t lds;
  const int tb = blk ? mp_latent_block(H, D, R, V, C, page_log2) : 1;
  const int rt = f32 ? 0 : latent_geometry(H, D, R, V, C, page_log2, tb * H, cw, lds);
  if (rt == 0 || qs % 8) return -1;
  if (NP < 1 || NP > LV_NP || (NP > 1 && (PS <= 0 || PS % LT_KEYS || part == nullptr))) return -2;
  const int nb16 = (n + 15) / 16;
  const int ctiles = (C / 16 + 3) / 4, vtiles = ((V + 15) / 16 + 3) / 4;
  const int zq = nb16 * H >= 1024 ? 1 : ctiles, zv = nb16 * H >= 1024 ? 1 : vtiles;
  if (D <= 64) hipLaunchKernelGGL(latent_query_kernel<2>, dim3(nb16, H, zq), dim3(256), 0, stream, a, n);
  else if (D <= 128) hipLaunchKernelGGL(latent_query_kernel<4>, dim3(nb16, H, zq), dim3(256), 0, stream, a, n);
  else hipLaunchKernelGGL(latent_query_kernel<8>, dim3(nb16, H, zq), dim3(256), 0, stream, a, n);
  int rc = (int)hipGetLastError();
  if (rc) return rc;
  const dim3 grid(blk ? nblk : T, (H + 16 * rt - 1) / (16 * rt), NP);
  float* pp = NP > 1 ? part : nullptr;
  const int ps = NP > 1 ? PS : 0;
#define MP_LA(RT_, CW_, NW_)                                                                                           \
  {                                                                                                                    \
    if (lds > 65536)                                                                                                   \
      (void)hipFuncSetAttribute((const void*)latent_attn_kernel<RT_, CW_, NW_>,                                        \
                                hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);                                 \
    hipLaunchKernelGGL((latent_attn_kernel<RT_, CW_, NW_>), grid, dim3(NW_ * 64), lds, stream, a, blk, nblk, ps, pp);   \
  }
#define MP_LAC(C_)                       \
  if (rt == 1) MP_LA(1, C_ / 64, 4)      \
  else if (rt == 2) MP_LA(2, C_ / 128, 8) \
  else MP_LA(4, C_ / 128, 8)
  if (cw == 128) { MP_LAC(128) } else if (cw == 256) { MP_LAC(256) } else { MP_LAC(512) }
#undef MP_LAC
#undef MP_LA
  rc = (int)hipGetLastError();
  if (rc) return rc;
  const dim3 gv(nb16, H, zv);
  if (cw == 128) hipLaunchKernelGGL(latent_value_kernel<4>, gv, dim3(256), 0, stream, a, n, pp, NP);
  else if (cw == 256) hipLaunchKernelGGL(latent_value_kernel<8>, gv, dim3(256), 0, stream, a, n, pp, NP);
  else hipLaunchKernelGGL(latent_value_kernel<16>, gv, dim3(256), 0, stream, a, n, pp, NP);
  return (int)hipGetLastError();
}

// Query tokens of a block of the wide form per wave (0: it does not cover the shape)
extern "C" int mp_latent_wide_ok(int D, int R, int V, int C) { return C % 8 == 0 && mp::latent_wide_form(D, R, V) != 0; }

extern "C" int mp_latent_gather(const void* cache, const int64_t* idx, void* out, int64_t n, int KW, hipStream_t stream) {
  using namespace mp;
  (void)hipGetLastError();
  if (n == 0) return 0;
  if (KW % 8) return -1;
  int64_t g = (n * (KW / 8) + 255) / 256;
  if (g > 16384) g = 16384;
  hipLaunchKernelGGL(latent_gather_kernel, dim3((unsigned)g), dim3(256), 0, stream, (const bf16_t*)cache, idx, (bf16_t*)out,
                     n, KW);
  return (int)hipGetLastError();
}

// blk [3, nblk]: first token, tokens (<= 32 nw) and first context row of every query block
extern "C" int mp_latent_wide(const void* q, int64_t qs, const void* kv, int64_t kvs, const void* lat, const float* sink,
                              const float* rope, const int32_t* q_ctx, void* out, int H, int D, int R, int V, int C,
                              float scale, const int32_t* blk, int nblk, int nw, int packed_mt, hipStream_t stream) {
  using namespace mp;
  (void)hipGetLastError();
  if (nblk == 0) return 0;
  const int form = latent_wide_form(D, R, V);
  if (form == 0 || C % 8 || qs % 8 || kvs % 8 || (nw != 4 && nw != 8)) return -1;
  LatentArgs a{};
  a.q = q, a.qs = qs, a.sink = sink, a.rope = rope, a.q_ctx = q_ctx, a.out = out;
  a.H = H, a.D = D, a.R = R, a.V = V, a.C = C, a.packed_mt = packed_mt, a.scale = scale;
  const WideArgs b{(const bf16_t*)kv, kvs, (const bf16_t*)lat, blk, nblk};
  const dim3 grid(H * ((nblk + 1) / 2));
#define MP_LW(DF_, RF_, VF_, NW_)                                                                                      \
  {                                                                                                                    \
    constexpr int lds = 2 * 64 * 64 * (DF_ + RF_ + VF_);                                                               \
    if (lds > 65536)                                                                                                   \
      (void)hipFuncSetAttribute((const void*)latent_wide_kernel<DF_, RF_, VF_, NW_>,                                   \
                                hipFuncAttributeMaxDynamicSharedMemorySize, lds);                                      \
    hipLaunchKernelGGL((latent_wide_kernel<DF_, RF_, VF_, NW_>), grid, dim3(NW_ * 64), lds, stream, a, b);              \
  }
  if (form == 1) {
    if (nw == 4) MP_LW(2, 1, 2, 4) else { return -1; }
  } else {
    if (nw == 4) MP_LW(4, 2, 4, 4) else MP_LW(4, 2, 4, 8)
  }
#undef MP_LW
  return (int)hipGetLastError();
}
