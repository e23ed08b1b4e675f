// MFMA forms of head-mixing attention (attention_mixed.hip has the equations and the cache layout): bf16, head sizes up to
// 128, at most 32 query heads, soft caps up to 64.  A capped score lies in [-cap, cap], so exp(s) fits fp32 as it is:
// no running maximum, and the weights of any split of the keys add up.
//
// Prompts: the mixing comes after the softmax, so it needs every head's denominator first.
//   mixed_sum_kernel   sum_j exp(s_g(i, j)) of every token and head
//   mixed_core_kernel  the scores again, p = exp(s) / (1 + sum); p goes to LDS as hi + lo bf16 (16 bits of mantissa), one
//                      MFMA with T mixes the heads of a (key, token), the mixed weights return through LDS to the waves
//                      that own the heads, where they are the B operand of O^T += V^T A^T
// A workgroup owns 16 or 8 tokens and all heads; a wave owns UPW units of 16 columns, a unit being HPU heads of 16 / HPU
// tokens.  K and V^T are read from the cache as A operands, a tile ahead.  Two barriers per 32 keys.
//
// Decode: a token's value product has all heads' weights as columns, so mixing after it costs no MFMA work:
//   mixed_decode_kernel  per (token, split of the keys): O_{g, c} = sum_j exp(s_g) v_c(j) for all heads g and kv heads c
//   mixed_merge_kernel   adds the splits, o_h = sum_g T[h, g] / (1 + sum_g) O_{g, c(h)}, turns back, applies the gate
#include <type_traits>

#include "attn_mixed.h"

namespace mp {

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8_t;
__device__ __forceinline__ f32x4 mfma_bf(const u16x8& a, const u16x8& b, const f32x4& c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, a), __builtin_bit_cast(bf16x8_t, b), c, 0,
                                                 0, 0);
}

constexpr int MX_KEYS = 32, MX_NW = 8, MX_HEADS = 32, MX_PITCH = 40;
constexpr float MX_LOG2E = 1.44269504088896340736f;

// exp(cap tanh(scale s / cap)) = 2^(c - 2 c / (2^(b s) + 1)),  b = 2 scale log2(e) / cap, c = cap log2(e); c0 in place of
// the first c: times 2^(c0 - c)
__device__ __forceinline__ float cap_exp(float s, float b, float c, float c0) {
  const float r = __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(s * b) + 1.f);
  return __builtin_amdgcn_exp2f(__builtin_fmaf(-2.f * c, r, c0));
}

// A query head's B operand: columns = tokens of the block, zero past the head and the block
template <int DH>
__device__ __forceinline__ void load_q(const MixedArgs& a, int tok, bool ok, int h, int g4, u16x8 (&q)[DH]) {
#pragma unroll
  for (int f = 0; f < DH; ++f) {
    const int d = 32 * f + 8 * g4;
    const u16x8 v = *reinterpret_cast<const u16x8*>((const bf16_t*)a.qn + ((int64_t)tok * a.H + h) * a.D + min(d, a.D - 8));
    q[f] = ok && d < a.D ? v : (u16x8)(0);
  }
}
// 16 keys from key ``off`` of a page: rows past ``last`` and columns past the head are clamped (their scores are masked,
// their factors in q are 0)
template <int DH>
__device__ __forceinline__ void load_k(const MixedArgs& a, const bf16_t* kp, int off, int last, int c16, int g4, u16x8 (&k)[DH]) {
  const bf16_t* p = kp + (int64_t)min(off + c16, last) * a.D;
#pragma unroll
  for (int f = 0; f < DH; ++f) k[f] = *reinterpret_cast<const u16x8*>(p + min(32 * f + 8 * g4, a.D - 8));
}
// keys past the context hold whatever the page held before: their value columns become 0
__device__ __forceinline__ void clear_tail(u16x8& v, int left, int g4) {
#pragma unroll
  for (int j = 0; j < 8; ++j)
    if (8 * g4 + j >= left) v[j] = 0;
}

struct BlockRange {
  int tok0, ntok, lo, hi;  // tokens, keys of this split
};
__device__ __forceinline__ BlockRange block_range(const MixedArgs& a, const int32_t* blk, int nblk, int PS) {
  const int bx = blockIdx.x;
  BlockRange r{blk[bx], blk[nblk + bx], 0, 0};
  if (r.ntok <= 0) return r;  // (a filler)
  r.hi = a.q_ctx[r.tok0 + r.ntok - 1];
  if (PS > 0) {
    r.lo = blockIdx.z * PS;
    r.hi = min(r.hi, r.lo + PS);
  }
  return r;
}

// What a lane owns of a wave's units: one token, heads head(u)
template <int UPW, int HPU>
struct Owner {
  int tok, h0, hh, khi;
  bool ok;
  __device__ __forceinline__ Owner(const MixedArgs& a, const BlockRange& br, int w, int c16) {
    constexpr int TB = 16 / HPU;
    const int t = c16 % TB;
    ok = t < br.ntok;
    tok = br.tok0 + min(t, br.ntok - 1);
    hh = c16 / TB;
    h0 = w * UPW * HPU;
    khi = ok ? a.q_ctx[tok] : 0;
  }
  __device__ __forceinline__ int head(int u) const { return h0 + hh * UPW + u; }
};

// sums [splits][T][H] of exp(s)
template <int DH, int UPW, int HPU, bool SHARE>
__global__ __launch_bounds__(MX_NW * 64) void mixed_sum_kernel(MixedArgs a, const int32_t* __restrict__ blk, int nblk, int PS,
                                                               float* __restrict__ sums, int T) {
  const int lane = threadIdx.x & 63, c16 = lane & 15, g4 = lane >> 4;
  const int w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), rep = a.H / a.G;
  const BlockRange br = block_range(a, blk, nblk, PS);
  if (br.lo >= br.hi || w * UPW * HPU >= a.H) return;
  const Owner<UPW, HPU> own(a, br, w, c16);
  const int32_t* bt = a.bt + (int64_t)a.q_seq[br.tok0] * a.bt_stride;
  const int pmask = (1 << a.page_log2) - 1;
  const int64_t prow = (int64_t)(a.D + a.V) << a.page_log2;
  const float sb = 2.f * a.scale * MX_LOG2E / a.cap, sc = a.cap * MX_LOG2E;
  const int first = a.q_ctx[br.tok0];
  u16x8 q[UPW][DH];
  float l[UPW];
#pragma unroll
  for (int u = 0; u < UPW; ++u) {
    load_q<DH>(a, own.tok, own.ok && own.head(u) < a.H, min(own.head(u), a.H - 1), g4, q[u]);
    l[u] = 0.f;
  }
  u16x8 kf[2][DH];
  auto fetch = [&](int s0, int u) {
    const bf16_t* kp = (const bf16_t*)a.cache + ((int64_t)bt[s0 >> a.page_log2] * a.G + min(own.h0 + u, a.H - 1) / rep) * prow;
    const int off = s0 & pmask, last = off + br.hi - 1 - s0;
#pragma unroll
    for (int sub = 0; sub < 2; ++sub) load_k<DH>(a, kp, off + 16 * sub, last, c16, g4, kf[sub]);
  };
  fetch(br.lo, 0);
  auto tile = [&](int s0, auto masked) {
    constexpr bool MASK = decltype(masked)::value;
    f32x4 st[2][UPW];
#pragma unroll
    for (int u = 0; u < UPW; ++u) {
      if (!SHARE && u > 0) fetch(s0, u);
#pragma unroll
      for (int sub = 0; sub < 2; ++sub) {
        st[sub][u] = (f32x4)(0.f);
#pragma unroll
        for (int f = 0; f < DH; ++f) st[sub][u] = mfma_bf(kf[sub][f], q[u][f], st[sub][u]);
      }
    }
    if (s0 + MX_KEYS < br.hi) fetch(s0 + MX_KEYS, 0);
    const int see = min(own.khi, br.hi) - s0 - 4 * g4;
#pragma unroll
    for (int sub = 0; sub < 2; ++sub)
#pragma unroll
      for (int r = 0; r < 4; ++r)
#pragma unroll
        for (int u = 0; u < UPW; ++u) {
          const float p = cap_exp(st[sub][u][r], sb, sc, sc);
          l[u] += !MASK || 16 * sub + r < see ? p : 0.f;
        }
  };
  int s0 = br.lo;  // (tiles that every token sees whole, then those with an edge)
  for (; s0 + MX_KEYS <= min(first, br.hi); s0 += MX_KEYS) tile(s0, std::false_type{});
  for (; s0 < br.hi; s0 += MX_KEYS) tile(s0, std::true_type{});
#pragma unroll
  for (int u = 0; u < UPW; ++u) {
    l[u] += __shfl_xor(l[u], 16, 64);
    l[u] += __shfl_xor(l[u], 32, 64);
    if (own.ok && g4 == 0 && own.head(u) < a.H) sums[((int64_t)blockIdx.z * T + own.tok) * a.H + own.head(u)] = l[u];
  }
}

// A pair-ordered quarter column (4 values from stored column v, a multiple of 4) of token t, head h: turned back, gated, stored
__device__ __forceinline__ void store_out(const MixedArgs& a, int t, int h, int v, const float* cs, float gate, const f32x4& o) {
  const int m = v >> 1, half = a.V >> 1;
  u16x2 lo, hi;
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const float c = cs[m + i], s = cs[half + m + i], x = o[2 * i], y = o[2 * i + 1];
    lo[i] = f2bf((x * c + y * s) * gate);
    hi[i] = f2bf((y * c - x * s) * gate);
  }
  bf16_t* out = (bf16_t*)a.out;
  const int col = h * a.V + m;
  auto at = [&](int k) { return a.packed_mt > 0 ? apk_off(t, k, a.packed_mt) : (int64_t)t * a.os + k; };
  *reinterpret_cast<u16x2*>(out + at(col)) = lo;
  *reinterpret_cast<u16x2*>(out + at(col + half)) = hi;
}
__device__ __forceinline__ float head_gate(const MixedArgs& a, int t, int h) {
  const float z = bf2f(((const bf16_t*)a.z)[(int64_t)t * a.zs + a.H * a.D + a.G * (a.D + a.V) + h]);
  return 1.f / (1.f + __expf(-z));
}

// LDS: p's two terms [key][token][head], mixed weights [head][token][key]
constexpr int mx_lds(int tb) { return (2 * MX_KEYS + MX_HEADS) * tb * MX_PITCH * 2; }

template <int DH, int VT, int UPW, int HPU, bool SHARE>
__global__ __launch_bounds__(MX_NW * 64) void mixed_core_kernel(MixedArgs a, const int32_t* __restrict__ blk, int nblk, int PS, int SPS,
                                                                const float* __restrict__ sums, float* __restrict__ part,
                                                                int T) {
  constexpr int HB = UPW * HPU > 2 ? 2 : 1, TB = 16 / HPU, NK = 4 / HPU, PTERM = MX_KEYS * TB * MX_PITCH;
  extern __shared__ __attribute__((aligned(16))) bf16_t ph[];
  bf16_t* wt = ph + 2 * PTERM;
  const int tid = threadIdx.x, lane = tid & 63, c16 = lane & 15, g4 = lane >> 4;
  const int w = __builtin_amdgcn_readfirstlane(tid >> 6), H = a.H, rep = a.H / a.G;
  const BlockRange br = block_range(a, blk, nblk, PS);
  if (br.lo >= br.hi) return;
  const Owner<UPW, HPU> own(a, br, w, c16);
  const int32_t* bt = a.bt + (int64_t)a.q_seq[br.tok0] * a.bt_stride;
  const int pmask = (1 << a.page_log2) - 1;
  const int64_t prow = (int64_t)(a.D + a.V) << a.page_log2, voff = (int64_t)a.D << a.page_log2;
  const float sb = 2.f * a.scale * MX_LOG2E / a.cap, sc = a.cap * MX_LOG2E;
  const bool mine = own.h0 < H;
  const int first = a.q_ctx[br.tok0];
  for (int i = tid; i < 2 * PTERM / 8; i += MX_NW * 64) reinterpret_cast<u16x8*>(ph)[i] = (u16x8)(0);
  u16x8 q[UPW][DH];
  f32x4 o[UPW][VT];
  float c0[UPW];  // the score's constant with the row's denominator in it
#pragma unroll
  for (int u = 0; u < UPW; ++u) {
    const int h = min(own.head(u), H - 1);
    load_q<DH>(a, own.tok, own.ok && own.head(u) < H, h, g4, q[u]);
    float l = 1.f;  // the sink
    for (int p = 0; p * SPS < max(own.khi, 1); ++p) l += sums[((int64_t)p * T + own.tok) * H + h];
    c0[u] = sc - __log2f(l);
#pragma unroll
    for (int t = 0; t < VT; ++t) o[u][t] = (f32x4)(0.f);
  }
  u16x8 tf[HB];  // T: row h = 16 hb + c16, column g = 8 g4 + j
#pragma unroll
  for (int hb = 0; hb < HB; ++hb)
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int h = 16 * hb + c16, g = 8 * g4 + j;
      const float t = a.talk[min(h, H - 1) * H + min(g, H - 1)];
      tf[hb][j] = h < H && g < H ? f2bf(t) : (bf16_t)0;
    }
  auto page = [&](int s0, int u) {
    return (const bf16_t*)a.cache + ((int64_t)bt[s0 >> a.page_log2] * a.G + min(own.h0 + u, H - 1) / rep) * prow;
  };
  u16x8 kf[2][DH], vf[VT];
  auto fetch = [&](int s0, int u) {
    const bf16_t* kp = page(s0, u);
    const int off = s0 & pmask, last = off + br.hi - 1 - s0;
#pragma unroll
    for (int sub = 0; sub < 2; ++sub) load_k<DH>(a, kp, off + 16 * sub, last, c16, g4, kf[sub]);
  };
  auto fetch_v = [&](int s0, int u) {
    const bf16_t* vp = page(s0, u) + voff + (int64_t)((s0 & pmask) >> 5) * a.V * 32 + 8 * g4;
#pragma unroll
    for (int t = 0; t < VT; ++t) vf[t] = *reinterpret_cast<const u16x8*>(vp + min(16 * t + c16, a.V - 1) * 32);
  };
  const int pw = (4 * g4 * TB + c16 % TB) * MX_PITCH + own.head(0);             // p: this lane's first place to write
  const int pr = ((4 * w + NK * own.hh) * TB + c16 % TB) * MX_PITCH + 8 * g4;   // and to read
  const int ww = (4 * g4 * TB + c16 % TB) * MX_PITCH + 4 * w + NK * own.hh;     // mixed weights
  if (mine) fetch(br.lo, 0);
  __syncthreads();
  auto tile = [&](int s0, auto masked) {
    constexpr bool MASK = decltype(masked)::value;
    if (mine) {
      if (SHARE) fetch_v(s0, 0);
      f32x4 st[2][UPW];
#pragma unroll
      for (int u = 0; u < UPW; ++u) {
        if (!SHARE && u > 0) fetch(s0, u);
#pragma unroll
        for (int sub = 0; sub < 2; ++sub) {
          st[sub][u] = (f32x4)(0.f);
#pragma unroll
          for (int f = 0; f < DH; ++f) st[sub][u] = mfma_bf(kf[sub][f], q[u][f], st[sub][u]);
        }
      }
      if (s0 + MX_KEYS < br.hi) fetch(s0 + MX_KEYS, 0);
      const int see = min(own.khi, br.hi) - s0 - 4 * g4;
#pragma unroll
      for (int sub = 0; sub < 2; ++sub)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          bf16_t hi[4], lo[4];
#pragma unroll
          for (int u = 0; u < UPW; ++u) {
            const float p = !MASK || 16 * sub + r < see ? cap_exp(st[sub][u][r], sb, sc, c0[u]) : 0.f;
            hi[u] = f2bf(p);
            lo[u] = f2bf(p - bf2f(hi[u]));
          }
          bf16_t* at = ph + pw + (16 * sub + r) * TB * MX_PITCH;
          if constexpr (UPW == 4) {
            *reinterpret_cast<u16x4*>(at) = (u16x4){hi[0], hi[1], hi[2], hi[3]};
            *reinterpret_cast<u16x4*>(at + PTERM) = (u16x4){lo[0], lo[1], lo[2], lo[3]};
          } else if constexpr (UPW == 2) {
            *reinterpret_cast<u16x2*>(at) = (u16x2){hi[0], hi[1]};
            *reinterpret_cast<u16x2*>(at + PTERM) = (u16x2){lo[0], lo[1]};
          } else {
            at[0] = hi[0];
            at[PTERM] = lo[0];
          }
        }
    }
    lds_wait_barrier();
    {  // mix: wave w takes keys 4 w .. 4 w + 3
      f32x4 y[NK][HB];
#pragma unroll
      for (int k = 0; k < NK; ++k) {
        const bf16_t* at = ph + pr + k * TB * MX_PITCH;
        const u16x8 bh = *reinterpret_cast<const u16x8*>(at), bl = *reinterpret_cast<const u16x8*>(at + PTERM);
#pragma unroll
        for (int hb = 0; hb < HB; ++hb) {
          y[k][hb] = mfma_bf(tf[hb], bl, (f32x4)(0.f));
          y[k][hb] = mfma_bf(tf[hb], bh, y[k][hb]);
        }
      }
#pragma unroll
      for (int hb = 0; hb < HB; ++hb)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          bf16_t* at = wt + ww + (16 * hb + r) * TB * MX_PITCH;
          if constexpr (NK == 4)
            *reinterpret_cast<u16x4*>(at) = (u16x4){f2bf(y[0][hb][r]), f2bf(y[1][hb][r]), f2bf(y[2][hb][r]), f2bf(y[NK - 1][hb][r])};
          else
            *reinterpret_cast<u16x2*>(at) = (u16x2){f2bf(y[0][hb][r]), f2bf(y[1][hb][r])};
        }
    }
    lds_wait_barrier();
    if (mine) {
      u16x8 wf[UPW];
#pragma unroll
      for (int u = 0; u < UPW; ++u)
        wf[u] = *reinterpret_cast<const u16x8*>(wt + (min(own.head(u), H - 1) * TB + c16 % TB) * MX_PITCH + 8 * g4);
#pragma unroll
      for (int v = 0; v < (SHARE ? 1 : UPW); ++v) {
        if (!SHARE) fetch_v(s0, v);
#pragma unroll
        for (int t = 0; t < VT; ++t) {
          if constexpr (MASK) clear_tail(vf[t], br.hi - s0, g4);
#pragma unroll
          for (int u = SHARE ? 0 : v; u < (SHARE ? UPW : v + 1); ++u) o[u][t] = mfma_bf(vf[t], wf[u], o[u][t]);
        }
      }
    }
  };
  int s0 = br.lo;  // (tiles that every token sees whole, then those with an edge)
  for (; s0 + MX_KEYS <= min(first, br.hi); s0 += MX_KEYS) tile(s0, std::false_type{});
  for (; s0 < br.hi; s0 += MX_KEYS) tile(s0, std::true_type{});
  if (!mine || !own.ok) return;
#pragma unroll
  for (int u = 0; u < UPW; ++u) {
    const int h = own.head(u);
    if (h >= H) continue;
    if (part != nullptr) {  // [splits][T][H][V]
      float* pp = part + (((int64_t)blockIdx.z * T + own.tok) * H + h) * a.V + 4 * g4;
#pragma unroll
      for (int t = 0; t < VT; ++t)
        if (16 * t < a.V) *reinterpret_cast<f32x4*>(pp + 16 * t) = o[u][t];
      continue;
    }
    const float gate = head_gate(a, own.tok, h);
    const float* cs = a.vrope + (int64_t)(own.khi - 1) * a.V;
#pragma unroll
    for (int t = 0; t < VT; ++t)
      if (16 * t < a.V) store_out(a, own.tok, h, 16 * t + 4 * g4, cs, gate, o[u][t]);
  }
}

// adds the splits of a prompt's block
__global__ __launch_bounds__(256) void mixed_add_kernel(MixedArgs a, const float* __restrict__ part, int T, int PS) {
  const int t = blockIdx.x, HV = a.H * a.V, ctx = a.q_ctx[t];
  if (ctx <= 0) return;
  const float* cs = a.vrope + (int64_t)(ctx - 1) * a.V;
  for (int e = (blockIdx.y * 256 + threadIdx.x) * 4; e < HV; e += gridDim.y * 1024) {
    f32x4 acc = (f32x4)(0.f);
    for (int p = 0; p * PS < ctx; ++p) acc += *reinterpret_cast<const f32x4*>(part + ((int64_t)p * T + t) * HV + e);
    const int h = e / a.V;
    store_out(a, t, h, e - h * a.V, cs, head_gate(a, t, h), acc);
  }
}

// ------------------------------------------------------------------------------------ decode
// UN: score units (kv head, 16 of its heads, 16 keys) of a wave; NT: (kv head, 16 value columns) of a wave
template <int DH, int UN, int NT>
__global__ __launch_bounds__(MX_NW * 64, 2) void mixed_decode_kernel(MixedArgs a, int VT, int PS, float* __restrict__ part,
                                                                     float* __restrict__ sums, int T) {
  __shared__ __attribute__((aligned(16))) bf16_t pb[2][2][MX_HEADS * MX_PITCH];  // [buffer][hi, lo][head][key]
  __shared__ float ls[MX_HEADS];
  const int tid = threadIdx.x, lane = tid & 63, c16 = lane & 15, g4 = lane >> 4;
  const int w = __builtin_amdgcn_readfirstlane(tid >> 6), H = a.H, G = a.G, rep = H / G, hbs = (rep + 15) >> 4;
  const int t = blockIdx.x, ctx = a.q_ctx[t];
  if (ctx <= 0) return;
  const int lo = blockIdx.y * PS, hi = min(ctx, lo + PS);
  if (lo >= hi) return;
  const int32_t* bt = a.bt + (int64_t)a.q_seq[t] * a.bt_stride;
  const int pmask = (1 << a.page_log2) - 1;
  const int64_t prow = (int64_t)(a.D + a.V) << a.page_log2, voff = (int64_t)a.D << a.page_log2;
  const float sb = 2.f * a.scale * MX_LOG2E / a.cap, sc = a.cap * MX_LOG2E;
  for (int i = tid; i < 4 * MX_HEADS * MX_PITCH / 8; i += MX_NW * 64) reinterpret_cast<u16x8*>(pb)[i] = (u16x8)(0);
  if (tid < MX_HEADS) ls[tid] = 0.f;
  // unit i of this wave: number x = w + 8 i of 2 G hbs; kv head x % G, then its head block, then the half of the tile
  int uc[UN], uh[UN], us[UN];
  u16x8 q[UN][DH];
  float l[UN];
#pragma unroll
  for (int i = 0; i < UN; ++i) {
    const int x = w + MX_NW * i, c = x % G, y = x / G;
    const bool on = x < 2 * G * hbs;
    uc[i] = on ? c : -1;
    us[i] = (y / hbs) & 1;
    const int hh = (y % hbs) * 16 + c16;
    uh[i] = on && hh < rep ? c * rep + hh : -1;
    load_q<DH>(a, t, uh[i] >= 0, max(uh[i], 0), g4, q[i]);
    l[i] = 0.f;
  }
  f32x4 o[NT][2];
#pragma unroll
  for (int k = 0; k < NT; ++k) o[k][0] = o[k][1] = (f32x4)(0.f);
  const int tiles = G * VT;
  u16x8 kf[UN][DH];
  auto page = [&](int s0) { return (const bf16_t*)a.cache + (int64_t)bt[s0 >> a.page_log2] * G * prow; };
  auto fetch = [&](const bf16_t* pg, int s0) {
    const int off = s0 & pmask, last = off + min(MX_KEYS, hi - s0) - 1;
#pragma unroll
    for (int i = 0; i < UN; ++i)
      if (uc[i] >= 0) load_k<DH>(a, pg + uc[i] * prow, off + 16 * us[i], last, c16, g4, kf[i]);
  };
  const bf16_t* pg = page(lo);
  fetch(pg, lo);
  __syncthreads();
  int cur = 0;
  auto tile = [&](int s0, auto partial) {
    constexpr bool TAIL = decltype(partial)::value;
    const int left = hi - s0;
    u16x8 vf[NT];
    const bf16_t* vb = pg + voff + (int64_t)((s0 & pmask) >> 5) * a.V * 32 + 8 * g4;
#pragma unroll
    for (int k = 0; k < NT; ++k) {  // wave w: tiles w NT .. of [kv head][16 columns]
      const int x = min(w * NT + k, tiles - 1), c = x / VT, v = (x - c * VT) * 16 + c16;
      vf[k] = *reinterpret_cast<const u16x8*>(vb + c * prow + (int64_t)v * 32);
    }
    f32x4 st[UN];
#pragma unroll
    for (int i = 0; i < UN; ++i) {
      st[i] = (f32x4)(0.f);
      if (uc[i] >= 0)
#pragma unroll
        for (int f = 0; f < DH; ++f) st[i] = mfma_bf(kf[i][f], q[i][f], st[i]);
    }
    if (s0 + MX_KEYS < hi) {
      pg = page(s0 + MX_KEYS);
      fetch(pg, s0 + MX_KEYS);
    }
#pragma unroll
    for (int i = 0; i < UN; ++i) {
      if (uh[i] < 0) continue;
      u16x4 h4, l4;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const bool see = !TAIL || 16 * us[i] + 4 * g4 + r < left;
        const float p = see ? cap_exp(st[i][r], sb, sc, sc) : 0.f;
        l[i] += p;
        h4[r] = f2bf(p);
        l4[r] = f2bf(p - bf2f(h4[r]));
      }
      const int at = uh[i] * MX_PITCH + 16 * us[i] + 4 * g4;
      *reinterpret_cast<u16x4*>(pb[cur][0] + at) = h4;
      *reinterpret_cast<u16x4*>(pb[cur][1] + at) = l4;
    }
    lds_wait_barrier();
    u16x8 bh[2], bl[2];
#pragma unroll
    for (int hb = 0; hb < 2; ++hb) {
      const int at = (16 * hb + c16) * MX_PITCH + 8 * g4;
      bh[hb] = *reinterpret_cast<const u16x8*>(pb[cur][0] + at);
      bl[hb] = *reinterpret_cast<const u16x8*>(pb[cur][1] + at);
    }
#pragma unroll
    for (int k = 0; k < NT; ++k) {
      if constexpr (TAIL) clear_tail(vf[k], left, g4);
#pragma unroll
      for (int hb = 0; hb < 2; ++hb)
        if (16 * hb < H) {  // (uniform)
          o[k][hb] = mfma_bf(vf[k], bl[hb], o[k][hb]);
          o[k][hb] = mfma_bf(vf[k], bh[hb], o[k][hb]);
        }
    }
    cur ^= 1;
  };
  int s0 = lo;
  for (; s0 + MX_KEYS <= hi; s0 += MX_KEYS) tile(s0, std::false_type{});
  if (s0 < hi) tile(s0, std::true_type{});
#pragma unroll
  for (int i = 0; i < UN; ++i) {
    l[i] += __shfl_xor(l[i], 16, 64);
    l[i] += __shfl_xor(l[i], 32, 64);
    if (uh[i] >= 0 && g4 == 0) atomicAdd(&ls[uh[i]], l[i]);  // (two addends a head: any order gives the same sum)
  }
  const int64_t pr = (int64_t)blockIdx.y * T + t;
#pragma unroll
  for (int k = 0; k < NT; ++k) {
    const int x = w * NT + k, c = x / VT, v = (x - c * VT) * 16 + 4 * g4;
    if (x >= tiles) continue;
#pragma unroll
    for (int hb = 0; hb < 2; ++hb)
      if (16 * hb + c16 < H) *reinterpret_cast<f32x4*>(part + ((pr * G + c) * H + 16 * hb + c16) * a.V + v) = o[k][hb];
  }
  __syncthreads();
  if (tid < H) sums[pr * H + tid] = ls[tid];
}

// grid (T, G, column chunks of 32)
__global__ __launch_bounds__(256) void mixed_merge_kernel(MixedArgs a, const float* __restrict__ part,
                                                          const float* __restrict__ sums, int T, int PS) {
  __shared__ float ox[MX_HEADS][36];
  __shared__ float tt[MX_HEADS * MX_HEADS];
  __shared__ float inv[MX_HEADS];
  const int t = blockIdx.x, c = blockIdx.y, v0 = blockIdx.z * 32, tid = threadIdx.x, H = a.H, G = a.G, rep = H / G;
  const int ctx = a.q_ctx[t];
  if (ctx <= 0) return;
  const int np = (ctx + PS - 1) / PS;
  for (int i = tid; i < rep * H; i += 256) tt[i] = a.talk[c * rep * H + i];
  if (tid < H) {
    float l = 1.f;  // the sink
    for (int p = 0; p < np; ++p) l += sums[((int64_t)p * T + t) * H + tid];
    inv[tid] = 1.f / l;
  }
  const int g = tid >> 3, v = v0 + 4 * (tid & 7);
  f32x4 acc = (f32x4)(0.f);
  if (g < H && v < a.V) {
    const int64_t stride = (int64_t)T * G * H * a.V;
    const float* pp = part + (((int64_t)t * G + c) * H + g) * a.V + v;
#pragma unroll 4
    for (int p = 0; p < np; ++p) acc += *reinterpret_cast<const f32x4*>(pp + p * stride);
  }
  __syncthreads();
  if (g < H) {
    const float f = inv[g];
    *reinterpret_cast<f32x4*>(&ox[g][4 * (tid & 7)]) = acc * f;
  }
  __syncthreads();
  const float* cs = a.vrope + (int64_t)(ctx - 1) * a.V;
  for (int i = tid; i < rep * 8; i += 256) {
    const int h = i >> 3, vv = 4 * (i & 7);
    if (v0 + vv >= a.V) continue;
    f32x4 y = (f32x4)(0.f);
    for (int x = 0; x < H; ++x) y += tt[h * H + x] * *reinterpret_cast<const f32x4*>(&ox[x][vv]);
    store_out(a, t, c * rep + h, v0 + vv, cs, head_gate(a, t, c * rep + h), y);
  }
}

struct MixGeom {
  int dh, vt, upw, hpu, share, un, nt;
};
static bool mixed_geometry(int H, int G, int D, int V, MixGeom& m) {
  if (H > MX_HEADS || G < 1 || H % G || D % 8 || D < 8 || D > 128 || V % 16 || V > 128) return false;
  const int rep = H / G;
  m.dh = D <= 64 ? 2 : 4;
  m.vt = V <= 64 ? 4 : 8;
  // many heads: a wave's four share a kv head, or they take a wave's registers to the last
  m.hpu = H > 16 && rep % 4 == 0 ? 2 : 1;
  m.upw = H <= 8 ? 1 : H <= 16 || m.hpu == 2 ? 2 : 4;
  m.share = rep % (m.upw * m.hpu) == 0;
  const int units = (2 * G * ((rep + 15) / 16) + MX_NW - 1) / MX_NW, tiles = (G * V / 16 + MX_NW - 1) / MX_NW;
  m.un = units <= 2 ? 2 : units <= 4 ? 4 : 0;
  m.nt = tiles <= 4 ? 4 : tiles <= 8 ? 8 : tiles <= 16 ? 16 : 0;
  return true;
}

}  // namespace mp

// bit 0: the prompt kernels cover the shape, bit 1: the decode kernels; from bit 8 on: tokens of a prompt's block
extern "C" int mp_mixed_mfma_ok(int H, int G, int D, int V, int page_log2, float cap) {
  using namespace mp;
  MixGeom m;
  if (page_log2 < 5 || !(cap > 0.f && cap <= 64.f) || !mixed_geometry(H, G, D, V, m)) return 0;
  return 1 | (m.un && m.nt ? 2 : 0) | (16 / m.hpu) << 8;
}

// blk [2, nblk] (first token, tokens <= a block's; no tokens: a filler).  The denominators in SNP splits of SPS keys
// (sums: SNP T H floats), the values in NP splits of PS keys (part: NP T H V floats when NP > 1)
extern "C" int mp_mixed_prompt(const void* z, int64_t zs, const void* qn, const float* talk, const void* cache,
                               const int32_t* bt, int bt_stride, const int32_t* q_seq, const int32_t* q_ctx,
                               const float* vrope, void* out, int64_t os, int packed_mt, int n, int H, int G, int D, int V,
                               int page_log2, float scale, float cap, const int32_t* blk, int nblk, int PS, int NP,
                               int SPS, int SNP, float* sums, float* part, hipStream_t stream) {
  using namespace mp;
  (void)hipGetLastError();
  if (n == 0 || nblk == 0) return 0;
  MixGeom m;
  if (!(mp_mixed_mfma_ok(H, G, D, V, page_log2, cap) & 1) || !mixed_geometry(H, G, D, V, m)) return -1;
  if (NP < 1 || NP > 65535 || (NP > 1 && (PS <= 0 || PS % MX_KEYS || part == nullptr))) return -2;
  if (SNP < 1 || SNP > 65535 || SPS <= 0 || SPS % MX_KEYS || sums == nullptr) return -2;
  MixedArgs a{};
  a.z = z, a.zs = zs, a.qn = (void*)qn, a.talk = talk, a.cache = (void*)cache, a.bt = bt, a.bt_stride = bt_stride;
  a.q_seq = q_seq, a.q_ctx = q_ctx, a.vrope = vrope, a.out = out, a.os = os, a.packed_mt = packed_mt;
  a.H = H, a.G = G, a.D = D, a.V = V, a.page_log2 = page_log2, a.scale = scale, a.cap = cap;
  const int ps = NP > 1 ? PS : 0;
  float* pp = NP > 1 ? part : nullptr;
  const dim3 grid(nblk, 1, NP), sgrid(nblk, 1, SNP), nt(MX_NW * 64);
#define MP_MC(DH_, VT_, UPW_, HPU_, SH_)                                                                                \
  {                                                                                                                     \
    constexpr int lds = mx_lds(16 / HPU_);                                                                              \
    (void)hipFuncSetAttribute((const void*)mixed_core_kernel<DH_, VT_, UPW_, HPU_, SH_>,                                \
                              hipFuncAttributeMaxDynamicSharedMemorySize, lds);                                         \
    hipLaunchKernelGGL((mixed_core_kernel<DH_, VT_, UPW_, HPU_, SH_>), grid, nt, lds, stream, a, blk, nblk, ps, SPS, sums, pp, n); \
  }
#define MP_MS(DH_, UPW_, HPU_, SH_)                                                                               \
  {                                                                                                               \
    hipLaunchKernelGGL((mixed_sum_kernel<DH_, UPW_, HPU_, SH_>), sgrid, nt, 0, stream, a, blk, nblk, SPS, sums, n); \
    if (m.vt == 4) MP_MC(DH_, 4, UPW_, HPU_, SH_) else MP_MC(DH_, 8, UPW_, HPU_, SH_)                             \
  }
#define MP_MD(DH_)                              \
  {                                             \
    if (m.hpu == 2) MP_MS(DH_, 2, 2, true)      \
    else if (m.upw == 4) MP_MS(DH_, 4, 1, false) \
    else if (m.upw == 1) MP_MS(DH_, 1, 1, true) \
    else if (m.share) MP_MS(DH_, 2, 1, true)    \
    else MP_MS(DH_, 2, 1, false)                \
  }
  if (m.dh == 2) MP_MD(2) else MP_MD(4)
#undef MP_MD
#undef MP_MS
#undef MP_MC
  if (NP > 1) hipLaunchKernelGGL(mixed_add_kernel, dim3(n, (H * V + 1023) / 1024), dim3(256), 0, stream, a, part, n, PS);
  return (int)hipGetLastError();
}

// every row one token; NP splits of PS keys; part NP n G H V floats, sums NP n H floats
extern "C" int mp_mixed_decode(const void* z, int64_t zs, const void* qn, const float* talk, const void* cache,
                               const int32_t* bt, int bt_stride, const int32_t* q_seq, const int32_t* q_ctx,
                               const float* vrope, void* out, int64_t os, int packed_mt, int n, int H, int G, int D, int V,
                               int page_log2, float scale, float cap, int PS, int NP, float* sums, float* part,
                               hipStream_t stream) {
  using namespace mp;
  (void)hipGetLastError();
  if (n == 0) return 0;
  MixGeom m;
  if (!(mp_mixed_mfma_ok(H, G, D, V, page_log2, cap) & 2) || !mixed_geometry(H, G, D, V, m)) return -1;
  if (NP < 1 || NP > 65535 || PS <= 0 || PS % MX_KEYS || sums == nullptr || part == nullptr) return -2;
  MixedArgs a{};
  a.z = z, a.zs = zs, a.qn = (void*)qn, a.talk = talk, a.cache = (void*)cache, a.bt = bt, a.bt_stride = bt_stride;
  a.q_seq = q_seq, a.q_ctx = q_ctx, a.vrope = vrope, a.out = out, a.os = os, a.packed_mt = packed_mt;
  a.H = H, a.G = G, a.D = D, a.V = V, a.page_log2 = page_log2, a.scale = scale, a.cap = cap;
  const dim3 grid(n, NP), nt(MX_NW * 64);
#define MP_DK(DH_, UN_, NT_) \
  hipLaunchKernelGGL((mixed_decode_kernel<DH_, UN_, NT_>), grid, nt, 0, stream, a, V / 16, PS, part, sums, n)
#define MP_DN(DH_, UN_)             \
  {                                 \
    if (m.nt == 4) MP_DK(DH_, UN_, 4); \
    else if (m.nt == 8) MP_DK(DH_, UN_, 8); \
    else MP_DK(DH_, UN_, 16);       \
  }
  if (m.dh == 2) {
    if (m.un == 2) MP_DN(2, 2) else MP_DN(2, 4)
  } else {
    if (m.un == 2) MP_DN(4, 2) else MP_DN(4, 4)
  }
#undef MP_DN
#undef MP_DK
  hipLaunchKernelGGL(mixed_merge_kernel, dim3(n, G, (V + 31) / 32), dim3(256), 0, stream, a, part, sums, n, PS);
  return (int)hipGetLastError();
}
