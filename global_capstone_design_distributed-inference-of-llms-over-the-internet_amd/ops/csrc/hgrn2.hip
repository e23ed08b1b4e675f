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

#include <type_traits>

namespace mp {

// sigmoid(x) and sigmoid(-x) (its own value, not a difference from 1: a gate near 1 writes little, but exactly)
__device__ __forceinline__ void sigmoid2(float x, float& s, float& c) {
  const float e = __builtin_amdgcn_exp2f(fminf(-1.44269504088896340736f * x, 120.f));  // (finite: e s stays a number)
  s = __builtin_amdgcn_rcpf(1.f + e);
  c = e * s;
}
__device__ __forceinline__ float silu_f(float x) {
  float s, c;
  sigmoid2(x, s, c);
  return x * s;
}

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
  constexpr int PRE = 16;
  extern __shared__ float sm[];  // q[D], f[D], k[D], red[256 * VEC], red16[16]
  const int h = blockIdx.x, D = a.D, V = a.V, tid = threadIdx.x;
  float *sq = sm, *sf = sm + D, *sk = sm + 2 * D, *red = sm + 3 * D, *r16 = red + 256 * VEC;
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
    // the first PRE state rows of this thread are on their way while the gates are made
    float pre[PRE][VEC];
    if (act) {
#pragma unroll
      for (int i = 0; i < PRE; ++i) ld_vec<VEC>(S + (int64_t)min(g + i * ng, D - 1) * V + c, pre[i]);
    }
    const bool fresh = t == tok0 && ctx0 == 1;  // a sequence's first token: the slot's old state does not count
    for (int d = tid; d < D; d += 256) {
      const float zq = ld_f(z, h * D + d), zf = ld_f(z, a.H * D + h * D + d);
      const float lo = a.lower[h * D + d];
      float s, c;
      sigmoid2(zf + a.bias[h * D + d], s, c);
      sq[d] = silu_f(zq);
      sf[d] = lo + (1.f - lo) * s;
      sk[d] = (1.f - lo) * c;
    }
    __syncthreads();
    float o[VEC], v[VEC];
#pragma unroll
    for (int j = 0; j < VEC; ++j) o[j] = 0.f;
    if (act) {
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[j] = ld_f(z, (int64_t)2 * a.H * D + h * V + c + j);
      auto row = [&](int d, float (&s)[VEC]) {
        const float f = sf[d], k = sk[d], qd = sq[d];
#pragma unroll
        for (int j = 0; j < VEC; ++j) {
          s[j] = (fresh ? 0.f : f * s[j]) + k * v[j];
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
  const size_t lds = (3 * a.D + 256 * vec + 16) * sizeof(float);
  if (lds > 60000) return -1;
  if (vec == 4) hipLaunchKernelGGL((hgrn2_scan_kernel<T, 4>), dim3(a.H, n), dim3(256), lds, stream, a, seg, nseg);
  else hipLaunchKernelGGL((hgrn2_scan_kernel<T, 1>), dim3(a.H, n), dim3(256), lds, stream, a, seg, nseg);
  return (int)hipGetLastError();
}

// ---------------------------------------------------------------------------------------
// Prompts.  A segment's tokens are taken 16 at a time by one workgroup per (segment, head), the state in
// registers across the blocks (wave w holds VT 16-column tiles of V for all of D, in the MFMA accumulator
// layout).  With P(a, b] = prod_{a < t <= b} f_t per channel, a block of 16 is
//
//   O  = (q_i P(-1, i]) S  +  tril(A) v        A_ij = sum_d q_i k_j P(j, i]
//   S <- diag(P(-1, 15]) S + (k_j P(j, 15])^T v
//
// every product of gates being a product of numbers <= 1: nothing is divided, no logarithm is taken, and a
// gate of 0 is as good as any other.  A's strictly lower part splits by the highest bit in which i and j
// differ: with L = 8, 4, 2, 1 and m the start of the upper half of their common 2L-block,
// P(j, i] = P(j, m - 1] P(m - 1, i], so ONE table M_L (row t = q_t P(m-1, t] in upper halves,
// k_t P(t, m-1] in lower ones) gives all pairs of that level as the masked product M_L M_L^T; the four
// waves take a level each, and a quarter of the channels of the diagonal.  All products run on v_mfma_f32_16x16x4_f32.
//
// seg [4, nseg]: first token, tokens, source and target of the state (-1: the session's slot, s >= 0: slot s
// of the workspace).  Long prompts are cut into segments so that all CUs work: a STATE pass leaves every
// segment's own contribution (and decay) in the next segment's slot, hgrn2_prefix_kernel turns the slots
// into initial states, and the full pass starts from them.
__device__ __forceinline__ f32x4 mfma_f32(float a, float b, const f32x4& c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

// sum over the 16 lanes of each row of the wave, in every lane
__device__ __forceinline__ float row16_sum(float v) {
  v += dppf<0xB1>(v, 0.f);
  v += dppf<0x4E>(v, 0.f);
  v += dppf<0x141>(v, 0.f);
  v += dppf<0x140>(v, 0.f);
  return v;
}

template <typename T, int DT, int VT, bool STATE>
__global__ __launch_bounds__(256, DT * VT > 32 ? 1 : 2) void hgrn2_chunk_kernel(Hgrn2Args a,
                                                                                const int32_t* __restrict__ seg,
                                                                                int nseg, float* __restrict__ ws,
                                                                                float* __restrict__ wdec) {
  constexpr int DC = DT * 16, DP = DC + 4;
  constexpr int NC = DC > 128 ? 2 : 1;  // gate channels of a thread
  constexpr int NTAB = STATE ? 1 : 7;
  constexpr int TKE = STATE ? 0 : 5, TQB = 4, TQK = 6;
  __shared__ __attribute__((aligned(16))) float tab[NTAB][16][DP];
  __shared__ __attribute__((aligned(16))) float dec[DC];
  __shared__ __attribute__((aligned(16))) float ap[STATE ? 1 : 4][16][20];
  __shared__ float rss[4][16];

  const int h = blockIdx.x, sg = blockIdx.y, tid = threadIdx.x, lane = tid & 63;
  const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int c16 = lane & 15, g4 = lane >> 4;
  const int tok0 = seg[sg], ntok = seg[nseg + sg], src = seg[2 * nseg + sg], dst = seg[3 * nseg + sg];
  if (ntok <= 0 || (STATE && dst < 0)) return;
  const int D = a.D, V = a.V, HD = a.H * D, row = a.q_seq[tok0];
  const bool fresh = src < 0 && a.q_ctx[tok0] <= 1;
  const int64_t blk = (int64_t)D * V;

  f32x4 S[DT][VT];
  {
    const float* sp = src < 0 ? a.state + ((int64_t)row * a.H + h) * blk : ws + ((int64_t)src * a.H + h) * blk;
    const bool zero = STATE || fresh;
#pragma unroll
    for (int m = 0; m < DT; ++m)
#pragma unroll
      for (int v = 0; v < VT; ++v)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int d = 16 * m + 4 * g4 + r, col = (w * VT + v) * 16 + c16;
          S[m][v][r] = !zero && d < D && col < V ? sp[(int64_t)d * V + col] : 0.f;
        }
  }

  // gates: neighbouring lanes share a channel, the even one takes tokens 0..7 of a block, the odd one 8..15
  const int half = tid & 1, ch0 = tid >> 1;
  float lo[NC], bi[NC], run[NC];
  unsigned oq[NC];  // element offset of the channel's first token of this half, from the block's first row
#pragma unroll
  for (int k = 0; k < NC; ++k) {
    const int ch = ch0 + 128 * k;
    lo[k] = ch < D ? a.lower[h * D + ch] : 0.f;
    bi[k] = ch < D ? a.bias[h * D + ch] : 0.f;
    run[k] = 1.f;  // decay of the whole segment (STATE)
    oq[k] = (unsigned)(8 * half * a.zs + h * D + min(ch, D - 1));
  }
  unsigned ov[VT];
  float nw[VT];
#pragma unroll
  for (int v = 0; v < VT; ++v) {
    const int col = (w * VT + v) * 16 + c16;
    ov[v] = (unsigned)(4 * g4 * a.zs + 2 * HD + h * V + min(col, V - 1));
    nw[v] = !STATE && col < V ? a.norm[col] : 0.f;
  }

  T rq[NC][8], rf[NC][8];  // raw gate inputs of the next block, in flight across the MFMAs
  T rv[VT][4];
  auto fetch = [&](int b) {
    const T* z0 = (const T*)a.z + (int64_t)(tok0 + b) * a.zs;
    if (b + 16 <= ntok) {
#pragma unroll
      for (int t = 0; t < 8; ++t) {
        const T* zt = z0 + t * a.zs;  // (uniform base, 32-bit lane offset)
#pragma unroll
        for (int k = 0; k < NC; ++k) {
          if constexpr (!STATE) rq[k][t] = zt[oq[k]];
          rf[k][t] = zt[oq[k] + HD];
        }
      }
#pragma unroll
      for (int s = 0; s < 4; ++s)
#pragma unroll
        for (int v = 0; v < VT; ++v) rv[v][s] = (z0 + s * a.zs)[ov[v]];
      return;
    }
    const int last = ntok - 1 - b;  // the tail block: rows past the end re-read the last one, unused
#pragma unroll
    for (int t = 0; t < 8; ++t)
#pragma unroll
      for (int k = 0; k < NC; ++k) {
        const T* zt = z0 + (int64_t)(min(8 * half + t, last) - 8 * half) * a.zs + oq[k];
        if constexpr (!STATE) rq[k][t] = zt[0];
        rf[k][t] = zt[HD];
      }
#pragma unroll
    for (int s = 0; s < 4; ++s)
#pragma unroll
      for (int v = 0; v < VT; ++v) rv[v][s] = (z0 + (int64_t)(min(4 * g4 + s, last) - 4 * g4) * a.zs)[ov[v]];
  };
  fetch(0);
  for (int b = 0; b < ntok; b += 16) {
    const int nb = min(16, ntok - b);
    if (ch0 < DC) {
#pragma unroll
      for (int kk = 0; kk < NC; ++kk) {
        const int ch = ch0 + 128 * kk;
        float q[8], f[8], k[8];
#pragma unroll
        for (int t = 0; t < 8; ++t) {
          const bool ok = ch < D && 8 * half + t < nb;  // past the end: f = 1, k = 0, q = 0
          if constexpr (!STATE) q[t] = ok ? silu_f(to_f(rq[kk][t])) : 0.f;
          float s, c;
          sigmoid2(to_f(rf[kk][t]) + bi[kk], s, c);
          f[t] = ok ? lo[kk] + (1.f - lo[kk]) * s : 1.f;
          k[t] = ok ? (1.f - lo[kk]) * c : 0.f;
        }
        const int r0 = 8 * half;
        if constexpr (!STATE) {
          auto level = [&](int ti, auto lc) {
            constexpr int L = decltype(lc)::value;
#pragma unroll
            for (int base = 0; base < 8; base += 2 * L) {
              float p = 1.f;
#pragma unroll
              for (int t = base + L - 1; t >= base; --t) {
                tab[ti][r0 + t][ch] = k[t] * p;
                p *= f[t];
              }
              p = 1.f;
#pragma unroll
              for (int t = base + L; t < base + 2 * L; ++t) {
                p *= f[t];
                tab[ti][r0 + t][ch] = q[t] * p;
              }
            }
          };
          level(1, std::integral_constant<int, 4>());
          level(2, std::integral_constant<int, 2>());
          level(3, std::integral_constant<int, 1>());
#pragma unroll
          for (int t = 0; t < 8; ++t) tab[TQK][r0 + t][ch] = q[t] * k[t];
        }
        // products within the half: fw[t] = P up to and with t, bw[t] = P after t
        float fw[8], bw[8];
        fw[0] = f[0];
        bw[7] = 1.f;
#pragma unroll
        for (int t = 1; t < 8; ++t) {
          fw[t] = fw[t - 1] * f[t];
          bw[7 - t] = bw[8 - t] * f[8 - t];
        }
        const float other = dppf<0xB1>(fw[7], 0.f);  // the neighbour lane's half
        const float fp = half ? other : 1.f, bp = half ? 1.f : other;
#pragma unroll
        for (int t = 0; t < 8; ++t) {
          const float x = k[t] * bw[t];
          if constexpr (!STATE) {
            const float y = q[t] * fw[t];
            tab[0][r0 + t][ch] = half ? y : x;  // level 8: upper tokens forward, lower ones backward
            tab[TQB][r0 + t][ch] = y * fp;
          }
          tab[TKE][r0 + t][ch] = x * bp;
        }
        const float all = fw[7] * other;
        if (half == 0) dec[ch] = all;
        run[kk] *= all;
      }
    }
    float vr[VT][4];
#pragma unroll
    for (int v = 0; v < VT; ++v)
#pragma unroll
      for (int s = 0; s < 4; ++s) vr[v][s] = 4 * g4 + s < nb && (w * VT + v) * 16 + c16 < V ? to_f(rv[v][s]) : 0.f;
    if (b + 16 < ntok) fetch(b + 16);
    __syncthreads();

    f32x4 O[VT];
    if constexpr (!STATE) {
      f32x4 sc = (f32x4)(0.f), dg = (f32x4)(0.f);
#pragma unroll
      for (int v = 0; v < VT; ++v) O[v] = (f32x4)(0.f);
#pragma unroll
      for (int m = 0; m < DT; ++m) {
        const f32x4 x = *reinterpret_cast<const f32x4*>(&tab[w][c16][16 * m + 4 * g4]);
        const f32x4 y = *reinterpret_cast<const f32x4*>(&tab[TQB][c16][16 * m + 4 * g4]);
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          sc = mfma_f32(x[r], x[r], sc);
#pragma unroll
          for (int v = 0; v < VT; ++v) O[v] = mfma_f32(y[r], S[m][v][r], O[v]);
        }
        if ((m & 3) == w) {  // the diagonal q_i . k_i: a quarter of the channels each
          const f32x4 u = *reinterpret_cast<const f32x4*>(&tab[TQK][c16][16 * m + 4 * g4]);
#pragma unroll
          for (int r = 0; r < 4; ++r) dg = mfma_f32(u[r], 1.f, dg);
        }
      }
      const int lw = 3 - w;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = 4 * g4 + r, j = c16;
        const bool pair = (i >> (lw + 1)) == (j >> (lw + 1)) && ((i >> lw) & 1) && !((j >> lw) & 1);
        ap[w][i][j] = pair ? sc[r] : i == j ? dg[r] : 0.f;
      }
      __syncthreads();
      f32x4 A = (f32x4)(0.f);
#pragma unroll
      for (int k = 0; k < 4; ++k) A += *reinterpret_cast<const f32x4*>(&ap[k][c16][4 * g4]);
#pragma unroll
      for (int s = 0; s < 4; ++s)
#pragma unroll
        for (int v = 0; v < VT; ++v) O[v] = mfma_f32(A[s], vr[v][s], O[v]);
    }
#pragma unroll
    for (int m = 0; m < DT; ++m) {
      const f32x4 p = *reinterpret_cast<const f32x4*>(&dec[16 * m + 4 * g4]);
      float k[4];
#pragma unroll
      for (int s = 0; s < 4; ++s) k[s] = tab[TKE][4 * g4 + s][16 * m + c16];
#pragma unroll
      for (int v = 0; v < VT; ++v) {
        S[m][v] *= p;
#pragma unroll
        for (int s = 0; s < 4; ++s) S[m][v] = mfma_f32(k[s], vr[v][s], S[m][v]);
      }
    }
    if constexpr (!STATE) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        float x = 0.f;
#pragma unroll
        for (int v = 0; v < VT; ++v) x += O[v][r] * O[v][r];  // (columns past V hold zeros)
        x = row16_sum(x);
        if (c16 == 0) rss[w][4 * g4 + r] = x;
      }
    }
    __syncthreads();
    if constexpr (!STATE) {
      const float inv_v = 1.f / (float)V;
      T* ob = (T*)a.out + (int64_t)(tok0 + b) * a.H * V + h * V;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = 4 * g4 + r;
        const float sc = rsqrtf((rss[0][i] + rss[1][i] + rss[2][i] + rss[3][i]) * inv_v + a.eps);
#pragma unroll
        for (int v = 0; v < VT; ++v) {
          const int col = (w * VT + v) * 16 + c16;
          if (i >= nb || col >= V) continue;
          if (a.packed_mt > 0) st_act((T*)a.out, tok0 + b + i, h * V + col, a.H * V, a.packed_mt, O[v][r] * sc * nw[v]);
          else from_f(O[v][r] * sc * nw[v], ob[(unsigned)(i * a.H * V + col)]);
        }
      }
    }
  }
  if (!STATE && dst >= 0) return;  // (the next segment's workgroup owns the state from here)
  float* sp = dst < 0 ? a.state + ((int64_t)row * a.H + h) * blk : ws + ((int64_t)dst * a.H + h) * blk;
#pragma unroll
  for (int m = 0; m < DT; ++m)
#pragma unroll
    for (int v = 0; v < VT; ++v)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = 16 * m + 4 * g4 + r, col = (w * VT + v) * 16 + c16;
        if (d < D && col < V) sp[(int64_t)d * V + col] = S[m][v][r];
      }
  if (STATE && half == 0) {
#pragma unroll
    for (int k = 0; k < NC; ++k)
      if (ch0 + 128 * k < D) wdec[((int64_t)dst * a.H + h) * D + ch0 + 128 * k] = run[k];
  }
}

// multi [4, nm]: first slot, slots, first token, unused.  Slot i holds segment i-1's contribution (i > 0):
// every slot becomes its segment's initial state.
__global__ __launch_bounds__(256) void hgrn2_prefix_kernel(Hgrn2Args a, const int32_t* __restrict__ multi, int nm,
                                                           float* __restrict__ ws, const float* __restrict__ wdec) {
  const int64_t blk = (int64_t)a.D * a.V;
  const int64_t e = blockIdx.x * (int64_t)256 + threadIdx.x;
  if (e >= blk) return;
  const int h = blockIdx.y, s = blockIdx.z;
  const int slot = multi[s], n = multi[nm + s], tok0 = multi[2 * nm + s];
  const int d = (int)(e / a.V);
  float p = a.q_ctx[tok0] <= 1 ? 0.f : a.state[((int64_t)a.q_seq[tok0] * a.H + h) * blk + e];
  float* x = ws + ((int64_t)slot * a.H + h) * blk + e;
  const float* f = wdec + ((int64_t)slot * a.H + h) * a.D + d;
  const int64_t xs = (int64_t)a.H * blk, fs = (int64_t)a.H * a.D;
  x[0] = p;
  for (int i = 1; i < n; i += 4) {  // four slots' loads in flight
    float u[4], g[4];
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      const int j = min(i + k, n - 1);
      u[k] = x[j * xs];
      g[k] = f[j * fs];
    }
#pragma unroll
    for (int k = 0; k < 4; ++k)
      if (i + k < n) {
        p = g[k] * p + u[k];
        x[(i + k) * xs] = p;
      }
  }
}

template <typename T, bool STATE>
static int launch_chunk(const Hgrn2Args& a, const int32_t* seg, int nseg, float* ws, float* wdec, hipStream_t stream) {
#define MP_HC(DT_, VT_)                                                                                            \
  hipLaunchKernelGGL((hgrn2_chunk_kernel<T, DT_, VT_, STATE>), dim3(a.H, nseg), dim3(256), 0, stream, a, seg, nseg, \
                     ws, wdec)
  const int dt = (a.D + 15) / 16, vt = (a.V + 63) / 64;
  if (dt > 16 || vt > 4) return -1;
  if (dt <= 4) {
    if (vt <= 1) MP_HC(4, 1); else if (vt <= 2) MP_HC(4, 2); else MP_HC(4, 4);
  } else if (dt <= 8) {
    if (vt <= 1) MP_HC(8, 1); else if (vt <= 2) MP_HC(8, 2); else MP_HC(8, 4);
  } else {
    if (vt <= 2) MP_HC(16, 2); else MP_HC(16, 4);
  }
#undef MP_HC
  return (int)hipGetLastError();
}

}  // namespace mp

// seg [4, nseg] (all of the step), multi [4, nm] (sequences cut into several segments; ws / wdec hold their slots)
extern "C" int mp_hgrn2_chunk(const void* z, int64_t zs, const float* bias, const float* lower, const float* norm,
                              float* state, const int32_t* q_seq, const int32_t* q_ctx, void* out, int H, int D, int V,
                              float eps, const int32_t* seg, int nseg, const int32_t* multi, int nm, float* ws,
                              float* wdec, int packed_mt, int f32, hipStream_t stream) {
  using namespace mp;
  (void)hipGetLastError();
  if (nseg == 0) return 0;
  if (nseg > 65535 || nm > 65535 || H > 65535) return -1;
  const Hgrn2Args a{z, zs, bias, lower, norm, state, q_seq, q_ctx, out, H, D, V, packed_mt, eps};
  int rc;
  if (nm > 0) {
    rc = f32 ? launch_chunk<float, true>(a, seg, nseg, ws, wdec, stream)
             : launch_chunk<bf16_t, true>(a, seg, nseg, ws, wdec, stream);
    if (rc) return rc;
    hipLaunchKernelGGL(hgrn2_prefix_kernel, dim3((unsigned)(((int64_t)D * V + 255) / 256), H, nm), dim3(256), 0, stream,
                       a, multi, nm, ws, wdec);
    rc = (int)hipGetLastError();
    if (rc) return rc;
  }
  return f32 ? launch_chunk<float, false>(a, seg, nseg, ws, wdec, stream)
             : launch_chunk<bf16_t, false>(a, seg, nseg, ws, wdec, stream);
}

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
