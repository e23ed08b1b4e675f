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
//   linear_chunk_kernel  prompts in bf16: 32-token blocks on bf16 MFMA, the state resident in registers
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

// ---------------------------------------------------------------------------------------
// Prompts.  A segment's tokens are taken 32 at a time by one workgroup per (segment, head); wave w holds VT 16-column
// tiles of S for all of D in fp32 accumulators.  With G_t the log2 decays summed from the block's start and i_t the log2
// input weights (retention: 0), every weight of a block is exp2 of a difference that is never positive:
//
//   M_t = max(M_in, max_{j <= t} (i_j - G_j))      the running maximum less G_t (retention: no maximum, M_t = -G_t)
//   A_tj = q_t . k_j exp2((i_j - G_j) - M_t)       o_t = exp2(M_in - M_t) S^T q_t + sum_{j <= t} A_tj v_j
//   S <- exp2(M_in - M_end) S + sum_j exp2((i_j - G_j) - M_end) k_j v_j^T
//
// 32-bit factors enter the bf16 products as hi + lo pairs (S, A, the weighted v, and retention's turned q and k); the
// projections themselves are bf16 and exact.  S is an operand straight from its accumulators: q and k lie in LDS in
// the column order that the accumulator layout gives (kpos), v and k^T come by transposed LDS reads.
//
// seg [4, nseg]: first token, tokens, source and target of the state (-1: the session's slot, s >= 0: slot s of the
// workspace).  Long prompts are cut into segments so that all CUs work: a STATE pass leaves every segment's own
// contribution in the next segment's slot, linear_prefix_kernel turns the slots into initial states, and the full pass
// starts from them.  A slot holds, per head, S, the normalizer and four numbers: the contribution's maximum, the
// segment's summed log2 decay, and the initial state's maximum.
typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8_c;
typedef short s16x4_c __attribute__((ext_vector_type(4)));
__device__ __forceinline__ f32x4 mfma_c(const u16x8& a, const u16x8& b, const f32x4& c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_c, a), __builtin_bit_cast(bf16x8_c, b), c, 0,
                                                 0, 0);
}
__device__ __forceinline__ u16x8 lds_tr8(const bf16_t* p, int step) {
  const s16x4_c a = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4_c*)(p));
  const s16x4_c b = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4_c*)(p + step));
  const u16x4 x = __builtin_bit_cast(u16x4, a), y = __builtin_bit_cast(u16x4, b);
  return (u16x8){x[0], x[1], x[2], x[3], y[0], y[1], y[2], y[3]};
}
__device__ __forceinline__ void split8(const float (&x)[8], u16x8& hi, u16x8& lo) {
#pragma unroll
  for (int j = 0; j < 8; ++j) {
    hi[j] = f2bf(x[j]);
    lo[j] = f2bf(x[j] - bf2f(hi[j]));
  }
}

constexpr int LC_TOK = 32, LC_AS = LC_TOK + 8, LC_EXTRA = 4;
constexpr float L2E = 1.44269504088896340736f, LN2 = 0.69314718055994530942f;

// LDS position of columns d .. d + 3 (d a multiple of 4) of a 32-column slice
__device__ __forceinline__ int kpos(int d) { return (d & ~31) + 8 * ((d & 15) >> 2) + 4 * ((d >> 4) & 1); }

template <int KIND, int DF, int VT, bool STATE>
struct ChunkLds {
  static constexpr int QS = 32 * DF + 8, VS = 64 * VT + 8;
  static constexpr int NQK = (STATE ? 1 : 2) * (KIND == RETENTION ? 2 : 1);  // q, k as hi (+ lo)
  static constexpr int K = 0, KL = LC_TOK * QS, Q = (KIND == RETENTION ? 2 : 1) * LC_TOK * QS, QL = Q + LC_TOK * QS;
  static constexpr int VV = NQK * LC_TOK * QS, AH = VV + LC_TOK * VS, AL = AH + LC_TOK * LC_AS;
  static constexpr int FL = (STATE ? AH : AL + LC_TOK * LC_AS);  // floats from here (in bf16 elements, a multiple of 8)
  static constexpr int NFL = 32 * 5 + 64 + 32 + 128 + 8 + (KIND == MLSTM ? 32 * DF : 0);
  static constexpr size_t BYTES = FL * 2 + NFL * 4;
};

template <int KIND, int DF, int VT, bool STATE>
__global__ __launch_bounds__(256, DF * VT <= 4 || (DF == 4 && VT == 2) ? 2 : 1) void linear_chunk_kernel(LinArgs a, const int32_t* __restrict__ seg,
                                                                                 int nseg, float* __restrict__ ws) {
  typedef ChunkLds<KIND, DF, VT, STATE> L;
  constexpr int NI = DF > 4 ? DF / 4 : 1;  // pair items of a thread
  constexpr int DT = 2 * DF;
  extern __shared__ __attribute__((aligned(16))) bf16_t lc[];
  float* fl = reinterpret_cast<float*>(lc + L::FL);
  float *xs = fl, *ys = fl + 32, *inter = fl + 64, *upd = fl + 96, *flo = fl + 128, *asum = fl + 160, *qnv = fl + 224,
        *rss = fl + 256, *scal = fl + 384, *nrm = fl + 392;

  const int h = blockIdx.x, sg = blockIdx.y, tid = threadIdx.x, lane = tid & 63;
  const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int c16 = lane & 15, g4 = lane >> 4;
  const int tok0 = seg[sg], ntok = seg[nseg + sg], src = seg[2 * nseg + sg], dst = seg[3 * nseg + sg];
  if (ntok <= 0 || (STATE && dst < 0)) return;
  const int H = a.H, D = a.D, V = a.V;
  const int64_t row = (int64_t)a.q_seq[tok0] * H + h;
  const int pos0 = a.q_ctx[tok0] - 1;
  const bool fresh = src < 0 && pos0 <= 0;
  const int64_t blk = (int64_t)D * V, wst = blk + D + LC_EXTRA;
  const bf16_t* zb = (const bf16_t*)a.z + (int64_t)tok0 * a.zs;
  const float ld = KIND == RETENTION ? a.decay[h] : 0.f, qks = a.qs * a.ks;

  for (int x = tid; x < L::FL / 8; x += 256) *reinterpret_cast<u16x8*>(lc + 8 * x) = (u16x8)(0);  // pads stay 0
  f32x4 S[DT][VT];
  {
    const float* sp = src < 0 ? a.state + row * blk : ws + ((int64_t)src * H + h) * wst;
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
  float m_in = STATE ? -INFINITY : 0.f, gsum = 0.f;  // wave 0's: running maximum (log2), summed log2 decay
  if constexpr (KIND == MLSTM) {
    const float* np = src < 0 ? a.aux + row * (D + 1) : ws + ((int64_t)src * H + h) * wst + blk;
    if (!STATE && !fresh) m_in = src < 0 ? np[D] * L2E : np[D + 2];
    for (int d = tid; d < 32 * DF; d += 256)
      nrm[kpos(d & ~3) + (d & 3)] = !STATE && !fresh && d < D ? np[d] : 0.f;
  }

  // pair items: columns c0 .. + 7 and c1 .. + 7 of a token; the first rot / 16 of a row turn together
  int it_row[NI], it_c0[NI], it_c1[NI], it_cs[NI];
#pragma unroll
  for (int n = 0; n < NI; ++n) {
    const int x = tid + 256 * n, per = D >> 4, r = x / per, it = x - r * per;
    it_row[n] = r < LC_TOK ? r : -1;
    const int nr = KIND == RETENTION ? a.rot >> 4 : 0;
    it_cs[n] = it < nr ? 8 * it : -1;
    it_c0[n] = it < nr ? 8 * it : (nr << 4) + 16 * (it - nr);
    it_c1[n] = it < nr ? 8 * it + (a.rot >> 1) : it_c0[n] + 8;
  }
  const int vper = V >> 3;
  u16x8 rq[NI][2], rk[NI][2], rv[VT];
  f32x4 rc[NI][4];
  float rgi = 0.f, rgf = 0.f;
  auto fetch = [&](int b) {
    const int last = ntok - 1 - b;
#pragma unroll
    for (int n = 0; n < NI; ++n) {
      const int r = min(max(it_row[n], 0), last);
      const bf16_t* z = zb + (int64_t)(b + r) * a.zs + h * D;
      const bf16_t* zk = z + H * D;
      if constexpr (!STATE) {
        rq[n][0] = *reinterpret_cast<const u16x8*>(z + it_c0[n]);
        rq[n][1] = *reinterpret_cast<const u16x8*>(z + it_c1[n]);
      }
      rk[n][0] = *reinterpret_cast<const u16x8*>(zk + it_c0[n]);
      rk[n][1] = *reinterpret_cast<const u16x8*>(zk + it_c1[n]);
      if constexpr (KIND == RETENTION) {
        if (a.rot > 0) {
          const float* cs = a.rope + (int64_t)(pos0 + b + r) * a.rot + max(it_cs[n], 0);
          rc[n][0] = *reinterpret_cast<const f32x4*>(cs);
          rc[n][1] = *reinterpret_cast<const f32x4*>(cs + 4);
          rc[n][2] = *reinterpret_cast<const f32x4*>(cs + (a.rot >> 1));
          rc[n][3] = *reinterpret_cast<const f32x4*>(cs + (a.rot >> 1) + 4);
        }
      }
    }
#pragma unroll
    for (int n = 0; n < VT; ++n) {
      const int x = tid + 256 * n, r = x / vper;
      rv[n] = *reinterpret_cast<const u16x8*>(zb + (int64_t)(b + min(r, last)) * a.zs + 2 * H * D + h * V +
                                              (x - r * vper) * 8);
    }
    if constexpr (KIND == MLSTM) {
      if (w == 0) {
        const bf16_t* z = zb + (int64_t)(b + min(lane & 31, last)) * a.zs + 2 * H * (D + V) + h;
        rgi = bf2f(z[0]);
        rgf = bf2f(z[H]);
      }
    }
  };
  auto put = [&](int r, int c, const u16x8& v, bf16_t* t) {  // 8 columns into their LDS order
    *reinterpret_cast<u16x4*>(t + r * L::QS + kpos(c)) = (u16x4){v[0], v[1], v[2], v[3]};
    *reinterpret_cast<u16x4*>(t + r * L::QS + kpos(c + 4)) = (u16x4){v[4], v[5], v[6], v[7]};
  };
  auto stash = [&](int nb) {
#pragma unroll
    for (int n = 0; n < NI; ++n) {
      const int r = it_row[n];
      if (r < 0) continue;
      const bool ok = r < nb;
      auto one = [&](const u16x8& x0, const u16x8& x1, bf16_t* th, bf16_t* tl) {
        if constexpr (KIND == MLSTM) {
          put(r, it_c0[n], ok ? x0 : (u16x8)(0), th);
          put(r, it_c1[n], ok ? x1 : (u16x8)(0), th);
        } else {
          float u[8], v[8];
#pragma unroll
          for (int j = 0; j < 8; ++j) {
            const float p = ok ? bf2f(x0[j]) : 0.f, q = ok ? bf2f(x1[j]) : 0.f;
            const float c = it_cs[n] >= 0 ? rc[n][j >> 2][j & 3] : 1.f, s = it_cs[n] >= 0 ? rc[n][2 + (j >> 2)][j & 3] : 0.f;
            u[j] = p * c - q * s;
            v[j] = q * c + p * s;
          }
          u16x8 uh, ul, vh, vl;
          split8(u, uh, ul);
          split8(v, vh, vl);
          put(r, it_c0[n], uh, th);
          put(r, it_c1[n], vh, th);
          put(r, it_c0[n], ul, tl);
          put(r, it_c1[n], vl, tl);
        }
      };
      one(rk[n][0], rk[n][1], lc + L::K, lc + L::KL);
      if constexpr (!STATE) one(rq[n][0], rq[n][1], lc + L::Q, lc + L::QL);
    }
#pragma unroll
    for (int n = 0; n < VT; ++n) {
      const int x = tid + 256 * n, r = x / vper;
      if (r < LC_TOK)
        *reinterpret_cast<u16x8*>(lc + L::VV + r * L::VS + (x - r * vper) * 8) = r < nb ? rv[n] : (u16x8)(0);
    }
    if (w == 0) {  // the block's weights
      const int j = lane & 31;
      if constexpr (KIND == MLSTM) {
        const bool ok = j < nb;
        float G = ok ? log_sigmoid(soft_cap(rgf + a.bias[H + h], a.cap)) * L2E : 0.f;
        const float li = soft_cap(rgi + a.bias[h], a.cap) * L2E;
#pragma unroll
        for (int s = 1; s < 32; s <<= 1) {
          const float o = __shfl_up(G, s, 32);
          if (j >= s) G += o;
        }
        const float y = ok ? li - G : -INFINITY;
        float M = y;
#pragma unroll
        for (int s = 1; s < 32; s <<= 1) {
          const float o = __shfl_up(M, s, 32);
          if (j >= s) M = fmaxf(M, o);
        }
        M = fmaxf(M, m_in);
        const float Me = __shfl(M, 31, 32), Ge = __shfl(G, 31, 32);
        if (lane < 32) {
          xs[j] = M;
          ys[j] = y;
          inter[j] = __builtin_amdgcn_exp2f(m_in - M) * a.qs;
          upd[j] = __builtin_amdgcn_exp2f(y - Me) * a.ks;
          flo[j] = __builtin_amdgcn_exp2f(-(G + M));
          if (j == 0) scal[0] = __builtin_amdgcn_exp2f(m_in - Me);
        }
        m_in = Ge + Me;
        gsum += Ge;
      } else if (lane < 32) {
        xs[j] = -(float)j * ld;
        ys[j] = -(float)j * ld;
        inter[j] = __builtin_amdgcn_exp2f((float)(j + 1) * ld) * a.qs;
        upd[j] = j < nb ? __builtin_amdgcn_exp2f((float)(nb - 1 - j) * ld) * a.ks : 0.f;
        if (j == 0) scal[0] = __builtin_amdgcn_exp2f((float)nb * ld);
      }
    }
  };

  const bf16_t *kf = lc + L::K + c16 * L::QS + 8 * g4, *qf = lc + L::Q + c16 * L::QS + 8 * g4;
  const bf16_t* kt = lc + L::K + (4 * g4 + (c16 >> 2)) * L::QS + 8 * (c16 & 3);
  const bf16_t* vt = lc + L::VV + (4 * g4 + (c16 >> 2)) * L::VS + w * VT * 16 + 4 * (c16 & 3);
  constexpr int LO = LC_TOK * L::QS;  // a lo tile lies behind its hi tile
  fetch(0);
  __syncthreads();  // (the pads are zero)
  for (int b = 0; b < ntok; b += LC_TOK) {
    const int nb = min(LC_TOK, ntok - b);
    stash(nb);
    if (b + LC_TOK < ntok) fetch(b + LC_TOK);
    __syncthreads();
    const float dec = scal[0];
    f32x4 O[2][VT];
    if constexpr (!STATE) {
      // scores of tile (query half w >> 1, key half w & 1); a lane owns query c16, keys 4 g4 ..
      const int it = w >> 1, jt = w & 1;
      f32x4 sc = (f32x4)(0.f);
      if (jt <= it) {
#pragma unroll
        for (int f = 0; f < DF; ++f) {
          const u16x8 kh = *reinterpret_cast<const u16x8*>(kf + 16 * jt * L::QS + 32 * f);
          const u16x8 qh = *reinterpret_cast<const u16x8*>(qf + 16 * it * L::QS + 32 * f);
          sc = mfma_c(kh, qh, sc);
          if constexpr (KIND == RETENTION) {
            const u16x8 kl = *reinterpret_cast<const u16x8*>(kf + LO + 16 * jt * L::QS + 32 * f);
            const u16x8 ql = *reinterpret_cast<const u16x8*>(qf + LO + 16 * it * L::QS + 32 * f);
            sc = mfma_c(kh, ql, sc);
            sc = mfma_c(kl, qh, sc);
          }
        }
      }
      const int i = 16 * it + c16;
      const float xi = xs[i];
      u16x4 ah, al;
      float sum = 0.f;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int j = 16 * jt + 4 * g4 + r;
        const float x = j <= i ? sc[r] * __builtin_amdgcn_exp2f(ys[j] - xi) * qks : 0.f;
        ah[r] = f2bf(x);
        al[r] = f2bf(x - bf2f(ah[r]));
        sum += x;
      }
      *reinterpret_cast<u16x4*>(lc + L::AH + i * LC_AS + 8 * g4 + 4 * jt) = ah;
      *reinterpret_cast<u16x4*>(lc + L::AL + i * LC_AS + 8 * g4 + 4 * jt) = al;
      if constexpr (KIND == MLSTM) {
        sum += __shfl_xor(sum, 16, 64);
        sum += __shfl_xor(sum, 32, 64);
        if (g4 == 0) asum[32 * jt + i] = sum;
        const int t = tid >> 3, p0 = (tid & 7) * 4 * DF;  // n . q of token t, an eighth of the columns each
        float s = 0.f;
#pragma unroll
        for (int p = 0; p < 4 * DF; p += 4) {
          const u16x4 q = *reinterpret_cast<const u16x4*>(lc + L::Q + t * L::QS + p0 + p);
          const f32x4 n = *reinterpret_cast<const f32x4*>(nrm + p0 + p);
#pragma unroll
          for (int j = 0; j < 4; ++j) s += bf2f(q[j]) * n[j];
        }
        s += __shfl_xor(s, 1, 64);
        s += __shfl_xor(s, 2, 64);
        s += __shfl_xor(s, 4, 64);
        if ((tid & 7) == 0) qnv[t] = s;
      }
#pragma unroll
      for (int i2 = 0; i2 < 2; ++i2)
#pragma unroll
        for (int v = 0; v < VT; ++v) O[i2][v] = (f32x4)(0.f);
    }
    u16x8 vf[VT], wh[VT], wl[VT];
    {
      const f32x4 u0 = *reinterpret_cast<const f32x4*>(upd + 4 * g4), u1 = *reinterpret_cast<const f32x4*>(upd + 16 + 4 * g4);
#pragma unroll
      for (int v = 0; v < VT; ++v) {
        vf[v] = lds_tr8(vt + 16 * v, 16 * L::VS);
        float x[8];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          x[j] = bf2f(vf[v][j]) * u0[j];
          x[4 + j] = bf2f(vf[v][4 + j]) * u1[j];
        }
        split8(x, wh[v], wl[v]);
      }
    }
#pragma unroll
    for (int f = 0; f < DF; ++f) {
      if constexpr (!STATE) {
        u16x8 qh[2], ql[2];
#pragma unroll
        for (int i2 = 0; i2 < 2; ++i2) {
          qh[i2] = *reinterpret_cast<const u16x8*>(qf + 16 * i2 * L::QS + 32 * f);
          if constexpr (KIND == RETENTION) ql[i2] = *reinterpret_cast<const u16x8*>(qf + LO + 16 * i2 * L::QS + 32 * f);
        }
#pragma unroll
        for (int v = 0; v < VT; ++v) {
          const f32x4 s0 = S[2 * f][v], s1 = S[2 * f + 1][v];
          const float x[8] = {s0[0], s0[1], s0[2], s0[3], s1[0], s1[1], s1[2], s1[3]};
          u16x8 sh, sl;
          split8(x, sh, sl);
#pragma unroll
          for (int i2 = 0; i2 < 2; ++i2) {
            O[i2][v] = mfma_c(sh, qh[i2], O[i2][v]);
            O[i2][v] = mfma_c(sl, qh[i2], O[i2][v]);
            if constexpr (KIND == RETENTION) O[i2][v] = mfma_c(sh, ql[i2], O[i2][v]);
          }
        }
      }
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        const u16x8 kh = lds_tr8(kt + 32 * f + 4 * half, 16 * L::QS);
        u16x8 kl;
        if constexpr (KIND == RETENTION) kl = lds_tr8(kt + LO + 32 * f + 4 * half, 16 * L::QS);
#pragma unroll
        for (int v = 0; v < VT; ++v) {
          f32x4& s = S[2 * f + half][v];
          s *= dec;
          s = mfma_c(kh, wh[v], s);
          s = mfma_c(kh, wl[v], s);
          if constexpr (KIND == RETENTION) s = mfma_c(kl, wh[v], s);
        }
      }
    }
    if constexpr (!STATE) {
#pragma unroll
      for (int i2 = 0; i2 < 2; ++i2)
#pragma unroll
        for (int v = 0; v < VT; ++v) O[i2][v] *= inter[16 * i2 + c16];
    }
    u16x4 gz[2][VT];
    if constexpr (!STATE) {
#pragma unroll
      for (int i2 = 0; i2 < 2; ++i2)
#pragma unroll
        for (int v = 0; v < VT; ++v)
          gz[i2][v] = *reinterpret_cast<const u16x4*>(zb + (int64_t)(b + min(16 * i2 + c16, nb - 1)) * a.zs + 2 * H * D +
                                                      H * V + h * V + min((w * VT + v) * 16 + 4 * g4, V - 4));
    }
    __syncthreads();
    if constexpr (KIND == MLSTM) {
      for (int p = tid; p < 32 * DF; p += 256) {
        float n = nrm[p] * dec;
#pragma unroll 8
        for (int j = 0; j < LC_TOK; ++j) n += upd[j] * bf2f(lc[L::K + j * L::QS + p]);
        nrm[p] = n;
      }
    }
    if constexpr (!STATE) {
#pragma unroll
      for (int i2 = 0; i2 < 2; ++i2) {
        const int i = 16 * i2 + c16;
        const u16x8 ah = *reinterpret_cast<const u16x8*>(lc + L::AH + i * LC_AS + 8 * g4);
        const u16x8 al = *reinterpret_cast<const u16x8*>(lc + L::AL + i * LC_AS + 8 * g4);
        float den = 1.f, ss = 0.f;
        if constexpr (KIND == MLSTM)
          den = 1.f / (fmaxf(fabsf(qnv[i] * inter[i] + asum[i] + asum[32 + i]), flo[i]) + 1e-6f);
#pragma unroll
        for (int v = 0; v < VT; ++v) {
          O[i2][v] = mfma_c(vf[v], ah, O[i2][v]);
          O[i2][v] = mfma_c(vf[v], al, O[i2][v]);
          O[i2][v] *= den;
#pragma unroll
          for (int r = 0; r < 4; ++r) ss += O[i2][v][r] * O[i2][v][r];  // (columns past V hold zeros)
        }
        ss += __shfl_xor(ss, 16, 64);
        ss += __shfl_xor(ss, 32, 64);
        if (g4 == 0) rss[w * 32 + i] = ss;
      }
    }
    __syncthreads();
    if constexpr (!STATE) {
      const float inv_v = 1.f / (float)V;
#pragma unroll
      for (int i2 = 0; i2 < 2; ++i2) {
        const int i = 16 * i2 + c16;
        const float sc = 1.f / sqrtf((rss[i] + rss[32 + i] + rss[64 + i] + rss[96 + i]) * inv_v + a.eps);
#pragma unroll
        for (int v = 0; v < VT; ++v) {
          const int col = (w * VT + v) * 16 + 4 * g4;
          if (i >= nb || col >= V) continue;
          float y[4];
          f32x4 nw = (f32x4)(1.f);
          if constexpr (KIND == MLSTM) nw = *reinterpret_cast<const f32x4*>(a.norm + h * V + col);
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const float g = bf2f(gz[i2][v][r]);
            const float s = __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(fminf(-L2E * g, 120.f)));
            y[r] = O[i2][v][r] * sc * (KIND == MLSTM ? nw[r] * s : g * s);
          }
          st_act_vec<4>((bf16_t*)a.out, tok0 + b + i, h * V + col, H * V, a.packed_mt, y);
        }
      }
    }
  }
  if (!STATE && dst >= 0) return;  // (the next segment's workgroup owns the state from here)
  float* sp = dst < 0 ? a.state + row * blk : ws + ((int64_t)dst * H + h) * wst;
#pragma unroll
  for (int m = 0; m < DT; ++m)
#pragma unroll
    for (int v = 0; v < VT; ++v)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = 16 * m + 4 * g4 + r, col = (w * VT + v) * 16 + c16;
        if (d < D && col < V) sp[(int64_t)d * V + col] = S[m][v][r];
      }
  if constexpr (KIND == MLSTM) {
    float* np = dst < 0 ? a.aux + row * (D + 1) : sp + blk;
    for (int d = tid; d < D; d += 256) np[d] = nrm[kpos(d & ~3) + (d & 3)];
    if (tid == 0) {
      np[D] = dst < 0 ? m_in * LN2 : m_in;
      if (dst >= 0) np[D + 1] = gsum;
    }
  } else if (STATE && tid == 0) {
    sp[blk + D + 1] = (float)ntok * ld;
  }
}

// multi [4, nm]: first slot, slots, first token, unused.  Slot i holds segment i-1's contribution (i > 0):
// every slot becomes its segment's initial state.
template <int KIND>
__global__ __launch_bounds__(256) void linear_prefix_kernel(LinArgs a, const int32_t* __restrict__ multi, int nm,
                                                            float* __restrict__ ws) {
  const int64_t blk = (int64_t)a.D * a.V, wst = blk + a.D + LC_EXTRA;
  const int64_t e = blockIdx.x * (int64_t)256 + threadIdx.x;
  if (e >= blk + (KIND == MLSTM ? a.D : 0)) return;
  const int h = blockIdx.y, s = blockIdx.z;
  const int slot = multi[s], n = multi[nm + s], tok0 = multi[2 * nm + s];
  const int64_t row = (int64_t)a.q_seq[tok0] * a.H + h, xs = (int64_t)a.H * wst;
  const bool fresh = a.q_ctx[tok0] <= 1;
  float p = fresh ? 0.f : e < blk ? a.state[row * blk + e] : a.aux[row * (a.D + 1) + e - blk];
  float m = KIND == MLSTM && !fresh ? a.aux[row * (a.D + 1) + a.D] * L2E : 0.f;
  float* x = ws + ((int64_t)slot * a.H + h) * wst;
  x[e] = p;
  if (KIND == MLSTM && e == 0) x[blk + a.D + 2] = m;
  for (int i = 1; i < n; i += 4) {  // four slots' loads in flight
    float u[4], mc[4], g[4];
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      const float* y = x + min(i + k, n - 1) * xs;
      u[k] = y[e];
      mc[k] = KIND == MLSTM ? y[blk + a.D] : 0.f;
      g[k] = y[blk + a.D + 1];
    }
#pragma unroll
    for (int k = 0; k < 4; ++k)
      if (i + k < n) {
        if constexpr (KIND == MLSTM) {
          const float mn = fmaxf(g[k] + m, mc[k]);
          p = __builtin_amdgcn_exp2f(g[k] + m - mn) * p + __builtin_amdgcn_exp2f(mc[k] - mn) * u[k];
          m = mn;
          if (e == 0) x[(i + k) * xs + blk + a.D + 2] = m;
        } else {
          p = __builtin_amdgcn_exp2f(g[k]) * p + u[k];
        }
        x[(i + k) * xs + e] = p;
      }
  }
}

template <int KIND, bool STATE>
static int launch_linear_chunk(const LinArgs& a, const int32_t* seg, int nseg, float* ws, hipStream_t stream) {
#define MP_LC(DF_, VT_)                                                                                              \
  {                                                                                                                  \
    constexpr size_t lds = ChunkLds<KIND, DF_, VT_, STATE>::BYTES;                                                   \
    if (lds > 65536)                                                                                                 \
      (void)hipFuncSetAttribute((const void*)linear_chunk_kernel<KIND, DF_, VT_, STATE>,                             \
                                hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);                               \
    hipLaunchKernelGGL((linear_chunk_kernel<KIND, DF_, VT_, STATE>), dim3(a.H, nseg), dim3(256), lds, stream, a, seg, \
                       nseg, ws);                                                                                    \
  }
#define MP_LCV(DF_)                 \
  if (a.V <= 64) MP_LC(DF_, 1)      \
  else if (a.V <= 128) MP_LC(DF_, 2) \
  else MP_LC(DF_, 4)
  if (a.D <= 64) { MP_LCV(2) } else if (a.D <= 128) { MP_LCV(4) } else { MP_LCV(8) }
#undef MP_LCV
#undef MP_LC
  return (int)hipGetLastError();
}

template <int KIND>
static int launch_linear_prompt(const LinArgs& a, const int32_t* seg, int nseg, const int32_t* multi, int nm, float* ws,
                                hipStream_t stream) {
  if (nm > 0) {
    int rc = launch_linear_chunk<KIND, true>(a, seg, nseg, ws, stream);
    if (rc) return rc;
    const int64_t n = (int64_t)a.D * a.V + (KIND == MLSTM ? a.D : 0);
    hipLaunchKernelGGL(linear_prefix_kernel<KIND>, dim3((unsigned)((n + 255) / 256), a.H, nm), dim3(256), 0, stream, a,
                       multi, nm, ws);
    rc = (int)hipGetLastError();
    if (rc) return rc;
  }
  return launch_linear_chunk<KIND, false>(a, seg, nseg, ws, stream);
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

// fp32 elements of a workspace slot per head
extern "C" int64_t mp_linear_slot(int D, int V) { return (int64_t)D * V + D + mp::LC_EXTRA; }

// Does the prompt form cover the shape?
extern "C" int mp_linear_chunk_ok(int D, int V, int rot) {
  return D % 16 == 0 && V % 8 == 0 && rot % 16 == 0 && D <= 256 && V <= 256;
}

// seg [4, nseg] (all of the step), multi [4, nm] (sequences cut into several segments; ws holds their slots)
extern "C" int mp_linear_chunk(int kind, const void* z, int64_t zs, const float* rope, int rot, const float* decay,
                               const float* bias, const float* norm, float* state, float* aux, const int32_t* q_seq,
                               const int32_t* q_ctx, void* out, int H, int D, int V, float cap, float eps, float qs,
                               float ks, const int32_t* seg, int nseg, const int32_t* multi, int nm, float* ws,
                               int packed_mt, hipStream_t stream) {
  using namespace mp;
  (void)hipGetLastError();
  if (nseg == 0) return 0;
  if (!mp_linear_chunk_ok(D, V, kind == MLSTM ? 0 : rot) || zs % 8 || nseg > 65535 || nm > 65535 || H > 65535) return -1;
  const LinArgs a{z, zs, rope, decay, bias, norm, state, aux, q_seq, q_ctx, out, H, D, V, rot, packed_mt, cap, eps, qs, ks};
  return kind == MLSTM ? launch_linear_prompt<MLSTM>(a, seg, nseg, multi, nm, ws, stream)
                       : launch_linear_prompt<RETENTION>(a, seg, nseg, multi, nm, ws, stream);
}
