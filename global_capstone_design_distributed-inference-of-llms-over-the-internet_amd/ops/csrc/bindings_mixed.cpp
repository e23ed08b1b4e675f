// torch custom-op registrations (namespace `mpamd`) of the kernels of decoders with head-mixing attention and routed
// experts.  Same rules as bindings.cpp: outputs come from the caller, launches go to the current stream, shapes and
// dtypes are checked here.
#include "bind_check.h"

extern "C" {
int mp_mixed_prep(const void* z, int64_t zs, const float* qg, const float* kg, void* qn, void* cache,
                  const int64_t* slots, const int32_t* q_ctx, const float* rope, int rot, const float* vrope, void* out,
                  int64_t os, int packed_mt, int kind, int F, int block, int col, int out_col, float limit, int n, int H,
                  int G, int D, int V, int page_log2, float eps, int f32, hipStream_t stream);
int mp_ffn_act(const void* z, int64_t zs, void* out, int64_t os, int packed_mt, int kind, int F, int block, float limit,
               int n, int f32, hipStream_t stream);
int mp_mixed_any(const void* z, int64_t zs, const void* qn, const float* talk, const void* cache, const int32_t* bt,
                 int bt_stride, const int32_t* q_seq, const int32_t* q_ctx, const float* vrope, void* out, int64_t os,
                 int packed_mt, int n, int H, int G, int D, int V, int page_log2, float scale, float cap, int f32,
                 hipStream_t stream);
int mp_mixed_mfma_ok(int H, int G, int D, int V, int page_log2, float cap);
int mp_mixed_prompt(const void* z, int64_t zs, const void* qn, const float* talk, const void* cache, const int32_t* bt,
                    int bt_stride, const int32_t* q_seq, const int32_t* q_ctx, const float* vrope, void* out, int64_t os,
                    int packed_mt, int n, int H, int G, int D, int V, int page_log2, float scale, float cap,
                    const int32_t* blk, int nblk, int PS, int NP, int SPS, int SNP, float* sums, float* part, hipStream_t stream);
int mp_mixed_decode(const void* z, int64_t zs, const void* qn, const float* talk, const void* cache, const int32_t* bt,
                    int bt_stride, const int32_t* q_seq, const int32_t* q_ctx, const float* vrope, void* out, int64_t os,
                    int packed_mt, int n, int H, int G, int D, int V, int page_log2, float scale, float cap, int PS, int NP,
                    float* sums, float* part, hipStream_t stream);
int64_t mp_moe_lists(int E);
int mp_moe_router_splits(int T, int W, int E, int f32);
int mp_moe_route(const void* x, int64_t xs, int mt, const void* w, const int32_t* ctx, float* part, int S, float* ew,
                 int32_t* idx, int32_t* slot, int32_t* lists, int32_t* tok, int T, int E, int W, int top, int groups,
                 int keep, float scale, int f32, hipStream_t stream);
int mp_moe_gemm(int form, int glu, const void* x, int64_t xs, int mt, const int32_t* tok, const int32_t* lists,
                const void* w, void* out, int out_f32, int rows, int E, int N, int K, int block, float limit, int f32,
                hipStream_t stream);
}

namespace {

typedef c10::optional<at::Tensor> opt_tensor;

int log2_page(const at::Tensor& cache) {
  const int64_t page = cache.size(2);
  MP_CHECK(page >= 1 && (page & (page - 1)) == 0, "page size must be a power of two");
  int l = 0;
  while ((1ll << l) < page) ++l;
  return l;
}

const float* angle_table(const at::Tensor& t, const char* name) {
  MP_CHECK(t.is_cuda() && t.dim() == 2 && t.scalar_type() == at::kFloat && t.is_contiguous() && t.size(1) % 2 == 0,
           std::string(name) + ": fp32 [positions, even]");
  return t.data_ptr<float>();
}

struct MixShape {
  int f32, pl2;
  int64_t T, H, G, D, V;
};
// the cache's and the value table's sizes against the projected rows
MixShape check_mixed(const at::Tensor& z, const at::Tensor& cache, const at::Tensor& vrope, int64_t H) {
  MixShape s{};
  s.f32 = act_type(z, "z");
  check_act(cache, s.f32, "cache");
  MP_CHECK(cache.dim() == 4 && cache.is_contiguous(), "cache [pages, G, page, D + V]");
  MP_CHECK(reinterpret_cast<uintptr_t>(cache.data_ptr()) % 16 == 0, "cache must be 16-B aligned");
  s.pl2 = log2_page(cache);
  s.T = z.size(0), s.H = H, s.G = cache.size(1), s.V = vrope.size(1), s.D = cache.size(3) - s.V;
  angle_table(vrope, "vrope");
  MP_CHECK(s.D >= 1 && s.V >= 2 && s.H >= 1 && s.H % s.G == 0, "head sizes");
  MP_CHECK(z.dim() == 2 && z.size(1) >= s.H * (s.D + 1) + s.G * (s.D + s.V), "z columns");
  check_rows(z, s.T, z.size(1), "z");
  return s;
}

void check_ff(const at::Tensor& z, int64_t kind, int64_t F, int64_t block, int64_t col) {
  MP_CHECK(kind >= 0 && kind <= 3, "feed-forward kind");
  if (!kind) return;
  MP_CHECK(F >= 1 && col >= 0 && z.size(1) >= col + (kind == 1 ? F : 2 * F) + (kind == 3 ? 1 : 0), "feed-forward columns");
  MP_CHECK(kind == 1 || (block >= 1 && F % block == 0), "gate / up blocks must divide the feed-forward width");
}

// out [T, K]: attention writes columns [0, H V), the feed-forward of this row its F columns after them
void mixed_prep(const at::Tensor& z, const at::Tensor& qg, const at::Tensor& kg, at::Tensor& qn, at::Tensor& cache,
                const at::Tensor& slots, const at::Tensor& q_ctx, const at::Tensor& rope, const at::Tensor& vrope,
                at::Tensor& out, int64_t K, int64_t kind, int64_t F, int64_t block, int64_t col, double limit,
                double eps, int64_t packed) {
  const int64_t V = vrope.size(1), D = cache.size(3) - V;
  MP_CHECK(D >= 1 && qn.dim() == 2 && qn.size(1) % D == 0, "qn [T, H D]");
  const MixShape s = check_mixed(z, cache, vrope, qn.size(1) / D);
  angle_table(rope, "rope");
  MP_CHECK(rope.size(1) <= s.D && rope.size(0) == vrope.size(0), "rope: at most D columns, as many positions as vrope");
  check_act(qn, s.f32, "qn");
  check_rows(qn, s.T, s.H * s.D, "qn");
  MP_CHECK(qn.is_contiguous(), "qn contiguous");
  check_ff(z, kind, F, block, col);
  MP_CHECK(K >= s.H * s.V + (kind ? F : 0), "out columns");
  const int mt = check_out(out, s.T, K, s.f32, packed, "out");
  check_launch(mp_mixed_prep(z.data_ptr(), z.stride(0), f32_vec(qg, s.D, "q gain"), f32_vec(kg, s.D, "k gain"),
                             qn.data_ptr(), cache.data_ptr(), i64_vec(slots, s.T, "slots"), i32_vec(q_ctx, s.T, "q_ctx"),
                             rope.data_ptr<float>(), rope.size(1), vrope.data_ptr<float>(), out.data_ptr(), K, mt, kind,
                             F, block, col, s.H * s.V, (float)limit, s.T, s.H, s.G, s.D, s.V, s.pl2, (float)eps, s.f32,
                             cur_stream()),
               "mixed_prep");
}

void ffn_act(const at::Tensor& z, at::Tensor& out, int64_t kind, int64_t F, int64_t block, double limit, int64_t packed) {
  const int f32 = act_type(z, "z");
  MP_CHECK(z.dim() == 2 && kind > 0, "z [T, cols]");
  check_rows(z, z.size(0), z.size(1), "z");
  check_ff(z, kind, F, block, 0);
  const int mt = check_out(out, z.size(0), F, f32, packed, "out");
  check_launch(mp_ffn_act(z.data_ptr(), z.stride(0), out.data_ptr(), F, mt, kind, F, block, (float)limit, z.size(0), f32,
                          cur_stream()),
               "ffn_act");
}

int64_t mixed_mfma_ok(int64_t H, int64_t G, int64_t D, int64_t V, int64_t page, double cap) {
  int l = 0;
  while ((1ll << l) < page) ++l;
  return (1ll << l) == page ? mp_mixed_mfma_ok((int)H, (int)G, (int)D, (int)V, l, (float)cap) : 0;
}

// form 0: any shape; 1: prompts, blk [2, nblk] (first token, tokens <= 16); 2: decode.  The keys in ``parts`` splits of
// ``part_size`` (a prompt's denominators in ``sum_parts`` of ``sum_size``); sums fp32 [parts (sum_parts) T H], part fp32 [parts T H V] (prompts, parts > 1) or [parts T G H V] (decode)
void mixed_attention(const at::Tensor& z, const at::Tensor& qn, const at::Tensor& talk, const at::Tensor& cache,
                     const at::Tensor& bt, const at::Tensor& q_seq, const at::Tensor& q_ctx, const at::Tensor& vrope,
                     at::Tensor& out, int64_t K, double scale, double cap, int64_t packed, int64_t form,
                     const opt_tensor& blk, int64_t part_size, int64_t parts, const opt_tensor& sums,
                     const opt_tensor& part, int64_t sum_size, int64_t sum_parts) {
  MP_CHECK(talk.dim() == 2 && talk.size(0) == talk.size(1), "talk [H, H]");
  const MixShape s = check_mixed(z, cache, vrope, talk.size(0));
  check_act(qn, s.f32, "qn");
  check_rows(qn, s.T, s.H * s.D, "qn");
  MP_CHECK(qn.is_contiguous(), "qn contiguous");
  MP_CHECK(bt.is_cuda() && bt.dim() == 2 && bt.scalar_type() == at::kInt && bt.stride(1) == 1, "block table int32");
  MP_CHECK(K >= s.H * s.V, "out columns");
  const int mt = check_out(out, s.T, K, s.f32, packed, "out");
  if (form) {
    MP_CHECK(!s.f32 && parts >= 1, "the MFMA forms are bf16");
    MP_CHECK(K % 2 == 0, "out columns");
    auto ws = [&](const opt_tensor& t, int64_t n, const char* name) {
      MP_CHECK(t.has_value() && t->is_cuda() && t->scalar_type() == at::kFloat && t->is_contiguous() && t->numel() >= n &&
                   reinterpret_cast<uintptr_t>(t->data_ptr()) % 16 == 0, std::string(name) + ": fp32 scratch");
      return t->data_ptr<float>();
    };
    float* sp = ws(sums, (form == 2 ? parts : sum_parts) * s.T * s.H, "sums");
    if (form == 2) {
      check_launch(mp_mixed_decode(z.data_ptr(), z.stride(0), qn.data_ptr(), f32_vec(talk, s.H * s.H, "talk"),
                                   cache.data_ptr(), bt.data_ptr<int32_t>(), bt.stride(0), i32_vec(q_seq, s.T, "q_seq"),
                                   i32_vec(q_ctx, s.T, "q_ctx"), vrope.data_ptr<float>(), out.data_ptr(), K, mt, s.T, s.H,
                                   s.G, s.D, s.V, s.pl2, (float)scale, (float)cap, part_size, parts, sp,
                                   ws(part, parts * s.T * s.G * s.H * s.V, "part"), cur_stream()),
                   "mixed_decode");
      return;
    }
    MP_CHECK(blk.has_value() && blk->dim() == 2 && blk->size(0) == 2, "blk int32 [2, nblk]");
    const int64_t nb = blk->size(1);
    check_launch(mp_mixed_prompt(z.data_ptr(), z.stride(0), qn.data_ptr(), f32_vec(talk, s.H * s.H, "talk"), cache.data_ptr(),
                                 bt.data_ptr<int32_t>(), bt.stride(0), i32_vec(q_seq, s.T, "q_seq"),
                                 i32_vec(q_ctx, s.T, "q_ctx"), vrope.data_ptr<float>(), out.data_ptr(), K, mt, s.T, s.H, s.G,
                                 s.D, s.V, s.pl2, (float)scale, (float)cap, i32_vec(*blk, 2 * nb, "blk"), nb, part_size,
                                 parts, sum_size, sum_parts, sp, parts > 1 ? ws(part, parts * s.T * s.H * s.V, "part") : nullptr, cur_stream()),
                 "mixed_prompt");
    return;
  }
  check_launch(mp_mixed_any(z.data_ptr(), z.stride(0), qn.data_ptr(), f32_vec(talk, s.H * s.H, "talk"), cache.data_ptr(),
                            bt.data_ptr<int32_t>(), bt.stride(0), i32_vec(q_seq, s.T, "q_seq"),
                            i32_vec(q_ctx, s.T, "q_ctx"), vrope.data_ptr<float>(), out.data_ptr(), K, mt, s.T, s.H, s.G,
                            s.D, s.V, s.pl2, (float)scale, (float)cap, s.f32, cur_stream()),
               "mixed_attention");
}

int64_t moe_lists(int64_t E) { return mp_moe_lists((int)E); }
int64_t moe_router_splits(int64_t T, int64_t W, int64_t E, bool f32) {
  return mp_moe_router_splits((int)T, (int)W, (int)E, f32);
}

// rows of x: row-major [T, W], or packed with T rows
int act_rows(const at::Tensor& x, int64_t T, int64_t W, int64_t packed, int f32, int64_t& xs) {
  check_act(x, f32, "x");
  MP_CHECK(reinterpret_cast<uintptr_t>(x.data_ptr()) % 16 == 0, "x must be 16-B aligned");
  xs = W;
  if (packed) {
    const int mt = (int)((T + 15) / 16);
    MP_CHECK(!f32 && x.is_contiguous() && W % 32 == 0 && x.numel() >= (int64_t)mt * 16 * W, "x: packed");
    return mt;
  }
  check_rows(x, T, W, "x");
  xs = x.stride(0);
  return 0;
}

void moe_route(const at::Tensor& x, const at::Tensor& w, const at::Tensor& ctx, at::Tensor& part, at::Tensor& ew,
               at::Tensor& idx, at::Tensor& slot, at::Tensor& lists, at::Tensor& tok, int64_t groups, int64_t keep,
               double scale, int64_t packed) {
  const int f32 = act_type(w, "router");
  MP_CHECK(w.dim() == 2 && w.is_contiguous() && reinterpret_cast<uintptr_t>(w.data_ptr()) % 16 == 0, "router [E, W]");
  MP_CHECK(ew.dim() == 2, "ew [T, top]");
  const int64_t T = ew.size(0), top = ew.size(1), E = w.size(0), W = w.size(1);
  MP_CHECK(E >= 1 && E <= 512 && groups >= 1 && E % groups == 0 && keep >= 1 && keep <= groups && top >= 1 &&
               top <= keep * (E / groups), "experts: at most 512, in equal groups, top within the kept groups");
  int64_t xs;
  const int mt = act_rows(x, T, W, packed, f32, xs);
  MP_CHECK(part.is_cuda() && part.dim() == 3 && part.scalar_type() == at::kFloat && part.is_contiguous() &&
               part.size(1) == T && part.size(2) == E, "part fp32 [S, T, E]");
  check_launch(mp_moe_route(x.data_ptr(), xs, mt, w.data_ptr(), i32_vec(ctx, T, "ctx"), part.data_ptr<float>(),
                            part.size(0), const_cast<float*>(f32_vec(ew, T * top, "ew")),
                            const_cast<int32_t*>(i32_vec(idx, T * top, "idx")),
                            const_cast<int32_t*>(i32_vec(slot, T * top, "slot")),
                            const_cast<int32_t*>(i32_vec(lists, mp_moe_lists(E), "lists")),
                            const_cast<int32_t*>(i32_vec(tok, T * top, "tok")), T, E, W, top, groups, keep,
                            (float)scale, f32, cur_stream()),
               "moe_route");
}

// form 0: w [E, N, K]; 1, 2, 3: w in fragment order [E, N / 16, K / 32, 64, 8].  ``glu``: N gate / up rows, out [rows, N / 2]
void moe_gemm(int64_t form, const at::Tensor& x, const opt_tensor& tok, const at::Tensor& lists, const at::Tensor& w,
              at::Tensor& out, int64_t rows, int64_t tokens, int64_t glu, int64_t block, double limit, int64_t packed) {
  const int f32 = act_type(w, "w");
  MP_CHECK(w.is_contiguous() && reinterpret_cast<uintptr_t>(w.data_ptr()) % 16 == 0, "w contiguous, aligned");
  int64_t N, K;
  if (form == 0) {
    MP_CHECK(w.dim() == 3, "w [E, N, K]");
    N = w.size(1), K = w.size(2);
  } else {
    MP_CHECK(!f32 && w.dim() == 5 && w.size(3) == 64 && w.size(4) == 8, "w [E, N / 16, K / 32, 64, 8]");
    N = 16 * w.size(1), K = 32 * w.size(2);
  }
  const int64_t E = w.size(0), O = glu ? N / 2 : N;
  MP_CHECK(!glu || (N % 2 == 0 && block >= 1 && O % block == 0 && (form == 0 || block == 16)), "gate / up blocks");
  int64_t xs;
  const int mt = act_rows(x, tok.has_value() ? tokens : rows, K, packed, f32, xs);
  MP_CHECK(!packed || tok.has_value(), "sorted rows are row-major");
  MP_CHECK(out.is_cuda() && out.dim() == 2 && out.is_contiguous() && out.size(0) >= rows && out.size(1) == O, "out [rows, O]");
  const int of = act_type(out, "out");
  MP_CHECK(glu ? of == f32 : (of || !f32), "out: the activations' type (down products: or fp32)");
  check_launch(mp_moe_gemm((int)form, (int)glu, x.data_ptr(), xs, mt, tok.has_value() ? i32_vec(*tok, rows, "tok") : nullptr,
                           i32_vec(lists, mp_moe_lists(E), "lists"), w.data_ptr(), out.data_ptr(), of, rows, E, N, K,
                           block, (float)limit, f32, cur_stream()),
               "moe_gemm");
}

}  // namespace

TORCH_LIBRARY_FRAGMENT(mpamd, m) {
  m.def(
      "mixed_prep(Tensor z, Tensor qg, Tensor kg, Tensor(a!) qn, Tensor(b!) cache, Tensor slots, Tensor q_ctx, Tensor "
      "rope, Tensor vrope, Tensor(c!) out, int K, int kind, int F, int block, int col, float limit, float eps, int packed) "
      "-> ()");
  m.def("ffn_act(Tensor z, Tensor(a!) out, int kind, int F, int block, float limit, int packed) -> ()");
  m.def(
      "mixed_attention(Tensor z, Tensor qn, Tensor talk, Tensor cache, Tensor bt, Tensor q_seq, Tensor q_ctx, Tensor "
      "vrope, Tensor(a!) out, int K, float scale, float cap, int packed, int form=0, Tensor? blk=None, int part_size=0, int "
      "parts=1, Tensor(b!)? sums=None, Tensor(c!)? part=None, int sum_size=0, int sum_parts=1) -> ()");
  m.def("mixed_mfma_ok(int H, int G, int D, int V, int page, float cap) -> int", &mixed_mfma_ok);
  m.def("moe_lists(int E) -> int", &moe_lists);
  m.def("moe_router_splits(int T, int W, int E, bool f32) -> int", &moe_router_splits);
  m.def(
      "moe_route(Tensor x, Tensor w, Tensor ctx, Tensor(a!) part, Tensor(b!) ew, Tensor(c!) idx, Tensor(d!) slot, "
      "Tensor(e!) lists, Tensor(f!) tok, int groups, int keep, float scale, int packed) -> ()");
  m.def(
      "moe_gemm(int form, Tensor x, Tensor? tok, Tensor lists, Tensor w, Tensor(a!) out, int rows, int tokens, int glu, "
      "int block, float limit, int packed) -> ()");
}

TORCH_LIBRARY_IMPL(mpamd, CUDA, m) {
  m.impl("mixed_prep", &mixed_prep);
  m.impl("ffn_act", &ffn_act);
  m.impl("mixed_attention", &mixed_attention);
  m.impl("moe_route", &moe_route);
  m.impl("moe_gemm", &moe_gemm);
}
