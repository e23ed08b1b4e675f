// torch custom-op registrations (namespace `mpamd`) of the hybrid decoders' kernels: post-norm residual
// stream, HGRN2 recurrence, chunked talking-heads attention.  Same rules as bindings.cpp: outputs come
// from the caller, launches go to the current stream, shapes and dtypes are checked here.
#include "bind_check.h"

extern "C" {
int mp_embed_pos(const int64_t* ids, const void* table, int64_t vocab, const int64_t* pos, const double* inv,
                 float* res, void* xb, int T, int W, int packed_mt, int f32, hipStream_t stream);
int mp_residual_norm(const void* y, int64_t ys, const float* part, int S, int64_t slab, float* res, const float* w,
                     void* xb, const int32_t* rows, int n, int W, float eps, int packed_mt, int f32,
                     hipStream_t stream);
int mp_relu2(const void* x, int64_t xs, void* out, int64_t M, int F, int packed_mt, int f32, hipStream_t stream);
int mp_hgrn2_scan(const void* z, int64_t zs, const float* bias, const float* lower, const float* norm, float* state,
                  const int32_t* q_seq, const int32_t* q_ctx, void* out, int H, int D, int V, float eps,
                  const int32_t* seg, int nseg, int n, int packed_mt, int f32, hipStream_t stream);
int mp_talk_prep(const void* z, int64_t zs, void* qn, const float* wqk, void* cache, float* rk, const int64_t* slots,
                 int n, int H, int G, int D, int page_log2, float eps, int f32, hipStream_t stream);
int mp_talk_attention(const void* z, int64_t zs, const void* qn, const float* talk, const void* cache, const float* rk,
                      const int32_t* bt, int bt_stride, const int32_t* q_seq, const int32_t* q_ctx, void* out, int n,
                      int H, int G, int D, int page_log2, int chunk, float scale, int packed_mt, int f32,
                      hipStream_t stream);
int mp_hgrn2_chunk(const void* z, int64_t zs, const float* bias, const float* lower, const float* norm, float* state,
                   const int32_t* q_seq, const int32_t* q_ctx, void* out, int H, int D, int V, float eps,
                   const int32_t* seg, int nseg, const int32_t* multi, int nm, float* ws, float* wdec, int packed_mt,
                   int f32, hipStream_t stream);
int mp_talk_block(int H, int G, int D, int form);
int mp_talk_mfma(const void* z, int64_t zs, const void* qn, const float* talk, const float* sigma, const void* cache,
                 const float* rk,
                 const int32_t* bt, int bt_stride, const int32_t* q_seq, const int32_t* q_ctx, void* out, int n, int H,
                 int G, int D, int page_log2, int chunk, float scale, const int32_t* blk, int nblk, int PS, int NP,
                 float* part, int packed_mt, int form, hipStream_t stream);
}

namespace {

void embed_pos(const at::Tensor& ids, const at::Tensor& table, const at::Tensor& pos, const at::Tensor& inv,
               at::Tensor& res, at::Tensor& xb, int64_t packed) {
  const int f32 = act_type(table, "table");
  const int64_t T = ids.numel(), W = table.size(1);
  MP_CHECK(table.dim() == 2 && table.is_contiguous(), "table [vocab, W]");
  MP_CHECK(inv.is_cuda() && inv.scalar_type() == at::kDouble && inv.numel() == (W + 1) / 2 && inv.is_contiguous(),
           "inv: fp64 [W / 2]");
  check_rows(res, T, W, "res");
  MP_CHECK(res.scalar_type() == at::kFloat && res.is_contiguous(), "res: fp32 contiguous");
  const int mt = check_out(xb, T, W, f32, packed, "xb");
  check_launch(mp_embed_pos(i64_vec(ids, T, "ids"), table.data_ptr(), table.size(0), i64_vec(pos, T, "pos"),
                            inv.data_ptr<double>(), res.data_ptr<float>(), xb.data_ptr(), T, W, mt, f32, cur_stream()),
               "embed_pos");
}

// y: [n, W] rows, or fp32 [S, n, W] slabs (``slabs``)
void residual_norm(const at::Tensor& y, at::Tensor& res, const at::Tensor& w, at::Tensor& xb, double eps,
                   int64_t packed, int64_t slabs) {
  const int f32 = act_type(xb, "xb");
  const int64_t n = res.size(0), W = res.size(1);
  check_rows(res, n, W, "res");
  MP_CHECK(res.scalar_type() == at::kFloat && res.is_contiguous(), "res: fp32 contiguous");
  const int mt = check_out(xb, n, W, f32, packed, "xb");
  const float* wp = f32_vec(w, W, "w");
  if (slabs) {
    MP_CHECK(y.is_cuda() && y.dim() == 3 && y.scalar_type() == at::kFloat && y.is_contiguous() && y.size(1) == n &&
                 y.size(2) == W, "slabs: fp32 [S, n, W]");
    check_launch(mp_residual_norm(nullptr, W, y.data_ptr<float>(), y.size(0), n * W, res.data_ptr<float>(), wp,
                                  xb.data_ptr(), nullptr, n, W, (float)eps, mt, f32, cur_stream()),
                 "residual_norm");
    return;
  }
  check_act(y, f32, "y");
  check_rows(y, n, W, "y");
  check_launch(mp_residual_norm(y.data_ptr(), y.stride(0), nullptr, 0, 0, res.data_ptr<float>(), wp, xb.data_ptr(),
                                nullptr, n, W, (float)eps, mt, f32, cur_stream()),
               "residual_norm");
}

void rows_norm(const at::Tensor& res, const at::Tensor& rows, const at::Tensor& w, at::Tensor& out, double eps,
               int64_t packed) {
  const int f32 = act_type(out, "out");
  const int64_t n = rows.numel(), W = res.size(1);
  check_rows(res, 0, W, "res");
  MP_CHECK(res.scalar_type() == at::kFloat && res.is_contiguous(), "res: fp32 contiguous");
  const int mt = check_out(out, n, W, f32, packed, "out");
  check_launch(mp_residual_norm(nullptr, W, nullptr, 0, 0, res.data_ptr<float>(), f32_vec(w, W, "w"), out.data_ptr(),
                                i32_vec(rows, n, "rows"), n, W, (float)eps, mt, f32, cur_stream()),
               "rows_norm");
}

void relu2(const at::Tensor& x, at::Tensor& out, int64_t packed) {
  const int f32 = act_type(x, "x");
  const int64_t n = x.size(0), F = x.size(1);
  check_rows(x, n, F, "x");
  const int mt = check_out(out, n, F, f32, packed, "out");
  check_launch(mp_relu2(x.data_ptr(), x.stride(0), out.data_ptr(), n, F, mt, f32, cur_stream()), "relu2");
}

struct Hgrn2Shape {
  int f32;
  int64_t T, H, D, V;
};
Hgrn2Shape check_hgrn2(const at::Tensor& z, const at::Tensor& bias, const at::Tensor& state) {
  Hgrn2Shape s;
  s.f32 = act_type(z, "z");
  MP_CHECK(state.is_cuda() && state.dim() == 4 && state.scalar_type() == at::kFloat && state.is_contiguous(),
           "state: fp32 [rows, H, D, V]");
  s.T = z.size(0), s.H = state.size(1), s.D = state.size(2), s.V = state.size(3);
  check_rows(z, s.T, s.H * (2 * s.D + s.V), "z");
  MP_CHECK(bias.numel() == s.H * s.D, "bias [H D]");
  return s;
}

void hgrn2_scan(const at::Tensor& z, const at::Tensor& bias, const at::Tensor& lower, const at::Tensor& norm,
                at::Tensor& state, const at::Tensor& q_seq, const at::Tensor& q_ctx, at::Tensor& out, double eps,
                const c10::optional<at::Tensor>& seg, int64_t packed) {
  const Hgrn2Shape s = check_hgrn2(z, bias, state);
  const int mt = check_out(out, s.T, s.H * s.V, s.f32, packed, "out");
  const int32_t* sp = nullptr;
  int64_t nseg = 0;
  if (seg.has_value()) {
    MP_CHECK(seg->dim() == 2 && seg->size(0) >= 2, "seg int32 [2+, nseg]");
    nseg = seg->size(1);
    sp = i32_vec(*seg, 2 * nseg, "seg");
  }
  check_launch(mp_hgrn2_scan(z.data_ptr(), z.stride(0), f32_vec(bias, s.H * s.D, "bias"),
                             f32_vec(lower, s.H * s.D, "lower"), f32_vec(norm, s.V, "norm"), state.data_ptr<float>(),
                             i32_vec(q_seq, s.T, "q_seq"), i32_vec(q_ctx, s.T, "q_ctx"), out.data_ptr(), s.H, s.D, s.V,
                             (float)eps, sp, nseg, sp ? nseg : s.T, mt, s.f32, cur_stream()),
               "hgrn2_scan");
}

// seg [4, nseg] (first token, tokens, state source, state target), multi [4, nm] (first slot, slots, first token, -):
// csrc/hgrn2.hip.  ``slots``: workspace slots the segments name.
void hgrn2_chunk(const at::Tensor& z, const at::Tensor& bias, const at::Tensor& lower, const at::Tensor& norm,
                 at::Tensor& state, const at::Tensor& q_seq, const at::Tensor& q_ctx, at::Tensor& out, double eps,
                 const at::Tensor& seg, const c10::optional<at::Tensor>& multi, int64_t slots,
                 const c10::optional<at::Tensor>& ws, int64_t packed) {
  const Hgrn2Shape s = check_hgrn2(z, bias, state);
  const int mt = check_out(out, s.T, s.H * s.V, s.f32, packed, "out");
  MP_CHECK(seg.dim() == 2 && seg.size(0) == 4, "seg int32 [4, nseg]");
  const int64_t nseg = seg.size(1);
  const int32_t* mp = nullptr;
  int64_t nm = 0;
  float *wp = nullptr, *wd = nullptr;
  if (multi.has_value() && multi->numel()) {
    MP_CHECK(multi->dim() == 2 && multi->size(0) == 4 && ws.has_value(), "multi int32 [4, nm] with a workspace");
    nm = multi->size(1);
    mp = i32_vec(*multi, 4 * nm, "multi");
    MP_CHECK(ws->is_cuda() && ws->scalar_type() == at::kFloat && ws->is_contiguous() &&
                 ws->numel() >= slots * s.H * s.D * (s.V + 1), "ws: fp32 [slots H D (V + 1)]");
    wp = ws->data_ptr<float>();
    wd = wp + slots * s.H * s.D * s.V;
  }
  check_launch(mp_hgrn2_chunk(z.data_ptr(), z.stride(0), f32_vec(bias, s.H * s.D, "bias"),
                              f32_vec(lower, s.H * s.D, "lower"), f32_vec(norm, s.V, "norm"), state.data_ptr<float>(),
                              i32_vec(q_seq, s.T, "q_seq"), i32_vec(q_ctx, s.T, "q_ctx"), out.data_ptr(), s.H, s.D,
                              s.V, (float)eps, i32_vec(seg, 4 * nseg, "seg"), nseg, mp, nm, wp, wd, mt, s.f32,
                              cur_stream()),
               "hgrn2_chunk");
}

struct TalkShape {
  int f32, page_log2;
  int64_t T, H, G, D;
};
TalkShape check_talk(const at::Tensor& z, const at::Tensor& qn, const at::Tensor& cache, const at::Tensor& rk) {
  TalkShape s;
  s.f32 = act_type(z, "z");
  check_act(qn, s.f32, "qn");
  check_act(cache, s.f32, "cache");
  MP_CHECK(cache.dim() == 4 && cache.is_contiguous(), "cache [pages, G, page, D]");
  const int64_t page = cache.size(2);
  MP_CHECK((page & (page - 1)) == 0, "page size must be a power of two");
  s.page_log2 = 0;
  while ((1ll << s.page_log2) < page) ++s.page_log2;
  MP_CHECK(rk.is_cuda() && rk.scalar_type() == at::kFloat && rk.is_contiguous() &&
               rk.numel() == cache.size(0) * page, "rk: fp32 [pages, page]");
  s.T = z.size(0), s.G = cache.size(1), s.D = cache.size(3);
  MP_CHECK(qn.dim() == 2 && qn.is_contiguous() && qn.size(0) >= s.T && qn.size(1) % s.D == 0, "qn [T, H D]");
  s.H = qn.size(1) / s.D;
  MP_CHECK(s.H % s.G == 0, "H must be a multiple of G");
  check_rows(z, s.T, (2 * s.H + s.G) * s.D, "z");
  return s;
}

void talk_prep(const at::Tensor& z, const at::Tensor& wqk, at::Tensor& qn, at::Tensor& cache, at::Tensor& rk,
               const at::Tensor& slots, double eps) {
  const TalkShape s = check_talk(z, qn, cache, rk);
  check_launch(mp_talk_prep(z.data_ptr(), z.stride(0), qn.data_ptr(), f32_vec(wqk, s.H * s.D, "wqk"), cache.data_ptr(),
                            rk.data_ptr<float>(), i64_vec(slots, s.T, "slots"), s.T, s.H, s.G, s.D, s.page_log2,
                            (float)eps, s.f32, cur_stream()),
               "talk_prep");
}

void talk_attention(const at::Tensor& z, const at::Tensor& qn, const at::Tensor& talk, const at::Tensor& cache,
                    const at::Tensor& rk, const at::Tensor& bt, const at::Tensor& q_seq, const at::Tensor& q_ctx,
                    at::Tensor& out, int64_t chunk, double scale, int64_t packed) {
  const TalkShape s = check_talk(z, qn, cache, rk);
  MP_CHECK(chunk >= 1 && chunk < (1ll << 31), "chunk");
  MP_CHECK(bt.is_cuda() && bt.dim() == 2 && bt.scalar_type() == at::kInt && bt.stride(1) == 1, "block table int32");
  const int mt = check_out(out, s.T, s.H * s.D, s.f32, packed, "out");
  check_launch(mp_talk_attention(z.data_ptr(), z.stride(0), qn.data_ptr(), f32_vec(talk, s.H * s.H, "talk"),
                                 cache.data_ptr(), rk.data_ptr<float>(), bt.data_ptr<int32_t>(), bt.stride(0),
                                 i32_vec(q_seq, s.T, "q_seq"), i32_vec(q_ctx, s.T, "q_ctx"), out.data_ptr(), s.T, s.H,
                                 s.G, s.D, s.page_log2, (int)chunk, (float)scale, mt, s.f32, cur_stream()),
               "talk_attention");
}

int64_t talk_block(int64_t H, int64_t G, int64_t D, int64_t form) {
  return mp_talk_block((int)H, (int)G, (int)D, (int)form);
}

// blk: int32 [2, nblk] query blocks of a prompt step, or none: one-token rows, the context in ``parts`` splits of
// ``part_size`` keys (``ws`` when parts > 1)
void talk_mfma(const at::Tensor& z, const at::Tensor& qn, const at::Tensor& talk, const at::Tensor& sigma,
               const at::Tensor& cache,
               const at::Tensor& rk, const at::Tensor& bt, const at::Tensor& q_seq, const at::Tensor& q_ctx,
               at::Tensor& out, int64_t chunk, double scale, const c10::optional<at::Tensor>& blk, int64_t part_size,
               int64_t parts, const c10::optional<at::Tensor>& ws, int64_t packed, int64_t form) {
  const TalkShape s = check_talk(z, qn, cache, rk);
  MP_CHECK(!s.f32, "talk_mfma is bf16");
  MP_CHECK(chunk >= 1 && chunk < (1ll << 31), "chunk");
  MP_CHECK(bt.is_cuda() && bt.dim() == 2 && bt.scalar_type() == at::kInt && bt.stride(1) == 1, "block table int32");
  const int mt = check_out(out, s.T, s.H * s.D, s.f32, packed, "out");
  const int32_t* bp = nullptr;
  int64_t nb = 0;
  if (blk.has_value()) {
    MP_CHECK(blk->dim() == 2 && blk->size(0) == 2, "blk int32 [2, nblk]");
    nb = blk->size(1);
    bp = i32_vec(*blk, 2 * nb, "blk");
    if (nb == 0) return;
  }
  float* wp = nullptr;
  if (parts > 1) {
    MP_CHECK(ws.has_value() && ws->is_cuda() && ws->scalar_type() == at::kFloat && ws->is_contiguous() &&
                 ws->numel() >= parts * s.T * s.H * (s.D + 2), "ws: fp32 [parts T H (D + 2)]");
    wp = ws->data_ptr<float>();
  }
  check_launch(mp_talk_mfma(z.data_ptr(), z.stride(0), qn.data_ptr(), f32_vec(talk, s.H * s.H, "talk"),
                            f32_vec(sigma, s.H, "sigma"),
                            cache.data_ptr(), rk.data_ptr<float>(), bt.data_ptr<int32_t>(), bt.stride(0),
                            i32_vec(q_seq, s.T, "q_seq"), i32_vec(q_ctx, s.T, "q_ctx"), out.data_ptr(), s.T, s.H, s.G,
                            s.D, s.page_log2, (int)chunk, (float)scale, bp, nb, (int)part_size, (int)parts, wp, mt,
                            (int)form, cur_stream()),
               "talk_mfma");
}

}  // namespace

TORCH_LIBRARY_FRAGMENT(mpamd, m) {
  m.def("embed_pos(Tensor ids, Tensor table, Tensor pos, Tensor inv, Tensor(a!) res, Tensor(b!) xb, int packed) -> ()");
  m.def("residual_norm(Tensor y, Tensor(a!) res, Tensor w, Tensor(b!) xb, float eps, int packed, int slabs) -> ()");
  m.def("rows_norm(Tensor res, Tensor rows, Tensor w, Tensor(a!) out, float eps, int packed) -> ()");
  m.def("relu2(Tensor x, Tensor(a!) out, int packed) -> ()");
  m.def(
      "hgrn2_scan(Tensor z, Tensor bias, Tensor lower, Tensor norm, Tensor(a!) state, Tensor q_seq, Tensor q_ctx, "
      "Tensor(b!) out, float eps, Tensor? seg, int packed) -> ()");
  m.def(
      "talk_prep(Tensor z, Tensor wqk, Tensor(a!) qn, Tensor(b!) cache, Tensor(c!) rk, Tensor slots, float eps) -> ()");
  m.def(
      "talk_attention(Tensor z, Tensor qn, Tensor talk, Tensor cache, Tensor rk, Tensor bt, Tensor q_seq, "
      "Tensor q_ctx, Tensor(a!) out, int chunk, float scale, int packed) -> ()");
  m.def(
      "hgrn2_chunk(Tensor z, Tensor bias, Tensor lower, Tensor norm, Tensor(a!) state, Tensor q_seq, Tensor q_ctx, "
      "Tensor(b!) out, float eps, Tensor seg, Tensor? multi, int slots, Tensor? ws, int packed) -> ()");
  m.def("talk_block(int H, int G, int D, int form) -> int", &talk_block);
  m.def(
      "talk_mfma(Tensor z, Tensor qn, Tensor talk, Tensor sigma, Tensor cache, Tensor rk, Tensor bt, Tensor q_seq, Tensor q_ctx, "
      "Tensor(a!) out, int chunk, float scale, Tensor? blk, int part_size, int parts, Tensor? ws, int packed, "
      "int form) -> ()");
}

TORCH_LIBRARY_IMPL(mpamd, CUDA, m) {
  m.impl("embed_pos", &embed_pos);
  m.impl("residual_norm", &residual_norm);
  m.impl("rows_norm", &rows_norm);
  m.impl("relu2", &relu2);
  m.impl("hgrn2_scan", &hgrn2_scan);
  m.impl("talk_prep", &talk_prep);
  m.impl("talk_attention", &talk_attention);
  m.impl("hgrn2_chunk", &hgrn2_chunk);
  m.impl("talk_mfma", &talk_mfma);
}
