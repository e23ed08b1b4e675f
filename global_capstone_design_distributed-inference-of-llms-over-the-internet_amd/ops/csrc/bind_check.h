// Argument checks of the hybrid decoders' op registrations: every tensor is checked before its pointer goes to a launcher.
#pragma once
#include <ATen/ATen.h>
#include <ATen/hip/HIPContext.h>
#include <torch/library.h>

namespace {

#define MP_CHECK(cond, msg) TORCH_CHECK(cond, "mpamd: ", msg)

inline void check_launch(int rc, const char* what) {
  TORCH_CHECK(rc == 0, "mpamd: ", what, " launch failed with code ", rc);
}
inline hipStream_t cur_stream() { return at::hip::getCurrentHIPStream().stream(); }

// activation element type: 0 = bf16, 1 = fp32
inline int act_type(const at::Tensor& t, const char* name) {
  MP_CHECK(t.is_cuda(), std::string(name) + " must be on the GPU");
  MP_CHECK(t.scalar_type() == at::kBFloat16 || t.scalar_type() == at::kFloat, std::string(name) + ": bf16 or fp32");
  return t.scalar_type() == at::kFloat;
}
inline void check_act(const at::Tensor& t, int f32, const char* name) {
  MP_CHECK(act_type(t, name) == f32, std::string(name) + ": element types differ");
}
inline void check_rows(const at::Tensor& t, int64_t rows, int64_t cols, const char* name) {
  MP_CHECK(t.dim() == 2 && t.size(0) >= rows && t.size(1) == cols && t.stride(1) == 1,
           std::string(name) + ": [rows, cols] with unit inner stride");
  MP_CHECK(reinterpret_cast<uintptr_t>(t.data_ptr()) % 16 == 0, std::string(name) + " must be 16-B aligned");
}
inline const float* f32_vec(const at::Tensor& t, int64_t n, const char* name) {
  MP_CHECK(t.is_cuda() && t.scalar_type() == at::kFloat && t.is_contiguous() && t.numel() == n,
           std::string(name) + ": fp32 contiguous, wrong size");
  return t.data_ptr<float>();
}
inline const int32_t* i32_vec(const at::Tensor& t, int64_t n, const char* name) {
  MP_CHECK(t.is_cuda() && t.scalar_type() == at::kInt && t.is_contiguous() && t.numel() >= n,
           std::string(name) + ": int32 contiguous");
  return t.data_ptr<int32_t>();
}
inline const int64_t* i64_vec(const at::Tensor& t, int64_t n, const char* name) {
  MP_CHECK(t.is_cuda() && t.scalar_type() == at::kLong && t.is_contiguous() && t.numel() >= n,
           std::string(name) + ": int64 contiguous");
  return t.data_ptr<int64_t>();
}
// an activation output of n rows x K: row-major contiguous, or packed (bf16, K a multiple of 32); returns packed_mt
inline int check_out(const at::Tensor& t, int64_t n, int64_t K, int f32, int64_t packed, const char* name) {
  check_act(t, f32, name);
  MP_CHECK(t.is_contiguous() && reinterpret_cast<uintptr_t>(t.data_ptr()) % 16 == 0,
           std::string(name) + ": contiguous, 16-B aligned");
  if (!packed) {
    MP_CHECK(t.numel() >= n * K, std::string(name) + ": too small");
    return 0;
  }
  const int mt = (int)((n + 15) / 16);
  MP_CHECK(!f32 && K % 32 == 0 && t.numel() >= (int64_t)mt * 16 * K, std::string(name) + ": packed output");
  return mt;
}

}  // namespace
