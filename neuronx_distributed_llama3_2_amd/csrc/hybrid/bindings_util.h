// Argument checks shared by the binding files of this module.
#pragma once
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>
#include <hip/hip_runtime.h>

namespace nxd {
namespace bind {

using at::Tensor;
using Opt = c10::optional<Tensor>;

inline hipStream_t cur_stream() { return at::hip::getCurrentHIPStream().stream(); }
inline void check_rc(int rc, const char* what) { TORCH_CHECK(rc == 0, what, " failed with code ", rc); }

// activation tensors: bf16 or fp32, unit inner stride
inline bool act_f32(const Tensor& t, const char* n) {
  TORCH_CHECK(t.is_cuda() && t.dim() >= 2 && t.stride(-1) == 1, n, ": GPU tensor with a unit inner stride");
  TORCH_CHECK(t.scalar_type() == at::kBFloat16 || t.scalar_type() == at::kFloat, n, ": bf16 or fp32");
  return t.scalar_type() == at::kFloat;
}
inline void same_act(const Tensor& t, const Tensor& like, const char* n) {
  act_f32(t, n);
  TORCH_CHECK(t.scalar_type() == like.scalar_type(), n, ": activation type differs");
}
inline float* f32_ptr(const Tensor& t, int64_t numel, const char* n) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == at::kFloat && t.is_contiguous() && t.numel() == numel, n,
              ": contiguous fp32 of ", numel, " elements");
  return t.data_ptr<float>();
}
inline float* f32_opt(const Opt& t, int64_t numel, const char* n) { return t.has_value() ? f32_ptr(*t, numel, n) : nullptr; }
inline const int* i32_opt(const Opt& t, int64_t numel, const char* n) {
  if (!t.has_value()) return nullptr;
  TORCH_CHECK(t->is_cuda() && t->scalar_type() == at::kInt && t->is_contiguous() && t->numel() == numel, n,
              ": contiguous int32 of ", numel, " elements");
  return t->data_ptr<int>();
}
// first position of every sequence: int64 [B] or [B, T'] (column 0)
inline const int64_t* pos_ptr(const Tensor& t, int64_t B, int64_t* stride) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == at::kLong && t.dim() >= 1 && t.dim() <= 2 && t.size(0) == B,
              "positions: int64 [B] or [B, T]");
  *stride = B > 1 ? t.stride(0) : 0;
  return t.data_ptr<int64_t>();
}
inline void check_align(const Tensor& t, const char* n) {
  TORCH_CHECK(reinterpret_cast<uintptr_t>(t.data_ptr()) % 16 == 0, n, ": 16-byte alignment");
}

}  // namespace bind
}  // namespace nxd
