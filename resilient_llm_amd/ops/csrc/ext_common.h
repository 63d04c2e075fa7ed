// Checks shared by the torch bindings of the mixed-layer kernels: every
// shape, dtype and index-table assumption of a kernel is checked before it
// is launched.
#pragma once

#include <torch/library.h>
#include <ATen/ATen.h>
#include <ATen/hip/impl/HIPStreamMasqueradingAsCUDA.h>
#include <ATen/hip/impl/HIPGuardImplMasqueradingAsCUDA.h>
#include <c10/hip/HIPGraphsC10Utils.h>

#include <algorithm>
#include <optional>

namespace rlli_ext {

using at::Tensor;
using OptTensor = std::optional<Tensor>;

inline hipStream_t stream_of(const Tensor& t) {
  return at::hip::getCurrentHIPStreamMasqueradingAsCUDA(
      t.device().index()).stream();
}

inline void check_launch(const char* op) {
  if (c10::hip::currentStreamCaptureStatusMayInitCtx() !=
      c10::hip::CaptureStatus::None)
    return;
  hipError_t e = hipGetLastError();
  TORCH_CHECK(e == hipSuccess, op, " launch failed: ", hipGetErrorString(e));
}

inline bool act_f32(const Tensor& t, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.is_contiguous(), name,
              " must be contiguous and on the GPU");
  const bool f32 = t.scalar_type() == at::kFloat;
  TORCH_CHECK(f32 || t.scalar_type() == at::kBFloat16, name,
              " must be bf16 or f32");
  return f32;
}

inline void same_act(const Tensor& t, const Tensor& like, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.is_contiguous() &&
              t.scalar_type() == like.scalar_type(), name,
              " must be contiguous, on the GPU and of the activation dtype");
}

inline const float* f32_vec(const Tensor& t, int64_t n, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.is_contiguous() &&
              t.scalar_type() == at::kFloat && t.numel() == n, name,
              " must be ", n, " contiguous f32 values on the GPU, got ",
              t.numel());
  return t.data_ptr<float>();
}

inline const int32_t* i32(const Tensor& t, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.is_contiguous() &&
              t.scalar_type() == at::kInt, name,
              " must be contiguous int32 on the GPU");
  return t.data_ptr<int32_t>();
}

// rows of ``t`` may lie further apart than their width (a column range of
// a wider matrix); columns are neighbours
inline int64_t row_stride(const Tensor& t, const Tensor& like, int64_t rows,
                          int64_t cols, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.dim() == 2 && t.size(0) == rows &&
              t.size(1) == cols && t.scalar_type() == like.scalar_type() &&
              (cols <= 1 || t.stride(1) == 1) &&
              (rows <= 1 || t.stride(0) >= cols), name, " must be [", rows,
              ", ", cols, "] of the activation dtype with unit columns");
  const int64_t s = rows > 1 ? t.stride(0) : std::max<int64_t>(cols, t.stride(0));
  TORCH_CHECK(s < (int64_t(1) << 31), name, " rows lie too far apart");
  return s;
}

}  // namespace rlli_ext
