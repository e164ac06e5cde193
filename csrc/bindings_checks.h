// Operand checks of the layer-stack bindings: shapes, dtypes and strides, before any launch.
#pragma once
#include "bindings_common.h"

namespace {

bool t_is_f32(const Tensor& t, const char* name) {
  TORCH_CHECK(t.is_cuda(), name, " must be a GPU tensor");
  TORCH_CHECK(t.scalar_type() == at::kBFloat16 || t.scalar_type() == at::kFloat, name, " must be bf16 or f32");
  return t.scalar_type() == at::kFloat;
}
void check_t(const Tensor& t, bool f32, const char* name) {
  TORCH_CHECK(t_is_f32(t, name) == f32, name, ": dtype differs from the other operands'");
}
void check_rows(const Tensor& t, int64_t rows, int64_t cols, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.dim() == 2 && t.stride(1) == 1 && t.size(0) >= rows && t.size(1) >= cols && t.stride(0) >= cols,
              name, " must be [>= ", rows, ", >= ", cols, "] with contiguous columns");
}
void check_aligned(const Tensor& t, const char* name) {
  TORCH_CHECK((reinterpret_cast<uintptr_t>(t.data_ptr()) & 15) == 0, name, " must be 16-byte aligned");
}
const int* i32p(const Tensor& t, int64_t n, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == at::kInt && t.is_contiguous() && t.numel() >= n, name, ": int32 [>= ", n, "]");
  return t.data_ptr<int>();
}
const int64_t* i64p(const Tensor& t, int64_t n, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == at::kLong && t.is_contiguous() && t.numel() >= n, name, ": int64 [>= ", n, "]");
  return t.data_ptr<int64_t>();
}
float* f32p(const Tensor& t, int64_t n, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == at::kFloat && t.is_contiguous() && t.numel() >= n, name, ": f32 [>= ", n, "]");
  return t.data_ptr<float>();
}

}  // namespace
