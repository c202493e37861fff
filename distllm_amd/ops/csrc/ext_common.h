// Shared by the torch binding files: tensor checks and the current stream.
#pragma once

#include <torch/extension.h>

#include <hip/hip_runtime.h>
#include <c10/hip/HIPStream.h>

#define CHECK_DEV(x) TORCH_CHECK(x.is_cuda(), #x " must be on GPU")
#define CHECK_CONT(x) TORCH_CHECK(x.is_contiguous(), #x " must be contiguous")
#define CHECK_BF16(x) \
  TORCH_CHECK(x.scalar_type() == at::kBFloat16, #x " must be bf16")
#define CHECK_F32(x) \
  TORCH_CHECK(x.scalar_type() == at::kFloat, #x " must be f32")
#define CHECK_I32(x) TORCH_CHECK(x.scalar_type() == at::kInt, #x " must be i32")

#define CHECK_T(x)                                              \
  TORCH_CHECK(x.scalar_type() == at::kBFloat16 ||               \
                  x.scalar_type() == at::kFloat,                \
              #x " must be bf16 or f32")
#define CHECK_SAME(x, y) \
  TORCH_CHECK(x.scalar_type() == y.scalar_type(), #x " and " #y " differ")

static inline bool is_f32(const torch::Tensor& t) {
  return t.scalar_type() == at::kFloat;
}

static inline hipStream_t cur_stream() {
  return c10::hip::getCurrentHIPStream().stream();
}

#define CHECK_INTS(x)                          \
  do {                                         \
    CHECK_DEV(x); CHECK_CONT(x); CHECK_I32(x); \
  } while (0)
#define CHECK_FLOATS(x)                        \
  do {                                         \
    CHECK_DEV(x); CHECK_CONT(x); CHECK_F32(x); \
  } while (0)

// stride of the rows of a matrix whose columns are contiguous
static inline int row_stride(const torch::Tensor& t) {
  CHECK_DEV(t);
  TORCH_CHECK(t.dim() == 2 && t.stride(1) == 1, "rows must be contiguous");
  return (int)t.stride(0);
}
