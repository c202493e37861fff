// Torch bindings of the matrix products, the hand-written MFMA GEMMs and
// hipBLASLt with a fused epilogue, and of gated units. Every model family needs these, so
// they form an extension of their own.
#include "ext_common.h"
#include "gelu_rows.h"

extern "C" {
void launch_gemm_bf16(const void*, const void*, const void*, void*, int, int,
                      int, int, hipStream_t);
void launch_gemm8_bf16(const void*, const void*, const void*, void*, int, int,
                       int, int, hipStream_t);
void launch_gemm16_bf16(const void*, const void*, const void*, void*, int,
                        int, int, int, hipStream_t);
void launch_decode_gemm(const void*, const void*, const void*, void*, void*,
                        int, int, int, int, int, float, float, float,
                        const float*, const RowsArgs*, hipStream_t);
void launch_clamped_glu(const void*, void*, long, int, float, float, float,
                        bool, hipStream_t);
void launch_relu2(const void*, void*, long, bool, hipStream_t);
void launch_gelu_rows(const void*, void*, long, int, const RowsArgs*, bool,
                      hipStream_t);
}

// ---- GEMM ------------------------------------------------------------------
torch::Tensor gemm_bf16(torch::Tensor A, torch::Tensor B,
                        c10::optional<torch::Tensor> bias, int64_t act) {
  CHECK_DEV(A); CHECK_CONT(A); CHECK_BF16(A);
  CHECK_DEV(B); CHECK_CONT(B); CHECK_BF16(B);
  const int M = A.size(0), K = A.size(1), N = B.size(0);
  TORCH_CHECK(B.size(1) == K, "K mismatch");
  TORCH_CHECK(M % 128 == 0 && N % 128 == 0 && K % 64 == 0,
              "gemm_bf16 requires M,N % 128 == 0 and K % 64 == 0");
  auto C = torch::empty({M, N}, A.options());
  launch_gemm_bf16(A.data_ptr(), B.data_ptr(),
                   bias ? bias->data_ptr() : nullptr, C.data_ptr(), M, N, K,
                   (int)act, cur_stream());
  return C;
}

torch::Tensor gemm8_bf16(torch::Tensor A, torch::Tensor B,
                         c10::optional<torch::Tensor> bias, int64_t act) {
  CHECK_DEV(A); CHECK_CONT(A); CHECK_BF16(A);
  CHECK_DEV(B); CHECK_CONT(B); CHECK_BF16(B);
  const int M = A.size(0), K = A.size(1), N = B.size(0);
  TORCH_CHECK(B.size(1) == K, "K mismatch");
  TORCH_CHECK(M % 256 == 0 && N % 256 == 0 && K % 64 == 0,
              "gemm8 requires M,N % 256 == 0 and K % 64 == 0");
  auto C = torch::empty({M, N}, A.options());
  launch_gemm8_bf16(A.data_ptr(), B.data_ptr(),
                    bias ? bias->data_ptr() : nullptr, C.data_ptr(), M, N, K,
                    (int)act, cur_stream());
  return C;
}

torch::Tensor gemm16_bf16(torch::Tensor A, torch::Tensor B,
                          c10::optional<torch::Tensor> bias, int64_t act) {
  CHECK_DEV(A); CHECK_CONT(A); CHECK_BF16(A);
  CHECK_DEV(B); CHECK_CONT(B); CHECK_BF16(B);
  const int M = A.size(0), K = A.size(1), N = B.size(0);
  TORCH_CHECK(B.size(1) == K, "K mismatch");
  TORCH_CHECK(M % 256 == 0 && N % 256 == 0 && K % 128 == 0,
              "gemm16 requires M,N % 256 == 0 and K % 128 == 0");
  auto C = torch::empty({M, N}, A.options());
  launch_gemm16_bf16(A.data_ptr(), B.data_ptr(),
                     bias ? bias->data_ptr() : nullptr, C.data_ptr(), M, N,
                     K, (int)act, cur_stream());
  return C;
}

static torch::Tensor decode_gemm_act(torch::Tensor X, torch::Tensor W,
                                     c10::optional<torch::Tensor> bias,
                                     int64_t splitk, int64_t act,
                                     double limit, double alpha,
                                     double shift,
                                     c10::optional<torch::Tensor> act_nums,
                                     const RowsArgs* rows) {
  // act 1, 2 = packed gated unit in the reduce (swiglu, clamped with the
  // given constants): W is [2I, K] (gate rows then up rows), output is
  // [M, I]. act 3 = xIELU with the raw numbers act_nums [2]. act 4 = GELU
  // times a part of a table's row. act 5 = relu(.)^2. All require splitk > 1.
  CHECK_DEV(X); CHECK_CONT(X); CHECK_BF16(X);
  CHECK_DEV(W); CHECK_CONT(W); CHECK_BF16(W);
  const int M = X.size(0), K = X.size(1), N = W.size(0);
  TORCH_CHECK(W.size(1) == K, "K mismatch");
  TORCH_CHECK(M <= 256, "decode_gemm is for M <= 256");
  TORCH_CHECK(N % 64 == 0, "N % 64");
  TORCH_CHECK(K % (64 * splitk) == 0, "K % (64*splitk)");
  const bool glu = act == 1 || act == 2;
  TORCH_CHECK(act == 0 || splitk > 1, "a fused activation needs splitk > 1");
  TORCH_CHECK(!glu || N % 128 == 0, "gated-unit fusion needs N % 128 == 0");
  const float* nums = nullptr;
  if (act == 3) {
    TORCH_CHECK(act_nums.has_value() && act_nums->numel() == 2, "act_nums");
    CHECK_DEV(act_nums.value()); CHECK_F32(act_nums.value());
    nums = act_nums->data_ptr<float>();
  }
  const int MP = M <= 128 ? 128 : 256;
  auto out = torch::empty({M, glu ? N / 2 : N}, X.options());
  torch::Tensor slabs;
  void* slabp = nullptr;
  if (splitk > 1) {
    slabs = torch::empty({splitk, (long)MP, (long)N},
                         X.options().dtype(at::kFloat));
    slabp = slabs.data_ptr();
  }
  launch_decode_gemm(X.data_ptr(), W.data_ptr(),
                     bias ? bias->data_ptr() : nullptr, out.data_ptr(),
                     slabp, M, N, K, (int)splitk, (int)act, (float)limit,
                     (float)alpha, (float)shift, nums, rows, cur_stream());
  return out;
}

torch::Tensor decode_gemm(torch::Tensor X, torch::Tensor W,
                          c10::optional<torch::Tensor> bias,
                          int64_t splitk, int64_t act = 0,
                          double limit = 0.0, double alpha = 0.0,
                          double shift = 0.0,
                          c10::optional<torch::Tensor> act_nums = {}) {
  TORCH_CHECK((act >= 0 && act <= 3) || act == 5, "activation");
  return decode_gemm_act(X, W, bias, splitk, act, limit, alpha, shift,
                         act_nums, nullptr);
}

static RowsArgs rows_args(const torch::Tensor& tokens,
                          const torch::Tensor& table, long M, int64_t col0,
                          int64_t n, long N) {
  CHECK_DEV(tokens); CHECK_CONT(tokens);
  CHECK_DEV(table); CHECK_CONT(table); CHECK_T(table);
  TORCH_CHECK(tokens.scalar_type() == at::kLong && tokens.numel() == M,
              "tokens must be int64, one per row");
  TORCH_CHECK(table.dim() == 2 && n > 0 && n <= N && col0 >= 0 &&
                  col0 + n <= table.size(1),
              "table columns");
  return {(const long*)tokens.data_ptr<int64_t>(), table.data_ptr(),
          (long)table.size(1), (int)col0, (int)n};
}

// gelu(X W^T) * table[token, col0 : col0 + n], zeros in the other columns
torch::Tensor decode_gemm_rows(torch::Tensor X, torch::Tensor W,
                               int64_t splitk, torch::Tensor tokens,
                               torch::Tensor table, int64_t col0, int64_t n) {
  CHECK_SAME(X, table);
  const RowsArgs r =
      rows_args(tokens, table, X.size(0), col0, n, W.size(0));
  return decode_gemm_act(X, W, {}, splitk, 4, 0., 0., 0., {}, &r);
}

torch::Tensor gelu_rows(torch::Tensor z, torch::Tensor tokens,
                        torch::Tensor table, int64_t col0, int64_t n) {
  CHECK_DEV(z); CHECK_CONT(z); CHECK_T(z); CHECK_SAME(z, table);
  TORCH_CHECK(z.dim() == 2 && z.size(1) % 8 == 0, "columns % 8");
  const long M = z.size(0);
  const int N = z.size(1);
  const RowsArgs r = rows_args(tokens, table, M, col0, n, N);
  auto out = torch::empty_like(z);
  if (M > 0)
    launch_gelu_rows(z.data_ptr(), out.data_ptr(), M, N, &r, is_f32(z),
                     cur_stream());
  return out;
}

torch::Tensor clamped_glu(torch::Tensor gu, double limit, double alpha,
                          double shift) {
  CHECK_DEV(gu); CHECK_CONT(gu); CHECK_T(gu);
  const long R = gu.size(0);
  const int F = gu.size(1) / 2;
  TORCH_CHECK(gu.dim() == 2 && F % 8 == 0, "halves must be % 8");
  auto out = torch::empty({R, F}, gu.options());
  if (R > 0)
    launch_clamped_glu(gu.data_ptr(), out.data_ptr(), R, F, (float)limit,
                       (float)alpha, (float)shift, is_f32(gu), cur_stream());
  return out;
}

torch::Tensor relu2(torch::Tensor z) {
  CHECK_DEV(z); CHECK_CONT(z); CHECK_T(z);
  TORCH_CHECK(z.numel() % 8 == 0, "size % 8");
  auto out = torch::empty_like(z);
  if (z.numel() > 0)
    launch_relu2(z.data_ptr(), out.data_ptr(), z.numel(), is_f32(z),
                 cur_stream());
  return out;
}

// blt_gemm.cpp: hipBLASLt GEMM with fused bias/GELU/swish epilogue.
torch::Tensor blt_linear(torch::Tensor x, torch::Tensor w,
                         c10::optional<torch::Tensor> bias, int64_t epi);

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("blt_linear", &blt_linear,
        "hipBLASLt linear with fused bias/GELU/swish epilogue");
  m.def("gemm_bf16", &gemm_bf16);
  m.def("gemm8_bf16", &gemm8_bf16);
  m.def("gemm16_bf16", &gemm16_bf16);
  m.def("decode_gemm", &decode_gemm, py::arg("X"), py::arg("W"),
        py::arg("bias"), py::arg("splitk"), py::arg("act") = 0,
        py::arg("limit") = 0.0, py::arg("alpha") = 0.0,
        py::arg("shift") = 0.0, py::arg("act_nums") = py::none());
  m.def("decode_gemm_rows", &decode_gemm_rows);
  m.def("gelu_rows", &gelu_rows);
  m.def("clamped_glu", &clamped_glu);
  m.def("relu2", &relu2);
}
