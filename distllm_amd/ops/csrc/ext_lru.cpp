// Torch binding of the linear recurrent unit.
#include "ext_common.h"

extern "C" void launch_gated_lru(
    const void*, int, int, int, const float*, const float*, int, const void*,
    const float*, int, int, const float*, float*, void*, void*, float*,
    float*, float*, void*, const int*, const int*, const int*, int, int,
    const int*, const int*, const int*, int, const int*, int, int, bool,
    hipStream_t);

static const int LCH = 64;  // rows of a chunk (lru.hip)

// longs [P, 2]: segments of more than max_rows rows and their first chunk,
// chunks [N, 2]: segment and number of every chunk; bf16 only
torch::Tensor gated_lru(torch::Tensor ab, torch::Tensor conv_w,
                        torch::Tensor conv_b, torch::Tensor gates,
                        torch::Tensor gates_b, torch::Tensor decay,
                        torch::Tensor state, torch::Tensor conv,
                        torch::Tensor seg_row0, torch::Tensor seg_rows,
                        torch::Tensor seg_slot, int64_t longest,
                        torch::Tensor row_seq, torch::Tensor ctx,
                        c10::optional<torch::Tensor> longs,
                        c10::optional<torch::Tensor> chunks, int64_t chunk,
                        int64_t max_rows) {
  CHECK_DEV(ab); CHECK_CONT(ab); CHECK_T(ab);
  CHECK_FLOATS(conv_w); CHECK_FLOATS(conv_b); CHECK_FLOATS(gates_b);
  CHECK_FLOATS(decay); CHECK_FLOATS(state);
  CHECK_DEV(gates); CHECK_CONT(gates); CHECK_SAME(gates, ab);
  CHECK_DEV(conv); CHECK_CONT(conv); CHECK_SAME(conv, ab);
  TORCH_CHECK(ab.dim() == 2 && conv_w.dim() == 2, "ranks");
  const int M = ab.size(0), ld = ab.size(1);
  const int taps = conv_w.size(0), C = conv_w.size(1);
  TORCH_CHECK(C % 64 == 0 && ld == 2 * C && taps >= 1, "projection columns");
  TORCH_CHECK(gates.dim() == 4 && gates.size(0) == 2 &&
                  gates.size(2) == gates.size(3) && gates.size(2) % 32 == 0 &&
                  gates.size(1) * gates.size(2) <= C,
              "gates must be [2, blocks, size, size], size % 32");
  TORCH_CHECK(conv_b.numel() == C && gates_b.numel() == 2 * C &&
                  decay.numel() == C,
              "vectors");
  TORCH_CHECK(state.dim() == 2 && state.size(1) == C && conv.dim() == 3 &&
                  conv.size(0) == state.size(0) &&
                  conv.size(1) == taps - 1 && conv.size(2) == C,
              "state must be [slots, width], conv [slots, taps - 1, width]");
  CHECK_INTS(seg_row0); CHECK_INTS(seg_rows); CHECK_INTS(seg_slot);
  CHECK_INTS(row_seq); CHECK_INTS(ctx);
  const int S = seg_row0.numel();
  TORCH_CHECK(seg_rows.numel() == S && seg_slot.numel() == S &&
                  row_seq.numel() == M && ctx.numel() == M,
              "segments");
  auto out = torch::empty({M, C}, ab.options());
  if (M == 0 || S == 0) return out;
  const bool chunked = longs && !is_f32(ab) && longs->size(0) > 0;
  int P = 0, N = 0;
  const int *lp = nullptr, *cp = nullptr;
  if (chunked) {
    TORCH_CHECK(chunks.has_value() && chunk == LCH, "chunks of 64 rows");
    CHECK_INTS(longs.value()); CHECK_INTS(chunks.value());
    TORCH_CHECK(longs->dim() == 2 && longs->size(1) == 2 &&
                    chunks->dim() == 2 && chunks->size(1) == 2 &&
                    chunks->size(0) >= longs->size(0),
                "chunk maps");
    P = longs->size(0);
    N = chunks->size(0);
    lp = longs->data_ptr<int>();
    cp = chunks->data_ptr<int>();
  }
  auto f32 = ab.options().dtype(at::kFloat);
  auto u = torch::empty({M, C}, ab.options());
  auto sum = torch::empty({M, C}, f32), hs = torch::empty({M, C}, f32);
  auto start = torch::empty({N, C}, f32);
  launch_gated_lru(
      ab.data_ptr(), ld, M, C, conv_w.data_ptr<float>(),
      conv_b.data_ptr<float>(), taps, gates.data_ptr(),
      gates_b.data_ptr<float>(), gates.size(1), gates.size(2),
      decay.data_ptr<float>(), state.data_ptr<float>(), conv.data_ptr(),
      u.data_ptr(), sum.data_ptr<float>(), hs.data_ptr<float>(),
      start.data_ptr<float>(), out.data_ptr(), seg_row0.data_ptr<int>(),
      seg_rows.data_ptr<int>(), seg_slot.data_ptr<int>(), S, (int)longest,
      row_seq.data_ptr<int>(), ctx.data_ptr<int>(), lp, P, cp, N,
      chunked ? (int)max_rows : INT_MAX, is_f32(ab), cur_stream());
  return out;
}

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("gated_lru", &gated_lru);
}
