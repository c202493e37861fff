// Torch bindings of retention.
#include "ext_common.h"

#include <cmath>

extern "C" {
void launch_retention_scan(const void*, int, int, int, int, int, float, float,
                           const float*, const float*, int, float*, void*,
                           const int*, const int*, const int*, const int*,
                           int, int, bool, hipStream_t);
void launch_retention_wide(const void*, int, int, int, int, int, float, float,
                           const float*, const float*, int, float*, void*,
                           const int*, const int*, const int*, const int*,
                           int, bool, hipStream_t);
void launch_retention_chunks(const void*, int, int, int, int, int, float,
                             float, const float*, const float*, int, float*,
                             void*, const int*, const int*, const int*,
                             const int*, const int*, int, const int*, int,
                             bool, float*, hipStream_t);
}

// sizes of which a workgroup holds the state
static bool held(int64_t d) { return d == 64 || d == 128 || d == 256; }

// Segments with state slots; those of more than max_rows rows are described
// by longs [L, 2] (segment, first piece) and pieces [P, 5], where there are
// any (bf16 only), and run in chunks.
torch::Tensor retention(torch::Tensor ab, int64_t H, int64_t dp, int64_t vp,
                        int64_t dim, int64_t vdim, torch::Tensor decay,
                        torch::Tensor table, double eps, torch::Tensor state,
                        torch::Tensor row0, torch::Tensor rows,
                        torch::Tensor slot, torch::Tensor ctx,
                        c10::optional<torch::Tensor> longs,
                        c10::optional<torch::Tensor> pieces, bool several,
                        int64_t max_rows) {
  CHECK_T(ab);
  const int M = ab.size(0), ld = row_stride(ab);
  CHECK_FLOATS(decay); CHECK_FLOATS(table); CHECK_FLOATS(state);
  CHECK_INTS(row0); CHECK_INTS(rows); CHECK_INTS(slot); CHECK_INTS(ctx);
  const int nseg = row0.numel();
  TORCH_CHECK(rows.numel() == nseg && slot.numel() == nseg &&
                  ctx.numel() == M,
              "segments and rows");
  TORCH_CHECK(H > 0 && dp % 64 == 0 && vp % 64 == 0 && dp <= 4096 &&
                  vp <= 4096 && dim > 0 && dim <= dp && vdim > 0 &&
                  vdim <= vp,
              "heads of up to 4096 numbers, padded to multiples of 64");
  TORCH_CHECK(ab.size(1) >= 2 * H * (dp + vp) && ld % 8 == 0 &&
                  (uintptr_t)ab.data_ptr() % 16 == 0,
              "projection columns");
  TORCH_CHECK(decay.numel() == 2 * H, "decays of the heads");
  TORCH_CHECK(table.dim() == 3 && table.size(0) == M && table.size(1) > 0 &&
                  2 * table.size(1) <= dim && table.size(2) == 2,
              "rotation table");
  TORCH_CHECK(state.dim() == 4 && state.size(1) == H && state.size(2) == vp &&
                  state.size(3) == dp,
              "state");
  auto y = torch::empty({M, H * vp}, ab.options());
  if (M == 0 || nseg == 0) return y;
  const float kscale = (float)(1.0 / std::sqrt((double)dim));
  if (!held(dp) || !held(vp)) {
    launch_retention_wide(
        ab.data_ptr(), ld, (int)H, (int)dp, (int)vp, (int)vdim, kscale,
        (float)eps, decay.data_ptr<float>(), table.data_ptr<float>(),
        table.size(1), state.data_ptr<float>(), y.data_ptr(),
        row0.data_ptr<int>(), rows.data_ptr<int>(), slot.data_ptr<int>(),
        ctx.data_ptr<int>(), nseg, is_f32(ab), cur_stream());
    return y;
  }
  const bool chunks = pieces.has_value() && !is_f32(ab);
  launch_retention_scan(
      ab.data_ptr(), ld, (int)H, (int)dp, (int)vp, (int)vdim, kscale,
      (float)eps, decay.data_ptr<float>(), table.data_ptr<float>(),
      table.size(1), state.data_ptr<float>(), y.data_ptr(),
      row0.data_ptr<int>(), rows.data_ptr<int>(), slot.data_ptr<int>(),
      ctx.data_ptr<int>(), nseg, chunks ? (int)max_rows : 1 << 30, is_f32(ab),
      cur_stream());
  if (!chunks) return y;
  CHECK_INTS(longs.value()); CHECK_INTS(pieces.value());
  TORCH_CHECK(longs->dim() == 2 && longs->size(1) == 2 && pieces->dim() == 2 &&
                  pieces->size(1) == 5,
              "long segments and their pieces");
  const int npieces = pieces->size(0), nlong = longs->size(0);
  torch::Tensor between;
  if (several)
    between = torch::empty({npieces, H, vp, dp}, state.options());
  launch_retention_chunks(
      ab.data_ptr(), ld, (int)H, (int)dp, (int)vp, (int)vdim, kscale,
      (float)eps, decay.data_ptr<float>(), table.data_ptr<float>(),
      table.size(1), state.data_ptr<float>(), y.data_ptr(),
      row0.data_ptr<int>(), rows.data_ptr<int>(), slot.data_ptr<int>(),
      ctx.data_ptr<int>(), longs->data_ptr<int>(), nlong,
      pieces->data_ptr<int>(), npieces, several,
      several ? between.data_ptr<float>() : nullptr, cur_stream());
  return y;
}

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) { m.def("retention", &retention); }
