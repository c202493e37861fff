// Torch bindings of attention with sinks over paged keys and values, of what
// precedes attention over pages, and of the gated delta rules.
#include "ext_attention.h"

extern "C" {
void launch_attn_prep(const void*, int, int, int, int, int, int, int,
                      const float*, const float*, float, void*, void*, void*,
                      const int*, int, int, const int*, const int*, int,
                      const float*, int, bool, hipStream_t);
void launch_sink_rows(const void*, const void*, const void*, const int*,
                      const int*, const int*, void*, long, int, int, int, int,
                      int, int, float, const float*, float, bool,
                      hipStream_t);
void launch_sink_decode(const void*, const void*, const void*, const int*,
                        const int*, const int*, void*, long, void*, void*,
                        int, int, int, int, int, int, int, float,
                        const float*, float, hipStream_t);
void launch_sink_flash(const void*, const void*, const void*, void*, long,
                       const int*, int, const int*, const int*, int, int, int,
                       int, int, float, const float*, float, hipStream_t);
void launch_delta_prep(const void*, int, const void*, int, int, int, int, int,
                       int, const float*, int, const float*, const float*,
                       float, float, float*, void*, float*, float*, void*,
                       const int*, const int*, const int*, int, int, int,
                       const int*, const int*, bool, bool, hipStream_t);
void launch_delta_scan(const float*, const void*, const float*, const float*,
                       const void*, int, const float*, float, float*, void*,
                       long, int, int, int, int, int, float, const int*,
                       const int*, const int*, int, const int*, int, bool,
                       bool, hipStream_t);
void launch_delta_chunks(const float*, const void*, const float*, const void*,
                         int, const float*, float*, void*, float*, float*,
                         float*, float*, int, int, int, int, int, int, float,
                         const int*, int, const int*, int, int, const int*,
                         const int*, const int*, const int*, const int*,
                         hipStream_t);
void launch_channel_chunks(const float*, const void*, const float*,
                           const void*, int, const float*, const float*,
                           const float*, float, float*, void*, long, float*,
                           float*, float*, float*, int, int, int, int, int,
                           int, float, const int*, int, const int*, int, int,
                           const int*, const int*, const int*, const int*,
                           const int*, hipStream_t);
}

torch::Tensor attn_prep(torch::Tensor ab, int64_t H, int64_t G, int64_t dp,
                        int64_t vp, int64_t n, torch::Tensor wq,
                        c10::optional<torch::Tensor> wk, double eps,
                        c10::optional<torch::Tensor> kpages,
                        c10::optional<torch::Tensor> vpages,
                        torch::Tensor bt, torch::Tensor row_seq,
                        torch::Tensor ctx) {
  CHECK_T(ab);
  const int M = ab.size(0), ld = row_stride(ab);
  check_rows(bt, row_seq, ctx, M);
  CHECK_FLOATS(wq);
  TORCH_CHECK(dp % 64 == 0 && vp % 64 == 0 && ld % 8 == 0 && n > 0 &&
                  n <= dp && wq.numel() == dp,
              "head sizes");
  void *kp = nullptr, *vpg = nullptr;
  int nblk = 0;
  const float* wkp = nullptr;
  long cols = H * dp;
  if (kpages) {
    TORCH_CHECK(vpages.has_value() && wk.has_value(), "keys and values");
    const Pages p = check_pages(*kpages, *vpages);
    CHECK_SAME(ab, kpages.value());
    TORCH_CHECK(p.G == G && p.DK == dp && p.DV == vp, "page sizes");
    CHECK_FLOATS(wk.value());
    TORCH_CHECK(wk->numel() == dp, "key norm size");
    kp = kpages->data_ptr();
    vpg = vpages->data_ptr();
    wkp = wk->data_ptr<float>();
    nblk = p.nblk;
    cols += G * (dp + vp);
  }
  TORCH_CHECK(ab.size(1) >= cols, "projection columns");
  TORCH_CHECK((long)M * (H + G) < (1L << 30), "too many rows");
  auto q = torch::empty({M, H, dp}, ab.options());
  if (M > 0)
    launch_attn_prep(ab.data_ptr(), ld, M, H, G, dp, vp, (int)n,
                     wq.data_ptr<float>(), wkp, (float)eps, q.data_ptr(), kp,
                     vpg, bt.data_ptr<int>(), bt.size(1), nblk,
                     row_seq.data_ptr<int>(), ctx.data_ptr<int>(),
                     (int)((H + G) * dp), nullptr, 0, is_f32(ab),
                     cur_stream());
  return q;
}

// ab: H query heads, G key heads of dp columns; keys as projected are the
// values. table [M, pairs, 2] of rotation_table.
torch::Tensor rotary_prep(torch::Tensor ab, int64_t H, int64_t G, int64_t dp,
                          int64_t n, torch::Tensor wq, torch::Tensor wk,
                          double eps, torch::Tensor table,
                          torch::Tensor kpages, torch::Tensor vpages,
                          torch::Tensor bt, torch::Tensor row_seq,
                          torch::Tensor ctx) {
  CHECK_T(ab); CHECK_SAME(ab, kpages);
  const int M = ab.size(0), ld = row_stride(ab);
  check_rows(bt, row_seq, ctx, M);
  CHECK_FLOATS(wq); CHECK_FLOATS(wk); CHECK_FLOATS(table);
  const Pages p = check_pages(kpages, vpages);
  TORCH_CHECK(dp % 64 == 0 && ld % 8 == 0 && n > 0 && n <= dp &&
                  wq.numel() == dp && wk.numel() == dp,
              "head sizes");
  TORCH_CHECK(p.G == G && p.DK == dp && p.DV == dp, "page sizes");
  TORCH_CHECK(ab.size(1) >= (H + G) * dp, "projection columns");
  TORCH_CHECK(table.dim() == 3 && table.size(0) == M && table.size(1) > 0 &&
                  2 * table.size(1) <= n && table.size(2) == 2,
              "rotation table");
  TORCH_CHECK((uintptr_t)ab.data_ptr() % 16 == 0, "alignment");
  TORCH_CHECK((long)M * (H + G) < (1L << 30), "too many rows");
  auto q = torch::empty({M, H, dp}, ab.options());
  if (M > 0)
    launch_attn_prep(ab.data_ptr(), ld, M, H, G, dp, dp, (int)n,
                     wq.data_ptr<float>(), wk.data_ptr<float>(), (float)eps,
                     q.data_ptr(), kpages.data_ptr(), vpages.data_ptr(),
                     bt.data_ptr<int>(), bt.size(1), p.nblk,
                     row_seq.data_ptr<int>(), ctx.data_ptr<int>(),
                     (int)(H * dp), table.data_ptr<float>(), table.size(1),
                     is_f32(ab), cur_stream());
  return q;
}

struct SinkArgs {
  Pages p;
  int M, H;
  long ld_out;
};

// out [M, H * DV], rows may be strided
static SinkArgs check_sink(const torch::Tensor& q, const torch::Tensor& k,
                           const torch::Tensor& v, const torch::Tensor& out,
                           const torch::Tensor& sink) {
  const Pages p = check_pages(k, v);
  CHECK_DEV(q); CHECK_CONT(q); CHECK_SAME(q, k);
  CHECK_SAME(out, k);
  CHECK_FLOATS(sink);
  TORCH_CHECK(q.dim() == 3, "rank");
  const int M = q.size(0), H = q.size(1), ld = row_stride(out);
  TORCH_CHECK(q.size(2) == p.DK && out.size(0) == M &&
                  out.size(1) == (long)H * p.DV && H % p.G == 0 &&
                  ld % 8 == 0 && (uintptr_t)out.data_ptr() % 16 == 0,
              "attention shapes");
  TORCH_CHECK(sink.numel() == H, "one sink per head");
  return {p, M, H, ld};
}

void sink_attn_rows(torch::Tensor q, torch::Tensor k, torch::Tensor v,
                    torch::Tensor out, torch::Tensor bt,
                    torch::Tensor row_seq, torch::Tensor ctx, double scale,
                    torch::Tensor sink, double out_scale, int64_t nsplit) {
  const SinkArgs a = check_sink(q, k, v, out, sink);
  check_rows(bt, row_seq, ctx, a.M);
  if (a.M == 0) return;
  const Pages& p = a.p;
  if (is_f32(q) || !mfma_size(p.DK) || !mfma_size(p.DV)) {
    TORCH_CHECK(p.DK <= 8192 && p.DV <= 4096, "head sizes");
    launch_sink_rows(q.data_ptr(), k.data_ptr(), v.data_ptr(),
                     bt.data_ptr<int>(), row_seq.data_ptr<int>(),
                     ctx.data_ptr<int>(), out.data_ptr(), a.ld_out, a.M, a.H,
                     p.G, p.DK, p.DV, bt.size(1), (float)scale,
                     sink.data_ptr<float>(), (float)out_scale, is_f32(q),
                     cur_stream());
    return;
  }
  const long NS = key_splits(nsplit, a.M, a.H, p.G, 1L << 30, bt.size(1));
  torch::Tensor pacc, pml;
  void *pa = nullptr, *pm = nullptr;
  if (NS > 1) {
    auto f32 = q.options().dtype(at::kFloat);
    pacc = torch::empty({(long)a.M * a.H * NS, p.DV}, f32);
    pml = torch::empty({(long)a.M * a.H * NS, 2}, f32);
    pa = pacc.data_ptr();
    pm = pml.data_ptr();
  }
  launch_sink_decode(q.data_ptr(), k.data_ptr(), v.data_ptr(),
                     bt.data_ptr<int>(), row_seq.data_ptr<int>(),
                     ctx.data_ptr<int>(), out.data_ptr(), a.ld_out, pa, pm,
                     a.M, a.H, p.G, p.DK, p.DV, (int)NS, bt.size(1),
                     (float)scale, sink.data_ptr<float>(), (float)out_scale,
                     cur_stream());
}

void sink_attn_prompts(torch::Tensor q, torch::Tensor k, torch::Tensor v,
                       torch::Tensor out, torch::Tensor bt,
                       torch::Tensor portions, torch::Tensor blocks,
                       double scale, torch::Tensor sink, double out_scale) {
  const SinkArgs a = check_sink(q, k, v, out, sink);
  CHECK_BF16(q);
  CHECK_INTS(bt); CHECK_INTS(portions); CHECK_INTS(blocks);
  TORCH_CHECK(bt.dim() == 2 && portions.dim() == 2 && portions.size(1) == 4 &&
                  blocks.dim() == 2 && blocks.size(1) == 2,
              "portion maps");
  TORCH_CHECK(mfma_size(a.p.DK) && mfma_size(a.p.DV),
              "head sizes must be 64, 128 or 256");
  if (blocks.size(0) == 0) return;
  launch_sink_flash(q.data_ptr(), k.data_ptr(), v.data_ptr(), out.data_ptr(),
                    a.ld_out, bt.data_ptr<int>(), bt.size(1),
                    portions.data_ptr<int>(), blocks.data_ptr<int>(),
                    blocks.size(0), a.H, a.p.G, a.p.DK, a.p.DV, (float)scale,
                    sink.data_ptr<float>(), (float)out_scale, cur_stream());
}

// longs [P, 2]: segments of more than max_rows rows and their first chunk,
// chunks [N, 2]: segment and number of every chunk of 32 rows; bf16 only
torch::Tensor gated_delta(torch::Tensor ab, int64_t H, int64_t G, int64_t dp,
                          int64_t vp, int64_t dim, int64_t vdim,
                          torch::Tensor conv_w, torch::Tensor decay,
                          torch::Tensor o_norm, double unit_eps, double eps,
                          torch::Tensor state, torch::Tensor conv,
                          torch::Tensor seg_row0, torch::Tensor seg_rows,
                          torch::Tensor seg_slot, int64_t longest,
                          torch::Tensor row_seq, torch::Tensor ctx,
                          c10::optional<torch::Tensor> longs,
                          c10::optional<torch::Tensor> chunks,
                          int64_t max_rows) {
  CHECK_DEV(ab); CHECK_CONT(ab); CHECK_T(ab);
  const int M = ab.size(0), ld = ab.size(1);
  auto size_ok = [](int64_t d) { return d == 64 || d == 128 || d == 256; };
  TORCH_CHECK(size_ok(dp) && size_ok(vp), "head sizes must be 64, 128, 256");
  TORCH_CHECK(dim > 0 && dim <= dp && vdim > 0 && vdim <= vp && G > 0 &&
                  H % G == 0,
              "head counts");
  const long C = 2 * G * dp + H * vp;
  TORCH_CHECK(ld >= C + H * vp + 2 * H && ld % 8 == 0, "projection columns");
  CHECK_FLOATS(conv_w); CHECK_FLOATS(decay); CHECK_FLOATS(o_norm);
  CHECK_FLOATS(state);
  CHECK_DEV(conv); CHECK_CONT(conv); CHECK_SAME(conv, ab);
  const int taps = conv_w.size(0);
  TORCH_CHECK(conv_w.dim() == 2 && conv_w.size(1) == C && taps >= 1,
              "convolution weights");
  TORCH_CHECK(decay.numel() == 2 * H && o_norm.numel() == vp, "weights");
  TORCH_CHECK(state.dim() == 4 && state.size(1) == H && state.size(2) == vp &&
                  state.size(3) == dp,
              "state must be [slots, heads, vdim, dim]");
  TORCH_CHECK(conv.dim() == 3 && conv.size(0) == state.size(0) &&
                  conv.size(1) == taps - 1 && conv.size(2) == C,
              "conv state must be [slots, taps - 1, channels]");
  CHECK_INTS(seg_row0); CHECK_INTS(seg_rows); CHECK_INTS(seg_slot);
  CHECK_INTS(row_seq); CHECK_INTS(ctx);
  const int S = seg_row0.numel();
  TORCH_CHECK(seg_rows.numel() == S && seg_slot.numel() == S &&
                  row_seq.numel() == M && ctx.numel() == M,
              "segments");
  auto f32 = ab.options().dtype(at::kFloat);
  auto y = torch::empty({M, H * vp}, ab.options());
  if (M == 0 || S == 0) return y;
  auto qk = torch::empty({M, 2 * G, dp}, f32);
  auto v = torch::empty({M, H * vp}, ab.options());
  auto gb = torch::empty({M, H, 2}, f32);
  const void* gate =
      (const char*)ab.data_ptr() + C * (long)ab.element_size();
  launch_delta_prep(ab.data_ptr(), ld, nullptr, 0, M, H, G, dp, vp,
                    conv_w.data_ptr<float>(), taps, decay.data_ptr<float>(),
                    decay.data_ptr<float>() + H, 1.f / sqrtf((float)dim),
                    (float)unit_eps, qk.data_ptr<float>(), v.data_ptr(),
                    gb.data_ptr<float>(), nullptr, conv.data_ptr(),
                    seg_row0.data_ptr<int>(), seg_rows.data_ptr<int>(),
                    seg_slot.data_ptr<int>(), S, (int)longest, INT_MAX,
                    row_seq.data_ptr<int>(), ctx.data_ptr<int>(), false,
                    is_f32(ab), cur_stream());
  const bool chunked = longs && !is_f32(ab) && longs->size(0) > 0;
  const int limit = chunked ? (int)max_rows : INT_MAX;
  launch_delta_scan(qk.data_ptr<float>(), v.data_ptr(), gb.data_ptr<float>(),
                    nullptr, gate, ld, o_norm.data_ptr<float>(), 1.f,
                    state.data_ptr<float>(), y.data_ptr(), H * vp, H, G, dp,
                    vp, vdim, (float)eps, seg_row0.data_ptr<int>(),
                    seg_rows.data_ptr<int>(), seg_slot.data_ptr<int>(), S,
                    ctx.data_ptr<int>(), limit, false, is_f32(ab),
                    cur_stream());
  if (chunked) {
    TORCH_CHECK(chunks.has_value(), "chunks");
    CHECK_INTS(longs.value()); CHECK_INTS(chunks.value());
    TORCH_CHECK(longs->dim() == 2 && longs->size(1) == 2 &&
                    chunks->dim() == 2 && chunks->size(1) == 2 &&
                    chunks->size(0) >= longs->size(0),
                "chunk maps");
    const int N = chunks->size(0);
    auto tp = torch::empty({2, N, H, 32 * 32}, f32);
    auto bsum = torch::empty({M, H}, f32);
    auto o = torch::empty({M, H * vp}, f32);
    launch_delta_chunks(
        qk.data_ptr<float>(), v.data_ptr(), gb.data_ptr<float>(), gate, ld,
        o_norm.data_ptr<float>(), state.data_ptr<float>(), y.data_ptr(),
        tp.data_ptr<float>(), tp.data_ptr<float>() + tp.numel() / 2,
        bsum.data_ptr<float>(), o.data_ptr<float>(), M, H, G, dp, vp, vdim,
        (float)eps, longs->data_ptr<int>(), longs->size(0),
        chunks->data_ptr<int>(), N, limit, seg_row0.data_ptr<int>(),
        seg_rows.data_ptr<int>(), seg_slot.data_ptr<int>(),
        row_seq.data_ptr<int>(), ctx.data_ptr<int>(), cur_stream());
  }
  return y;
}

// ab: queries, keys, values and b of every head; ag: decays [H * dp] and
// output gates [H * vp]; out [M, H * vp], rows may be strided. longs and
// chunks as for gated_delta.
void channel_delta(torch::Tensor ab, torch::Tensor ag, int64_t H, int64_t G,
                   int64_t dp, int64_t vp, int64_t dim, int64_t vdim,
                   torch::Tensor conv_w, torch::Tensor a_log,
                   torch::Tensor dt_bias, torch::Tensor o_norm,
                   double unit_eps, double eps, double out_scale,
                   torch::Tensor state, torch::Tensor conv,
                   torch::Tensor seg_row0, torch::Tensor seg_rows,
                   torch::Tensor seg_slot, int64_t longest,
                   torch::Tensor row_seq, torch::Tensor ctx,
                   c10::optional<torch::Tensor> longs,
                   c10::optional<torch::Tensor> chunks, int64_t max_rows,
                   torch::Tensor out) {
  CHECK_T(ab); CHECK_SAME(ag, ab); CHECK_SAME(out, ab);
  const int M = ab.size(0), ld = row_stride(ab), ld_ag = row_stride(ag);
  const int ld_y = row_stride(out);
  auto size_ok = [](int64_t d) { return d == 64 || d == 128 || d == 256; };
  TORCH_CHECK(size_ok(dp) && size_ok(vp), "head sizes must be 64, 128, 256");
  TORCH_CHECK(dim > 0 && dim <= dp && vdim > 0 && vdim <= vp && G > 0 &&
                  H % G == 0,
              "head counts");
  const long C = 2 * G * dp + H * vp;
  auto aligned = [](const torch::Tensor& t) {
    return (uintptr_t)t.data_ptr() % 16 == 0 && t.stride(0) % 8 == 0;
  };
  TORCH_CHECK(ab.size(1) >= C + H && ag.size(0) == M &&
                  ag.size(1) == H * (dp + vp) && out.size(0) == M &&
                  out.size(1) == H * vp && aligned(ab) && aligned(ag) &&
                  aligned(out),
              "projection columns");
  CHECK_FLOATS(conv_w); CHECK_FLOATS(a_log); CHECK_FLOATS(dt_bias);
  CHECK_FLOATS(o_norm); CHECK_FLOATS(state);
  CHECK_DEV(conv); CHECK_CONT(conv); CHECK_SAME(conv, ab);
  const int taps = conv_w.size(0);
  TORCH_CHECK(conv_w.dim() == 2 && conv_w.size(1) == C && taps >= 1,
              "convolution weights");
  TORCH_CHECK(a_log.numel() == H && dt_bias.numel() == H * dp &&
                  o_norm.numel() == vp,
              "weights");
  TORCH_CHECK(state.dim() == 4 && state.size(1) == H && state.size(2) == vp &&
                  state.size(3) == dp,
              "state must be [slots, heads, vdim, dim]");
  TORCH_CHECK(conv.dim() == 3 && conv.size(0) == state.size(0) &&
                  conv.size(1) == taps - 1 && conv.size(2) == C,
              "conv state must be [slots, taps - 1, channels]");
  CHECK_INTS(seg_row0); CHECK_INTS(seg_rows); CHECK_INTS(seg_slot);
  CHECK_INTS(row_seq); CHECK_INTS(ctx);
  const int S = seg_row0.numel();
  TORCH_CHECK(seg_rows.numel() == S && seg_slot.numel() == S &&
                  row_seq.numel() == M && ctx.numel() == M,
              "segments");
  if (M == 0 || S == 0) return;
  const bool chunked = longs && !is_f32(ab) && longs->size(0) > 0;
  const int limit = chunked ? (int)max_rows : INT_MAX;
  auto f32 = ab.options().dtype(at::kFloat);
  auto qk = torch::empty({M, 2 * G, dp}, f32);
  auto v = torch::empty({M, H * vp}, ab.options());
  auto beta = torch::empty({M, H}, f32);
  // decays of short segments, sums of logarithms in chunks of long ones
  auto gc = torch::empty({M, H, dp}, f32);
  const void* gate =
      (const char*)ag.data_ptr() + H * dp * (long)ag.element_size();
  launch_delta_prep(ab.data_ptr(), ld, ag.data_ptr(), ld_ag, M, H, G, dp, vp,
                    conv_w.data_ptr<float>(), taps, a_log.data_ptr<float>(),
                    dt_bias.data_ptr<float>(), 1.f / sqrtf((float)dim),
                    (float)unit_eps, qk.data_ptr<float>(), v.data_ptr(),
                    beta.data_ptr<float>(), gc.data_ptr<float>(),
                    conv.data_ptr(), seg_row0.data_ptr<int>(),
                    seg_rows.data_ptr<int>(), seg_slot.data_ptr<int>(), S,
                    (int)longest, limit, row_seq.data_ptr<int>(),
                    ctx.data_ptr<int>(), true, is_f32(ab), cur_stream());
  if (!chunked || longs->size(0) < S)
    launch_delta_scan(
        qk.data_ptr<float>(), v.data_ptr(), beta.data_ptr<float>(),
        gc.data_ptr<float>(), gate, ld_ag, o_norm.data_ptr<float>(),
        (float)out_scale, state.data_ptr<float>(), out.data_ptr(), ld_y, H, G,
        dp, vp, vdim, (float)eps, seg_row0.data_ptr<int>(),
        seg_rows.data_ptr<int>(), seg_slot.data_ptr<int>(), S,
        ctx.data_ptr<int>(), limit, true, is_f32(ab), cur_stream());
  if (!chunked) return;
  TORCH_CHECK(chunks.has_value(), "chunks");
  CHECK_INTS(longs.value()); CHECK_INTS(chunks.value());
  TORCH_CHECK(longs->dim() == 2 && longs->size(1) == 2 &&
                  chunks->dim() == 2 && chunks->size(1) == 2 &&
                  chunks->size(0) >= longs->size(0),
              "chunk maps");
  const int N = chunks->size(0);
  auto tp = torch::empty({2, N, H, 32 * 32}, f32);
  auto o = torch::empty({M, H * vp}, f32);
  launch_channel_chunks(
      qk.data_ptr<float>(), v.data_ptr(), beta.data_ptr<float>(),
      ag.data_ptr(), ld_ag, a_log.data_ptr<float>(),
      dt_bias.data_ptr<float>(), o_norm.data_ptr<float>(), (float)out_scale,
      state.data_ptr<float>(), out.data_ptr(), ld_y, tp.data_ptr<float>(),
      tp.data_ptr<float>() + tp.numel() / 2, gc.data_ptr<float>(),
      o.data_ptr<float>(), M, H, G, dp, vp, vdim, (float)eps,
      longs->data_ptr<int>(), longs->size(0), chunks->data_ptr<int>(), N,
      limit, seg_row0.data_ptr<int>(), seg_rows.data_ptr<int>(),
      seg_slot.data_ptr<int>(), row_seq.data_ptr<int>(),
      ctx.data_ptr<int>(), cur_stream());
}

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("attn_prep", &attn_prep);
  m.def("rotary_prep", &rotary_prep);
  m.def("sink_attn_rows", &sink_attn_rows);
  m.def("sink_attn_prompts", &sink_attn_prompts);
  m.def("gated_delta", &gated_delta);
  m.def("channel_delta", &channel_delta);
}
