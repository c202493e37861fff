// Torch bindings of chunked attention over paged keys and values, the gated
// delta rule, xIELU and routed experts.
#include "ext_common.h"

extern "C" {
void launch_attn_prep(const void*, int, int, int, int, int, int, int,
                      const float*, const float*, float, void*, void*, void*,
                      const int*, int, int, const int*, const int*, bool,
                      hipStream_t);
void launch_chunk_rows(const void*, const void*, const void*, const void*,
                       int, const int*, const int*, const int*, void*, int,
                       int, int, int, int, int, int, float, float,
                       const float*, bool, hipStream_t);
void launch_chunk_decode(const void*, const void*, const void*, const void*,
                         int, const int*, const int*, const int*, void*,
                         void*, void*, int, int, int, int, int, int, int, int,
                         float, float, const float*, hipStream_t);
void launch_chunk_flash(const void*, const void*, const void*, const void*,
                        int, void*, const int*, int, const int*, const int*,
                        int, int, int, int, int, int, float, float,
                        const float*, hipStream_t);
void launch_delta_prep(const void*, int, int, int, int, int, int,
                       const float*, int, const float*, float, float, float*,
                       void*, float*, void*, const int*, const int*,
                       const int*, int, int, const int*, const int*, bool,
                       hipStream_t);
void launch_delta_scan(const float*, const void*, const float*, const void*,
                       int, const float*, float*, void*, int, int, int, int,
                       int, float, const int*, const int*, const int*, int,
                       const int*, int, bool, hipStream_t);
void launch_delta_chunks(const float*, const void*, const float*, const void*,
                         int, const float*, float*, void*, float*, float*,
                         float*, float*, int, int, int, int, int, int, float,
                         const int*, int, const int*, int, int, const int*,
                         const int*, const int*, const int*, const int*,
                         hipStream_t);
void launch_xielu(const void*, const float*, void*, long, bool, hipStream_t);
bool route_covers(int);
bool expert_gemm16_covers(int, int);
void launch_select(const float*, const int*, int, int, int, int, int, int*,
                   float*, hipStream_t);
void launch_route(const void*, const void*, const int*, int, int, int, int,
                  int, int, int*, float*, hipStream_t);
void launch_expert_plan(const int*, int, int, int, int, int*, int*, int*,
                        hipStream_t);
void launch_expert_gemm(const void*, const void*, void*, const int*,
                        const int*, const int*, int, int, int, int, int, bool,
                        bool, hipStream_t);
}

#define CHECK_INTS(x)                       \
  do {                                      \
    CHECK_DEV(x); CHECK_CONT(x); CHECK_I32(x); \
  } while (0)
#define CHECK_FLOATS(x)                     \
  do {                                      \
    CHECK_DEV(x); CHECK_CONT(x); CHECK_F32(x); \
  } while (0)

// rows of a matrix whose columns are contiguous
static int row_stride(const torch::Tensor& t) {
  CHECK_DEV(t);
  TORCH_CHECK(t.dim() == 2 && t.stride(1) == 1, "rows must be contiguous");
  return (int)t.stride(0);
}

struct Pages {
  int nblk, G, DK, DV;
};

static Pages check_pages(const torch::Tensor& k, const torch::Tensor& v) {
  CHECK_DEV(k); CHECK_CONT(k); CHECK_T(k);
  CHECK_DEV(v); CHECK_CONT(v); CHECK_SAME(k, v);
  TORCH_CHECK(k.dim() == 4 && v.dim() == 4 && k.size(2) == 16 &&
                  v.size(3) == 16 && k.size(0) == v.size(0) &&
                  k.size(1) == v.size(1),
              "pages must be [blocks, heads, 16, dim], [blocks, heads, "
              "vdim, 16]");
  TORCH_CHECK(k.size(3) % 64 == 0 && v.size(2) % 64 == 0,
              "head sizes % 64");
  return {(int)k.size(0), (int)k.size(1), (int)k.size(3), (int)v.size(2)};
}

static void check_rows(const torch::Tensor& bt, const torch::Tensor& row_seq,
                       const torch::Tensor& ctx, long M) {
  CHECK_INTS(bt); CHECK_INTS(row_seq); CHECK_INTS(ctx);
  TORCH_CHECK(bt.dim() == 2 && row_seq.numel() == M && ctx.numel() == M,
              "one row_seq and ctx entry per row");
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
                     is_f32(ab), cur_stream());
  return q;
}

struct AttnArgs {
  Pages p;
  int M, H, ld;
  const void* gate;
};

static AttnArgs check_attn(const torch::Tensor& q, const torch::Tensor& k,
                           const torch::Tensor& v, const torch::Tensor& ab,
                           int64_t gate_at, const torch::Tensor& out,
                           int64_t chunk, double softcap,
                           const torch::Tensor& dist) {
  const Pages p = check_pages(k, v);
  CHECK_DEV(q); CHECK_CONT(q); CHECK_SAME(q, k);
  CHECK_DEV(out); CHECK_CONT(out); CHECK_SAME(out, k);
  CHECK_SAME(ab, k);
  CHECK_FLOATS(dist);
  TORCH_CHECK(q.dim() == 3 && out.dim() == 3, "ranks");
  const int M = q.size(0), H = q.size(1), ld = row_stride(ab);
  TORCH_CHECK(q.size(2) == p.DK && out.size(0) == M && out.size(1) == H &&
                  out.size(2) == p.DV && H % p.G == 0 && ab.size(0) == M,
              "attention shapes");
  TORCH_CHECK(gate_at >= 0 && gate_at % 8 == 0 && ld % 8 == 0 &&
                  ab.size(1) >= gate_at + (long)H * p.DV,
              "gate columns");
  TORCH_CHECK(dist.numel() == 2 * H && chunk > 0 && softcap > 0, "constants");
  return {p, M, H, ld,
          (const char*)ab.data_ptr() + gate_at * ab.element_size()};
}

static bool mfma_size(int d) { return d == 64 || d == 128 || d == 256; }

void paged_attn_rows(torch::Tensor q, torch::Tensor k, torch::Tensor v,
                     torch::Tensor ab, int64_t gate_at, torch::Tensor out,
                     torch::Tensor bt, torch::Tensor row_seq,
                     torch::Tensor ctx, int64_t chunk, double scale,
                     double softcap, torch::Tensor dist, int64_t nsplit) {
  const AttnArgs a = check_attn(q, k, v, ab, gate_at, out, chunk, softcap,
                                dist);
  check_rows(bt, row_seq, ctx, a.M);
  if (a.M == 0) return;
  const int ch = (int)std::min<int64_t>(chunk, 1 << 30);
  const Pages& p = a.p;
  if (is_f32(q) || !mfma_size(p.DK) || !mfma_size(p.DV)) {
    TORCH_CHECK(p.DK <= 8192 && p.DV <= 4096, "head sizes");
    launch_chunk_rows(q.data_ptr(), k.data_ptr(), v.data_ptr(), a.gate, a.ld,
                      bt.data_ptr<int>(), row_seq.data_ptr<int>(),
                      ctx.data_ptr<int>(), out.data_ptr(), a.M, a.H, p.G,
                      p.DK, p.DV, bt.size(1), ch, (float)scale,
                      (float)softcap, dist.data_ptr<float>(), is_f32(q),
                      cur_stream());
    return;
  }
  // Split each row's keys until the CUs are full (four workgroups each), as
  // long as a wave keeps two tiles. All sizes are known on the host, so a
  // captured graph stays valid as contexts grow.
  long NS = nsplit;
  if (NS <= 0) {
    const long wgs = (long)a.M * p.G * ((a.H / p.G + 15) / 16);
    const long keys = std::min<long>(ch, bt.size(1) * 16L);
    const long tiles = keys / 32 + 1;
    NS = std::min<long>({(1024 + wgs - 1) / wgs, tiles / 8, 64L});
  }
  NS = std::max<long>(NS, 1);
  torch::Tensor pacc, pml;
  void *pa = nullptr, *pm = nullptr;
  if (NS > 1) {
    auto f32 = q.options().dtype(at::kFloat);
    pacc = torch::empty({(long)a.M * a.H * NS, p.DV}, f32);
    pml = torch::empty({(long)a.M * a.H * NS, 2}, f32);
    pa = pacc.data_ptr();
    pm = pml.data_ptr();
  }
  launch_chunk_decode(q.data_ptr(), k.data_ptr(), v.data_ptr(), a.gate, a.ld,
                      bt.data_ptr<int>(), row_seq.data_ptr<int>(),
                      ctx.data_ptr<int>(), out.data_ptr(), pa, pm, a.M, a.H,
                      p.G, p.DK, p.DV, (int)NS, bt.size(1), ch, (float)scale,
                      (float)softcap, dist.data_ptr<float>(), cur_stream());
}

// portions [P, 4]: block-table row, first row, first position, rows;
// blocks [N, 2]: portion, block of 128 queries
void paged_attn_prompts(torch::Tensor q, torch::Tensor k, torch::Tensor v,
                        torch::Tensor ab, int64_t gate_at, torch::Tensor out,
                        torch::Tensor bt, torch::Tensor portions,
                        torch::Tensor blocks, int64_t chunk, double scale,
                        double softcap, torch::Tensor dist) {
  const AttnArgs a = check_attn(q, k, v, ab, gate_at, out, chunk, softcap,
                                dist);
  CHECK_BF16(q);
  CHECK_INTS(bt); CHECK_INTS(portions); CHECK_INTS(blocks);
  TORCH_CHECK(bt.dim() == 2 && portions.dim() == 2 && portions.size(1) == 4 &&
                  blocks.dim() == 2 && blocks.size(1) == 2,
              "portion maps");
  TORCH_CHECK(mfma_size(a.p.DK) && mfma_size(a.p.DV),
              "head sizes must be 64, 128 or 256");
  if (blocks.size(0) == 0) return;
  launch_chunk_flash(q.data_ptr(), k.data_ptr(), v.data_ptr(), a.gate, a.ld,
                     out.data_ptr(), bt.data_ptr<int>(), bt.size(1),
                     portions.data_ptr<int>(), blocks.data_ptr<int>(),
                     blocks.size(0), a.H, a.p.G, a.p.DK, a.p.DV,
                     (int)std::min<int64_t>(chunk, 1 << 30), (float)scale,
                     (float)softcap, dist.data_ptr<float>(), cur_stream());
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
  launch_delta_prep(ab.data_ptr(), ld, M, H, G, dp, vp,
                    conv_w.data_ptr<float>(), taps, decay.data_ptr<float>(),
                    1.f / sqrtf((float)dim), (float)unit_eps,
                    qk.data_ptr<float>(), v.data_ptr(), gb.data_ptr<float>(),
                    conv.data_ptr(), seg_row0.data_ptr<int>(),
                    seg_rows.data_ptr<int>(), seg_slot.data_ptr<int>(), S,
                    (int)longest, row_seq.data_ptr<int>(),
                    ctx.data_ptr<int>(), is_f32(ab), cur_stream());
  const bool chunked = longs && !is_f32(ab) && longs->size(0) > 0;
  const int limit = chunked ? (int)max_rows : INT_MAX;
  launch_delta_scan(qk.data_ptr<float>(), v.data_ptr(), gb.data_ptr<float>(),
                    gate, ld, o_norm.data_ptr<float>(), state.data_ptr<float>(),
                    y.data_ptr(), H, G, dp, vp, vdim, (float)eps,
                    seg_row0.data_ptr<int>(), seg_rows.data_ptr<int>(),
                    seg_slot.data_ptr<int>(), S, ctx.data_ptr<int>(), limit,
                    is_f32(ab), cur_stream());
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

torch::Tensor xielu(torch::Tensor z, torch::Tensor act) {
  CHECK_DEV(z); CHECK_CONT(z); CHECK_T(z);
  CHECK_FLOATS(act);
  TORCH_CHECK(act.numel() == 2 && z.numel() % 8 == 0, "xielu sizes");
  auto out = torch::empty_like(z);
  if (z.numel() > 0)
    launch_xielu(z.data_ptr(), act.data_ptr<float>(), out.data_ptr(),
                 z.numel(), is_f32(z), cur_stream());
  return out;
}

static void check_route(int64_t E, int64_t top, int64_t groups,
                        int64_t keep) {
  TORCH_CHECK(E > 0 && E <= 1024, "1 to 1024 experts");
  TORCH_CHECK(groups > 0 && E % groups == 0 && keep > 0 && keep <= groups &&
                  top > 0 && top <= E / groups * keep,
              "experts, groups and choices");
}

// h: bf16 rows with the router's weights, or fp32 logits (W absent)
std::tuple<torch::Tensor, torch::Tensor> route(
    torch::Tensor h, c10::optional<torch::Tensor> W, torch::Tensor ctx,
    int64_t top, int64_t groups, int64_t keep) {
  CHECK_DEV(h); CHECK_CONT(h);
  CHECK_INTS(ctx);
  const int M = h.size(0);
  const int E = W ? W->size(0) : h.size(1);
  check_route(E, top, groups, keep);
  TORCH_CHECK(h.dim() == 2 && ctx.numel() == M, "one ctx entry per row");
  auto ids = torch::empty({M, top}, h.options().dtype(at::kInt));
  auto w = torch::empty({M, top}, h.options().dtype(at::kFloat));
  if (M == 0) return {ids, w};
  if (W) {
    CHECK_BF16(h);
    CHECK_DEV(W.value()); CHECK_CONT(W.value()); CHECK_BF16(W.value());
    const int K = h.size(1);
    TORCH_CHECK(W->size(1) == K && K % 32 == 0 && route_covers(E),
                "router shape");
    launch_route(h.data_ptr(), W->data_ptr(), ctx.data_ptr<int>(), M, E, K,
                 groups, keep, top, ids.data_ptr<int>(),
                 w.data_ptr<float>(), cur_stream());
  } else {
    CHECK_F32(h);
    launch_select(h.data_ptr<float>(), ctx.data_ptr<int>(), M, E, groups,
                  keep, top, ids.data_ptr<int>(), w.data_ptr<float>(),
                  cur_stream());
  }
  return {ids, w};
}

torch::Tensor experts(torch::Tensor h, torch::Tensor ids, torch::Tensor wgup,
                      torch::Tensor wdown) {
  CHECK_DEV(h); CHECK_CONT(h); CHECK_T(h);
  CHECK_INTS(ids);
  CHECK_DEV(wgup); CHECK_CONT(wgup); CHECK_SAME(wgup, h);
  CHECK_DEV(wdown); CHECK_CONT(wdown); CHECK_SAME(wdown, h);
  const int M = h.size(0), K = h.size(1), top = ids.size(1);
  const int E = wgup.size(0), F = wdown.size(2);
  TORCH_CHECK(ids.size(0) == M && wgup.dim() == 3 && wdown.dim() == 3 &&
                  wgup.size(1) == 2L * F && wgup.size(2) == K &&
                  wdown.size(0) == E && wdown.size(1) == K,
              "expert shapes");
  TORCH_CHECK(K % 64 == 0 && F % 64 == 0 && E <= 1024,
              "sizes % 64, at most 1024 experts");
  const long A = (long)M * top;
  TORCH_CHECK(A < (1L << 31), "too many rows");
  auto y = torch::empty({A, K}, h.options());
  if (A == 0) return y;
  // rows of a tile: twice what an expert gets on average, large tiles from
  // about 48 rows on
  const bool f32 = is_f32(h);
  const long mean = (A + E - 1) / E;
  int TM = f32 || mean <= 8 ? 16 : mean <= 16 ? 32 : mean <= 48 ? 64 : 128;
  if (!f32 && mean >= 512 && expert_gemm16_covers(2 * F, K) &&
      expert_gemm16_covers(K, F))
    TM = 256;
  const int max_tiles = (int)std::min<long>(A, A / TM + E);
  auto i32 = ids.options();
  auto plan = torch::empty({A + 4L * max_tiles + 1}, i32);
  int* perm = plan.data_ptr<int>();
  int* tiles = perm + A;
  int* ntiles = tiles + 4L * max_tiles;
  launch_expert_plan(ids.data_ptr<int>(), (int)A, E, TM, max_tiles, perm,
                     tiles, ntiles, cur_stream());
  auto inter = torch::empty({A, F}, h.options());
  launch_expert_gemm(h.data_ptr(), wgup.data_ptr(), inter.data_ptr(), perm,
                     tiles, ntiles, max_tiles, 2 * F, K, top, TM, true, f32,
                     cur_stream());
  launch_expert_gemm(inter.data_ptr(), wdown.data_ptr(), y.data_ptr(), perm,
                     tiles, ntiles, max_tiles, K, F, top, TM, false, f32,
                     cur_stream());
  return y;
}

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("attn_prep", &attn_prep);
  m.def("paged_attn_rows", &paged_attn_rows);
  m.def("paged_attn_prompts", &paged_attn_prompts);
  m.def("gated_delta", &gated_delta);
  m.def("xielu", &xielu);
  m.def("route", &route);
  m.def("experts", &experts);
}
