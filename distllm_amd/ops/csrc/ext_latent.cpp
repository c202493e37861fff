// Torch bindings of the latent-attention decoder kernels: latent
// preparation and attention.
#include "ext_common.h"

extern "C" {
void launch_latent_prep(const void*, int, int, int, int, int, int,
                        const float*, const float*, float, void*, void*,
                        const int*, int, int, const int*, const int*, bool,
                        hipStream_t);
void launch_latent_gather(const void*, const int*, int, int, const int*,
                          const int*, void*, void*, int, int, int,
                          hipStream_t);
void launch_rotary_latent_prep(void*, int, int, int, int, int, int, int,
                               const float*, float, const float*, int, void*,
                               int, int, void*, const int*, int, int,
                               const int*, const int*, bool, hipStream_t);
void launch_head_gemm(const void*, const void*, void*, int, int, int, int,
                      long, int, long, int, hipStream_t);
void launch_latent_attn_rows(const void*, const void*, const int*,
                             const int*, const int*, void*, int, int, int,
                             int, int, int, float, const float*, const void*,
                             int, bool, hipStream_t);
int latent_decode_heads(int);
bool latent_decode_covers(int, int);
void launch_latent_decode(const void*, const void*, const int*, const int*,
                          const int*, void*, void*, void*, int, int, int, int,
                          int, int, int, float, const float*, const void*,
                          int, hipStream_t);
void launch_attn_window(const void*, const void*, const void*, const void*,
                        void*, const int*, const int*, const int*, const int*,
                        int, int, int, int, int, long, long, int, float,
                        const float*, const void*, int, hipStream_t);
}

static void check_pages(const torch::Tensor& cache, const torch::Tensor& bt,
                        const torch::Tensor& row_seq,
                        const torch::Tensor& ctx, long M) {
  CHECK_DEV(cache); CHECK_CONT(cache); CHECK_T(cache);
  TORCH_CHECK(cache.dim() == 3 && cache.size(1) == 16 &&
                  cache.size(2) % 64 == 0,
              "cache must be [blocks, 16, rank % 64 == 0]");
  CHECK_DEV(bt); CHECK_CONT(bt); CHECK_I32(bt);
  CHECK_DEV(row_seq); CHECK_CONT(row_seq); CHECK_I32(row_seq);
  CHECK_DEV(ctx); CHECK_CONT(ctx); CHECK_I32(ctx);
  TORCH_CHECK(bt.dim() == 2 && row_seq.numel() == M && ctx.numel() == M,
              "one row_seq and ctx entry per row");
}

torch::Tensor latent_prep(torch::Tensor ab, int64_t QP, int64_t qn,
                          int64_t rn, torch::Tensor wq,
                          c10::optional<torch::Tensor> wc, double eps,
                          c10::optional<torch::Tensor> cache,
                          torch::Tensor bt, torch::Tensor row_seq,
                          torch::Tensor ctx) {
  CHECK_DEV(ab); CHECK_CONT(ab); CHECK_T(ab);
  CHECK_DEV(wq); CHECK_CONT(wq); CHECK_F32(wq);
  const int M = ab.size(0), ld = ab.size(1);
  const int R = ld - (int)QP;
  TORCH_CHECK(R >= 0 && wq.numel() == QP && qn > 0 && qn <= QP, "q sizes");
  TORCH_CHECK(QP % 8 == 0 && QP <= 8192 && R <= 8192,
              "latent sizes must be multiples of 8, at most 8192");
  void* cp = nullptr;
  const float* wcp = nullptr;
  int nblk = 0;
  if (cache) {
    check_pages(cache.value(), bt, row_seq, ctx, M);
    CHECK_SAME(ab, cache.value());
    TORCH_CHECK(cache->size(2) == R && rn > 0 && rn <= R, "rank");
    TORCH_CHECK(wc.has_value() && wc->numel() == R, "latent norm size");
    CHECK_DEV(wc.value()); CHECK_CONT(wc.value()); CHECK_F32(wc.value());
    cp = cache->data_ptr();
    wcp = wc->data_ptr<float>();
    nblk = cache->size(0);
  } else {
    TORCH_CHECK(R == 0, "latent columns without a cache");
  }
  auto cq = torch::empty({M, QP}, ab.options());
  if (M > 0)
    launch_latent_prep(ab.data_ptr(), M, ld, (int)QP, (int)qn, R, (int)rn,
                       wq.data_ptr<float>(), wcp, (float)eps, cq.data_ptr(),
                       cp, bt.data_ptr<int>(), bt.size(1), nblk,
                       row_seq.data_ptr<int>(), ctx.data_ptr<int>(),
                       is_f32(ab), cur_stream());
  return cq;
}

typedef c10::optional<torch::Tensor> Maybe;

// Rows ab: H heads of dp and tp columns, then, with a cache, latent and key
// part (see latent_attention.hip). ql [n, H, latent + tp].
void rotary_latent_prep(torch::Tensor ab, int64_t H, int64_t dp, int64_t tp,
                        int64_t rn, Maybe wc, double eps, torch::Tensor table,
                        Maybe cache, torch::Tensor bt, torch::Tensor row_seq,
                        torch::Tensor ctx, torch::Tensor ql) {
  CHECK_T(ab); CHECK_CONT(ab);
  const int M = ab.size(0), ld = row_stride(ab);
  CHECK_FLOATS(table);
  CHECK_DEV(ql); CHECK_CONT(ql); CHECK_SAME(ql, ab);
  TORCH_CHECK(dp % 8 == 0 && tp % 8 == 0 && H > 0 && ld % 8 == 0, "sizes % 8");
  TORCH_CHECK(table.dim() == 3 && table.size(0) == M && table.size(1) > 0 &&
                  2 * table.size(1) <= tp && table.size(2) == 2,
              "rotation table");
  const int n = ql.size(0), R = (int)(ql.size(2) - tp);
  TORCH_CHECK(ql.dim() == 3 && n <= M && ql.size(1) == H && R > 0 &&
                  R % 8 == 0 && R <= 4096,
              "query rows, latents of up to 4096");
  void* cp = nullptr;
  const float* wcp = nullptr;
  int nblk = 0;
  if (cache) {
    check_pages(cache.value(), bt, row_seq, ctx, M);
    CHECK_SAME(ab, cache.value());
    TORCH_CHECK(cache->size(2) == R + tp && rn > 0 && rn <= R, "rank");
    TORCH_CHECK(wc.has_value() && wc->numel() == R, "latent norm size");
    CHECK_FLOATS(wc.value());
    cp = cache->data_ptr();
    wcp = wc->data_ptr<float>();
    nblk = cache->size(0);
  } else {
    CHECK_INTS(bt);
  }
  TORCH_CHECK(ab.size(1) >= H * (dp + tp) + (cache ? R + tp : 0),
              "projection columns");
  if (M > 0)
    launch_rotary_latent_prep(
        ab.data_ptr(), M, ld, (int)H, (int)dp, (int)tp, R, (int)rn, wcp,
        (float)eps, table.data_ptr<float>(), table.size(1), ql.data_ptr(), n,
        R + (int)tp, cp, bt.data_ptr<int>(), bt.size(1), nblk,
        row_seq.data_ptr<int>(), ctx.data_ptr<int>(), is_f32(ab),
        cur_stream());
}

// -> the first `rank` columns of the cache rows, and the others
std::tuple<torch::Tensor, torch::Tensor> latent_gather(
    torch::Tensor cache, torch::Tensor bt, torch::Tensor key_seq,
    torch::Tensor key_pos, int64_t rank) {
  const long T = key_seq.numel();
  check_pages(cache, bt, key_seq, key_pos, T);
  const long R = cache.size(2), el = cache.element_size();
  TORCH_CHECK(rank > 0 && rank <= R && rank % 8 == 0, "rank");
  auto out = torch::empty({T, rank}, cache.options());
  auto rest = torch::empty({T, R - rank}, cache.options());
  if (T > 0)
    launch_latent_gather(cache.data_ptr(), bt.data_ptr<int>(), bt.size(1),
                         cache.size(0), key_seq.data_ptr<int>(),
                         key_pos.data_ptr<int>(), out.data_ptr(),
                         rest.data_ptr(), (int)T, R * el, rank * el,
                         cur_stream());
  return {out, rest};
}

static void check_heads(const torch::Tensor& t) {
  CHECK_DEV(t); CHECK_BF16(t);
  TORCH_CHECK(t.dim() == 3 && t.stride(2) == 1 && t.stride(0) % 8 == 0 &&
                  t.stride(1) % 8 == 0 && t.stride(1) < (1L << 31) &&
                  (uintptr_t)t.data_ptr() % 16 == 0,
              "heads must be rows of aligned, contiguous numbers");
}

void head_gemm(torch::Tensor x, torch::Tensor W, torch::Tensor out) {
  check_heads(x);
  check_heads(out);
  CHECK_DEV(W); CHECK_CONT(W); CHECK_BF16(W);
  TORCH_CHECK(W.dim() == 3, "weights of heads");
  const int M = x.size(0), H = x.size(1), K = x.size(2), N = W.size(1);
  TORCH_CHECK(W.size(0) == H && W.size(2) == K && out.size(0) == M &&
                  out.size(1) == H && out.size(2) == N,
              "head_gemm: shape mismatch");
  TORCH_CHECK(N % 64 == 0 && K % 64 == 0, "N % 64, K % 64");
  if (M > 0)
    launch_head_gemm(x.data_ptr(), W.data_ptr(), out.data_ptr(), M, H, N, K,
                     x.stride(0), (int)x.stride(1), out.stride(0),
                     (int)out.stride(1), cur_stream());
}

struct HeadEnds {
  const float* sink = nullptr;
  const void* gate = nullptr;
  int ld_gate = 0;
};

// sink [H] and gate [M, H] (strided rows) of attention outputs
static HeadEnds head_ends(const Maybe& sink, const Maybe& gate,
                          const torch::Tensor& q, long M, long H) {
  HeadEnds e;
  if (sink) {
    CHECK_FLOATS(sink.value());
    TORCH_CHECK(sink->numel() == H, "one sink per head");
    e.sink = sink->data_ptr<float>();
  }
  if (gate) {
    e.ld_gate = row_stride(gate.value());
    CHECK_SAME(gate.value(), q);
    TORCH_CHECK(gate->size(0) == M && gate->size(1) == H,
                "one gate per row and head");
    e.gate = gate->data_ptr();
  }
  return e;
}

torch::Tensor latent_attn(torch::Tensor q, torch::Tensor cache,
                          torch::Tensor bt, torch::Tensor row_seq,
                          torch::Tensor ctx, int64_t window, double scale,
                          int64_t nsplit, int64_t rank, Maybe sink,
                          Maybe gate) {
  // nsplit: workgroups that share a row's keys; 0 = choose
  CHECK_DEV(q); CHECK_CONT(q); CHECK_T(q);
  TORCH_CHECK(q.dim() == 3, "q [rows, heads, row of the cache]");
  const int M = q.size(0), H = q.size(1), RT = q.size(2), R = (int)rank;
  check_pages(cache, bt, row_seq, ctx, M);
  CHECK_SAME(q, cache);
  TORCH_CHECK(cache.size(2) == RT, "q and cache ranks differ");
  TORCH_CHECK(R > 0 && R <= RT && R % 8 == 0 && R <= 4096,
              "values of up to 4096 numbers of a row");
  TORCH_CHECK(RT <= 8192, "cache rows of up to 8192 numbers");
  TORCH_CHECK(window > 0, "window must be positive");
  const HeadEnds e = head_ends(sink, gate, q, M, H);
  const int win = (int)std::min<int64_t>(window, 1 << 30);
  auto out = torch::empty({M, H, R}, q.options());
  if (M == 0) return out;
  if (is_f32(q) || !latent_decode_covers(R, RT - R)) {
    launch_latent_attn_rows(q.data_ptr(), cache.data_ptr(),
                            bt.data_ptr<int>(), row_seq.data_ptr<int>(),
                            ctx.data_ptr<int>(), out.data_ptr(), M, H, R, RT,
                            bt.size(1), win, (float)scale, e.sink, e.gate,
                            e.ld_gate, is_f32(q), cur_stream());
    return out;
  }
  // Split each row's keys until the CUs are full (two workgroups each, one
  // of the largest), as long as a split keeps four tiles. All sizes are
  // known on the host, so a captured graph stays valid as contexts grow.
  long NS = nsplit;
  if (NS <= 0) {
    const long per_wg = latent_decode_heads(H);
    const long wgs = (long)M * ((H + per_wg - 1) / per_wg);
    const long keys = std::min<long>(win, bt.size(1) * 16L);
    const long tiles = keys / 32 + 1;
    const long fill = per_wg > 32 ? 256 : 512;
    NS = std::min<long>({(fill + wgs - 1) / wgs, (tiles + 3) / 4, 64L});
  }
  NS = std::max<long>(NS, 1);
  torch::Tensor pacc, pml;
  void *pa = nullptr, *pm = nullptr;
  if (NS > 1) {
    auto f32 = q.options().dtype(at::kFloat);
    pacc = torch::empty({(long)M * H * NS, R}, f32);
    pml = torch::empty({(long)M * H * NS, 2}, f32);
    pa = pacc.data_ptr();
    pm = pml.data_ptr();
  }
  launch_latent_decode(q.data_ptr(), cache.data_ptr(), bt.data_ptr<int>(),
                       row_seq.data_ptr<int>(), ctx.data_ptr<int>(),
                       out.data_ptr(), pa, pm, M, H, R, RT - R, (int)NS,
                       bt.size(1), win, (float)scale, e.sink, e.gate,
                       e.ld_gate, cur_stream());
  return out;
}

// q [Tq, H, DK (+ DR)], rows strided; kv [Tk, H*DK + H*DV] (keys, then
// values); kr [Tk, DR], keys' numbers that all heads share; out [Tq, H, DV]
void attn_window(torch::Tensor q, torch::Tensor kv, torch::Tensor out,
                 torch::Tensor cu_q, torch::Tensor cu_k,
                 torch::Tensor blk_seq, torch::Tensor blk_qb, int64_t window,
                 double scale, Maybe kr, Maybe sink, Maybe gate) {
  check_heads(q);
  CHECK_DEV(kv); CHECK_CONT(kv); CHECK_BF16(kv);
  CHECK_DEV(out); CHECK_CONT(out); CHECK_BF16(out);
  for (const auto& t : {cu_q, cu_k, blk_seq, blk_qb}) {
    CHECK_DEV(t); CHECK_CONT(t); CHECK_I32(t);
  }
  const void* krp = nullptr;
  int DR = 0;
  if (kr) {
    CHECK_DEV(kr.value()); CHECK_CONT(kr.value()); CHECK_BF16(kr.value());
    DR = kr->size(1);
    TORCH_CHECK(kr->size(0) == kv.size(0) && DR == 64,
                "shared key numbers: 64 per key");
    krp = kr->data_ptr();
  }
  const int H = q.size(1), DK = q.size(2) - DR, DV = out.size(2);
  TORCH_CHECK((DK == 64 || DK == 128 || DK == 256) &&
                  (DV == 64 || DV == 128 || DV == 256),
              "head sizes must be 64, 128 or 256");
  TORCH_CHECK(q.stride(1) == DK + DR, "heads of q must be neighbours");
  TORCH_CHECK(kv.size(1) == (long)H * (DK + DV), "kv row size");
  TORCH_CHECK(out.size(0) == q.size(0) && out.size(1) == H, "out shape");
  TORCH_CHECK(cu_q.numel() == cu_k.numel() &&
                  blk_seq.numel() == blk_qb.numel() && window > 0,
              "sequence maps");
  const HeadEnds e = head_ends(sink, gate, q, q.size(0), H);
  const int win = (int)std::min<int64_t>(window, 1 << 30);
  const int nblocks = blk_seq.numel();
  if (nblocks > 0)
    launch_attn_window(
        q.data_ptr(), kv.data_ptr(),
        (const char*)kv.data_ptr() + (long)H * DK * kv.element_size(), krp,
        out.data_ptr(), cu_q.data_ptr<int>(), cu_k.data_ptr<int>(),
        blk_seq.data_ptr<int>(), blk_qb.data_ptr<int>(), nblocks,
        cu_q.numel() - 1, H, DK, DV, q.stride(0), kv.size(1), win,
        (float)scale, e.sink, e.gate, e.ld_gate, cur_stream());
}

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("latent_prep", &latent_prep);
  m.def("latent_gather", &latent_gather);
  m.def("head_gemm", &head_gemm);
  m.def("latent_attn", &latent_attn);
  m.def("rotary_latent_prep", &rotary_latent_prep);
  m.def("attn_window", &attn_window);
}
