// Torch bindings of the latent-attention decoder kernels: latent
// preparation and attention.
#include "ext_common.h"

extern "C" {
void launch_latent_prep(const void*, int, int, int, int, int, int,
                        const float*, const float*, float, void*, void*,
                        const int*, int, int, const int*, const int*, bool,
                        hipStream_t);
void launch_latent_gather(const void*, const int*, int, int, const int*,
                          const int*, void*, int, int, hipStream_t);
void launch_head_gemm(const void*, const void*, void*, int, int, int, int,
                      hipStream_t);
void launch_latent_attn_rows(const void*, const void*, const int*,
                             const int*, const int*, void*, int, int, int,
                             int, int, float, bool, hipStream_t);
int latent_decode_heads(int);
bool latent_decode_covers(int);
void launch_latent_decode(const void*, const void*, const int*, const int*,
                          const int*, void*, void*, void*, int, int, int, int,
                          int, int, float, hipStream_t);
void launch_attn_window(const void*, const void*, const void*, void*,
                        const int*, const int*, const int*, const int*, int,
                        int, int, int, int, long, int, float, hipStream_t);
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

torch::Tensor latent_gather(torch::Tensor cache, torch::Tensor bt,
                            torch::Tensor key_seq, torch::Tensor key_pos) {
  const long T = key_seq.numel();
  check_pages(cache, bt, key_seq, key_pos, T);
  auto out = torch::empty({T, cache.size(2)}, cache.options());
  if (T > 0)
    launch_latent_gather(cache.data_ptr(), bt.data_ptr<int>(), bt.size(1),
                         cache.size(0), key_seq.data_ptr<int>(),
                         key_pos.data_ptr<int>(), out.data_ptr(), (int)T,
                         cache.size(2) * cache.element_size(), cur_stream());
  return out;
}

void head_gemm(torch::Tensor x, torch::Tensor W, torch::Tensor out) {
  CHECK_DEV(x); CHECK_CONT(x); CHECK_BF16(x);
  CHECK_DEV(W); CHECK_CONT(W); CHECK_BF16(W);
  CHECK_DEV(out); CHECK_CONT(out); CHECK_BF16(out);
  TORCH_CHECK(x.dim() == 3 && W.dim() == 3 && out.dim() == 3, "ranks");
  const int M = x.size(0), H = x.size(1), K = x.size(2), N = W.size(1);
  TORCH_CHECK(W.size(0) == H && W.size(2) == K && out.size(0) == M &&
                  out.size(1) == H && out.size(2) == N,
              "head_gemm: shape mismatch");
  TORCH_CHECK(N % 64 == 0 && K % 64 == 0, "N % 64, K % 64");
  if (M > 0)
    launch_head_gemm(x.data_ptr(), W.data_ptr(), out.data_ptr(), M, H, N, K,
                     cur_stream());
}

torch::Tensor latent_attn(torch::Tensor q, torch::Tensor cache,
                          torch::Tensor bt, torch::Tensor row_seq,
                          torch::Tensor ctx, int64_t window, double scale,
                          int64_t nsplit) {
  // nsplit: workgroups that share a row's keys; 0 = choose
  CHECK_DEV(q); CHECK_CONT(q); CHECK_T(q);
  const int M = q.size(0), H = q.size(1), R = q.size(2);
  check_pages(cache, bt, row_seq, ctx, M);
  CHECK_SAME(q, cache);
  TORCH_CHECK(cache.size(2) == R, "q and cache ranks differ");
  TORCH_CHECK(R <= 4096, "rank above 4096");
  TORCH_CHECK(window > 0, "window must be positive");
  const int win = (int)std::min<int64_t>(window, 1 << 30);
  auto out = torch::empty_like(q);
  if (M == 0) return out;
  if (is_f32(q) || !latent_decode_covers(R)) {
    launch_latent_attn_rows(q.data_ptr(), cache.data_ptr(),
                            bt.data_ptr<int>(), row_seq.data_ptr<int>(),
                            ctx.data_ptr<int>(), out.data_ptr(), M, H, R,
                            bt.size(1), win, (float)scale, is_f32(q),
                            cur_stream());
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
                       out.data_ptr(), pa, pm, M, H, R, (int)NS, bt.size(1),
                       win, (float)scale, cur_stream());
  return out;
}

// q [Tq, H, DK]; kv [Tk, H*DK + H*DV] (keys, then values); out [Tq, H, DV]
void attn_window(torch::Tensor q, torch::Tensor kv, torch::Tensor out,
                 torch::Tensor cu_q, torch::Tensor cu_k,
                 torch::Tensor blk_seq, torch::Tensor blk_qb, int64_t window,
                 double scale) {
  CHECK_DEV(q); CHECK_CONT(q); CHECK_BF16(q);
  CHECK_DEV(kv); CHECK_CONT(kv); CHECK_BF16(kv);
  CHECK_DEV(out); CHECK_CONT(out); CHECK_BF16(out);
  for (const auto& t : {cu_q, cu_k, blk_seq, blk_qb}) {
    CHECK_DEV(t); CHECK_CONT(t); CHECK_I32(t);
  }
  const int H = q.size(1), DK = q.size(2), DV = out.size(2);
  TORCH_CHECK((DK == 64 || DK == 128 || DK == 256) &&
                  (DV == 64 || DV == 128 || DV == 256),
              "head sizes must be 64, 128 or 256");
  TORCH_CHECK(kv.size(1) == (long)H * (DK + DV), "kv row size");
  TORCH_CHECK(out.size(0) == q.size(0) && out.size(1) == H, "out shape");
  TORCH_CHECK(cu_q.numel() == cu_k.numel() &&
                  blk_seq.numel() == blk_qb.numel() && window > 0,
              "sequence maps");
  const int win = (int)std::min<int64_t>(window, 1 << 30);
  const int nblocks = blk_seq.numel();
  if (nblocks > 0)
    launch_attn_window(
        q.data_ptr(), kv.data_ptr(),
        (const char*)kv.data_ptr() + (long)H * DK * kv.element_size(),
        out.data_ptr(), cu_q.data_ptr<int>(), cu_k.data_ptr<int>(),
        blk_seq.data_ptr<int>(), blk_qb.data_ptr<int>(), nblocks,
        cu_q.numel() - 1, H, DK, DV, kv.size(1), win, (float)scale,
        cur_stream());
}

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("latent_prep", &latent_prep);
  m.def("latent_gather", &latent_gather);
  m.def("head_gemm", &head_gemm);
  m.def("latent_attn", &latent_attn, py::arg("q"), py::arg("cache"),
        py::arg("block_table"), py::arg("row_seq"), py::arg("ctx"),
        py::arg("window"), py::arg("scale"), py::arg("nsplit") = 0);
  m.def("attn_window", &attn_window);
}
