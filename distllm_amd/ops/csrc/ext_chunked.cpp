// Torch bindings of attention over the chunks of paged keys and values, with
// capped scores and a distance bias.
#include "ext_attention.h"

extern "C" {
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
  const long NS = key_splits(nsplit, a.M, a.H, p.G, ch, bt.size(1));
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

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("paged_attn_rows", &paged_attn_rows);
  m.def("paged_attn_prompts", &paged_attn_prompts);
}
