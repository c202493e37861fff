// Torch bindings of xIELU and routed experts.
#include "ext_common.h"

extern "C" {
void launch_xielu(const void*, const float*, void*, long, bool, hipStream_t);
bool route_covers(int);
bool expert_gemm16_covers(int, int);
void launch_select(const float*, const int*, int, int, int, int, int,
                   const float*, float, bool, int, int*, float*, hipStream_t);
void launch_route(const void*, const void*, const int*, int, int, int, int,
                  int, int, const float*, float, bool, int, int*, float*,
                  hipStream_t);
long expert_plan_scratch(long, int);
void launch_expert_plan(const int*, int, int, int, int, int*, int*, int*,
                        int*, hipStream_t);
void launch_expert_gemm(const void*, const void*, void*, const int*,
                        const int*, const int*, int, int, int, int, int, int,
                        bool, hipStream_t);
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

// h: bf16 rows with the router's weights, or fp32 logits (W absent). gate:
// the last logit is that of an expert that serves every row, in `shards`
// pieces behind the experts, or (0) as a weight only.
static std::tuple<torch::Tensor, torch::Tensor> choose(
    torch::Tensor h, c10::optional<torch::Tensor> W, torch::Tensor ctx,
    int64_t top, int64_t groups, int64_t keep, const float* correction,
    double scale, bool gate, int64_t shards) {
  CHECK_DEV(h); CHECK_CONT(h);
  CHECK_INTS(ctx);
  const int M = h.size(0);
  const int logits = W ? W->size(0) : h.size(1), E = logits - gate;
  check_route(E, top, groups, keep);
  TORCH_CHECK(h.dim() == 2 && ctx.numel() == M, "one ctx entry per row");
  TORCH_CHECK(shards >= 0 && (gate || shards == 0), "shards of no expert");
  auto ids = torch::empty({M, top + shards}, h.options().dtype(at::kInt));
  auto w = torch::empty({M, top + (shards > 0 ? shards : (int64_t)gate)},
                        h.options().dtype(at::kFloat));
  if (M == 0) return {ids, w};
  if (W) {
    CHECK_BF16(h);
    CHECK_DEV(W.value()); CHECK_CONT(W.value()); CHECK_BF16(W.value());
    const int K = h.size(1);
    TORCH_CHECK(W->size(1) == K && K % 32 == 0 && route_covers(logits),
                "router shape");
    launch_route(h.data_ptr(), W->data_ptr(), ctx.data_ptr<int>(), M, E, K,
                 groups, keep, top, correction, (float)scale, gate,
                 (int)shards, ids.data_ptr<int>(), w.data_ptr<float>(), cur_stream());
  } else {
    CHECK_F32(h);
    launch_select(h.data_ptr<float>(), ctx.data_ptr<int>(), M, E, groups,
                  keep, top, correction, (float)scale, gate, (int)shards,
                  ids.data_ptr<int>(), w.data_ptr<float>(), cur_stream());
  }
  return {ids, w};
}

std::tuple<torch::Tensor, torch::Tensor> route(
    torch::Tensor h, c10::optional<torch::Tensor> W, torch::Tensor ctx,
    int64_t top, int64_t groups, int64_t keep) {
  return choose(h, W, ctx, top, groups, keep, nullptr, 1.0, false, 0);
}

std::tuple<torch::Tensor, torch::Tensor> route_sigmoid(
    torch::Tensor h, c10::optional<torch::Tensor> W, torch::Tensor correction,
    torch::Tensor ctx, int64_t top, double scale, int64_t shards) {
  CHECK_FLOATS(correction);
  const long n = W ? W->size(0) : h.size(1);
  const long gate = n - correction.numel();
  TORCH_CHECK(gate == 0 || gate == 1, "one correction per expert");
  return choose(h, W, ctx, top, 1, 1, correction.data_ptr<float>(), scale,
                gate == 1, shards);
}

// gated units, wup [E, 2F, K], or squared ReLU, wup [E, F, K]
torch::Tensor experts(torch::Tensor h, torch::Tensor ids, torch::Tensor wup,
                      torch::Tensor wdown, bool gated) {
  CHECK_DEV(h); CHECK_CONT(h); CHECK_T(h);
  CHECK_INTS(ids);
  CHECK_DEV(wup); CHECK_CONT(wup); CHECK_SAME(wup, h);
  CHECK_DEV(wdown); CHECK_CONT(wdown); CHECK_SAME(wdown, h);
  const int M = h.size(0), K = h.size(1), top = ids.size(1);
  const int E = wup.size(0), F = wdown.size(2);
  const int N = gated ? 2 * F : F;  // columns of the first product
  TORCH_CHECK(ids.size(0) == M && wup.dim() == 3 && wdown.dim() == 3 &&
                  wup.size(1) == N && wup.size(2) == K &&
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
  if (!f32 && mean >= 512 && expert_gemm16_covers(N, K) &&
      expert_gemm16_covers(K, F))
    TM = 256;
  const int max_tiles = (int)std::min<long>(A, A / TM + E);
  auto i32 = ids.options();
  auto plan = torch::empty(
      {A + 4L * max_tiles + 1 + expert_plan_scratch(A, E)}, i32);
  int* perm = plan.data_ptr<int>();
  int* tiles = perm + A;
  int* ntiles = tiles + 4L * max_tiles;
  launch_expert_plan(ids.data_ptr<int>(), (int)A, E, TM, max_tiles, perm,
                     tiles, ntiles, ntiles + 1, cur_stream());
  auto inter = torch::empty({A, F}, h.options());
  launch_expert_gemm(h.data_ptr(), wup.data_ptr(), inter.data_ptr(), perm,
                     tiles, ntiles, max_tiles, N, K, top, TM, gated ? 1 : 2,
                     f32, cur_stream());
  launch_expert_gemm(inter.data_ptr(), wdown.data_ptr(), y.data_ptr(), perm,
                     tiles, ntiles, max_tiles, K, F, top, TM, 0, f32,
                     cur_stream());
  return y;
}

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("xielu", &xielu);
  m.def("route", &route);
  m.def("route_sigmoid", &route_sigmoid);
  m.def("experts", &experts);
}
