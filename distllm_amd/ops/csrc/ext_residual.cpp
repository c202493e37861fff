// Torch bindings of what all layered decoders share: boundaries of fp32
// residual streams, rotation tables.
#include "ext_common.h"

extern "C" {
void launch_sandwich_norm(const void*, const long*, float*, const float*,
                          const float*, void*, int, int, int, float, bool,
                          hipStream_t);
void launch_embed_positions(const void*, const void*, const long*, const int*,
                            float*, void*, int, int, int, bool, hipStream_t);
void launch_layer_norm_add(const void*, const float*, int, float*,
                           const float*, const float*, const float*,
                           const float*, void*, int, int, int, float, bool,
                           hipStream_t);
void launch_residual_step(const void*, const void*, float*, const float*,
                          const float*, int, float, const long*, float,
                          const float*, const float*, const float*,
                          const float*, bool, void*, int, int, bool,
                          hipStream_t);
void launch_stream_step(const void*, const void*, const float*, int,
                        const long*, const void*, float*, const float*,
                        const float*, const float*, int, float, bool, void*,
                        int, int, int, bool, hipStream_t);
void launch_rotation_table(const int*, const double*, float, float*, int, int,
                           hipStream_t);
}

// y == embedding table when tokens are given
torch::Tensor sandwich_norm(torch::Tensor y,
                            c10::optional<torch::Tensor> tokens,
                            torch::Tensor x,
                            c10::optional<torch::Tensor> w_post,
                            torch::Tensor w_next, int64_t n, double eps) {
  CHECK_DEV(y); CHECK_CONT(y); CHECK_T(y);
  CHECK_DEV(x); CHECK_CONT(x); CHECK_F32(x);
  CHECK_DEV(w_next); CHECK_CONT(w_next); CHECK_F32(w_next);
  const int M = x.size(0), W = x.size(1);
  TORCH_CHECK(x.dim() == 2 && y.dim() == 2 && y.size(1) == W, "row sizes");
  TORCH_CHECK(W % 8 == 0 && W <= 16384 && n > 0 && n <= W,
              "width must be a multiple of 8, at most 16384");
  TORCH_CHECK(w_next.numel() == W, "w_next size");
  const long* tok = nullptr;
  if (tokens) {
    CHECK_DEV(tokens.value()); CHECK_CONT(tokens.value());
    TORCH_CHECK(tokens->scalar_type() == at::kLong && tokens->numel() == M,
                "tokens must be int64, one per row");
    tok = (const long*)tokens->data_ptr<int64_t>();
  } else {
    TORCH_CHECK(y.size(0) == M, "y rows");
    TORCH_CHECK(w_post.has_value() && w_post->numel() == W, "w_post size");
    CHECK_DEV(w_post.value()); CHECK_CONT(w_post.value());
    CHECK_F32(w_post.value());
  }
  auto h = torch::empty({M, W}, y.options());
  if (M > 0)
    launch_sandwich_norm(y.data_ptr(), tok, x.data_ptr<float>(),
                         tok ? nullptr : w_post->data_ptr<float>(),
                         w_next.data_ptr<float>(), h.data_ptr(), M, W,
                         (int)n, (float)eps, is_f32(y), cur_stream());
  return h;
}

torch::Tensor embed_positions(torch::Tensor tokens, torch::Tensor ctx,
                              torch::Tensor table, torch::Tensor pos,
                              torch::Tensor x) {
  CHECK_DEV(table); CHECK_CONT(table); CHECK_T(table);
  CHECK_DEV(pos); CHECK_CONT(pos); CHECK_SAME(pos, table);
  CHECK_DEV(tokens); CHECK_CONT(tokens);
  CHECK_DEV(ctx); CHECK_CONT(ctx); CHECK_I32(ctx);
  CHECK_DEV(x); CHECK_CONT(x); CHECK_F32(x);
  const int M = x.size(0), W = x.size(1);
  TORCH_CHECK(tokens.scalar_type() == at::kLong && tokens.numel() == M &&
                  ctx.numel() == M,
              "tokens (int64) and ctx: one per row");
  TORCH_CHECK(W % 8 == 0 && table.size(1) == W && pos.size(1) == W &&
                  pos.size(0) > 0,
              "row sizes");
  auto h = torch::empty({M, W}, table.options());
  if (M > 0)
    launch_embed_positions(table.data_ptr(), pos.data_ptr(),
                           (const long*)tokens.data_ptr<int64_t>(),
                           ctx.data_ptr<int>(), x.data_ptr<float>(),
                           h.data_ptr(), M, W, pos.size(0), is_f32(table),
                           cur_stream());
  return h;
}

static const float* norm_vec(const torch::Tensor& t, long W) {
  CHECK_DEV(t); CHECK_CONT(t); CHECK_F32(t);
  TORCH_CHECK(t.numel() == W, "norm size");
  return t.data_ptr<float>();
}

torch::Tensor layer_norm_add(torch::Tensor y, torch::Tensor x,
                             torch::Tensor w, torch::Tensor b, int64_t n,
                             double eps, c10::optional<torch::Tensor> wf,
                             c10::optional<torch::Tensor> bf,
                             c10::optional<torch::Tensor> mix) {
  CHECK_DEV(y); CHECK_CONT(y); CHECK_T(y);
  CHECK_DEV(x); CHECK_CONT(x); CHECK_F32(x);
  const int M = x.size(0), W = x.size(1);
  TORCH_CHECK(x.dim() == 2 && y.dim() == 2 && y.size(1) == W, "row sizes");
  TORCH_CHECK(W % 8 == 0 && W <= 16384 && n > 0 && n <= W,
              "width must be a multiple of 8, at most 16384");
  TORCH_CHECK(wf.has_value() == bf.has_value(), "final weight and bias");
  int top = 1;
  if (mix) {
    CHECK_DEV(mix.value()); CHECK_CONT(mix.value()); CHECK_F32(mix.value());
    TORCH_CHECK(mix->dim() == 2 && mix->size(0) == M, "mix rows");
    top = mix->size(1);
  }
  TORCH_CHECK(y.size(0) == (long)M * top, "y rows");
  auto h = torch::empty({M, W}, y.options());
  if (M > 0)
    launch_layer_norm_add(y.data_ptr(), mix ? mix->data_ptr<float>() : nullptr,
                          top, x.data_ptr<float>(), norm_vec(w, W),
                          norm_vec(b, W), wf ? norm_vec(*wf, W) : nullptr,
                          bf ? norm_vec(*bf, W) : nullptr, h.data_ptr(), M, W,
                          (int)n, (float)eps, is_f32(y), cur_stream());
  return h;
}

typedef c10::optional<torch::Tensor> Maybe;

void residual_step(torch::Tensor x, Maybe y, Maybe bias, Maybe w_rms,
                   int64_t n, double eps, Maybe tokens, Maybe table,
                   double scale, Maybe vec, Maybe w, Maybe b, Maybe alpha,
                   bool fresh, torch::Tensor h) {
  CHECK_DEV(x); CHECK_CONT(x); CHECK_F32(x);
  CHECK_DEV(h); CHECK_CONT(h); CHECK_T(h);
  TORCH_CHECK(x.dim() == 2 && h.sizes() == x.sizes(), "row sizes");
  const int M = x.size(0), W = x.size(1);
  TORCH_CHECK(W % 8 == 0 && W <= 16384 && n > 0 && n <= W,
              "width must be a multiple of 8, at most 16384");
  const void *yp = nullptr, *tab = nullptr;
  const long* tok = nullptr;
  if (y) {
    CHECK_DEV(y.value()); CHECK_CONT(y.value()); CHECK_SAME(y.value(), h);
    TORCH_CHECK(y->sizes() == x.sizes(), "y rows");
    yp = y->data_ptr();
  }
  TORCH_CHECK(y.has_value() || (!bias && !w_rms), "bias or norm without y");
  if (tokens) {
    TORCH_CHECK(table.has_value(), "tokens without a table");
    CHECK_DEV(tokens.value()); CHECK_CONT(tokens.value());
    CHECK_DEV(table.value()); CHECK_CONT(table.value());
    CHECK_SAME(table.value(), h);
    TORCH_CHECK(tokens->scalar_type() == at::kLong && tokens->numel() == M &&
                    table->dim() == 2 && table->size(1) == W,
                "tokens (int64, one per row) and table");
    tok = (const long*)tokens->data_ptr<int64_t>();
    tab = table->data_ptr();
  }
  auto opt = [&](const Maybe& t) {
    return t ? norm_vec(*t, W) : (const float*)nullptr;
  };
  TORCH_CHECK(w.has_value() == b.has_value() &&
                  w.has_value() == alpha.has_value(),
              "weight, bias and alpha");
  if (M > 0)
    launch_residual_step(yp, tab, x.data_ptr<float>(), opt(bias), opt(w_rms),
                         (int)n, (float)eps, tok, (float)scale, opt(vec),
                         opt(w), opt(b), alpha ? norm_vec(*alpha, 1) : nullptr,
                         fresh, h.data_ptr(), M, W, is_f32(h), cur_stream());
}

// x [M, S, W]; y [M, W], or [M * top, W] with weights mix [M, top] (and one
// more column for `shared` [M, W])
void stream_step(torch::Tensor x, Maybe y, Maybe writes, Maybe mix,
                 Maybe shared, Maybe tokens, Maybe table, Maybe read,
                 torch::Tensor w, int64_t n, double eps, bool store,
                 torch::Tensor h) {
  CHECK_FLOATS(x);
  CHECK_DEV(h); CHECK_CONT(h); CHECK_T(h);
  TORCH_CHECK(x.dim() == 3 && h.dim() == 2 && h.size(0) == x.size(0) &&
                  h.size(1) == x.size(2),
              "row sizes");
  const int M = x.size(0), S = x.size(1), W = x.size(2);
  TORCH_CHECK(W % 8 == 0 && W <= 16384 && n > 0 && n <= W,
              "width must be a multiple of 8, at most 16384");
  TORCH_CHECK(S >= 1 && S <= 16, "1 to 16 streams");
  const void *yp = nullptr, *sp = nullptr, *tab = nullptr;
  const float* mp = nullptr;
  const long* tok = nullptr;
  int top = 1;
  TORCH_CHECK(y.has_value() == writes.has_value() &&
                  (y.has_value() || (!mix && !shared)) &&
                  (mix.has_value() || !shared),
              "output, its weights and the shared output");
  if (mix) {
    CHECK_FLOATS(mix.value());
    top = (int)mix->size(1) - (shared ? 1 : 0);
    TORCH_CHECK(mix->dim() == 2 && mix->size(0) == M && top > 0, "mix rows");
    mp = mix->data_ptr<float>();
  }
  if (y) {
    CHECK_DEV(y.value()); CHECK_CONT(y.value()); CHECK_SAME(y.value(), h);
    TORCH_CHECK(y->dim() == 2 && y->size(0) == (long)M * top &&
                    y->size(1) == W,
                "y rows");
    yp = y->data_ptr();
  }
  if (shared) {
    CHECK_DEV(shared.value()); CHECK_CONT(shared.value());
    CHECK_SAME(shared.value(), h);
    TORCH_CHECK(shared->sizes() == h.sizes(), "shared rows");
    sp = shared->data_ptr();
  }
  if (tokens) {
    TORCH_CHECK(table.has_value(), "tokens without a table");
    CHECK_DEV(tokens.value()); CHECK_CONT(tokens.value());
    CHECK_DEV(table.value()); CHECK_CONT(table.value());
    CHECK_SAME(table.value(), h);
    TORCH_CHECK(tokens->scalar_type() == at::kLong && tokens->numel() == M &&
                    table->dim() == 2 && table->size(1) == W,
                "tokens (int64, one per row) and table");
    tok = (const long*)tokens->data_ptr<int64_t>();
    tab = table->data_ptr();
  }
  auto opt = [&](const Maybe& t, long k) {
    return t ? norm_vec(*t, k) : (const float*)nullptr;
  };
  if (M > 0)
    launch_stream_step(yp, sp, mp, top, tok, tab, x.data_ptr<float>(),
                       opt(writes, (long)S * (S + 1)), opt(read, S),
                       norm_vec(w, W), (int)n, (float)eps,
                       store && y.has_value(), h.data_ptr(), M, S, W,
                       is_f32(h), cur_stream());
}

torch::Tensor rotation_table(torch::Tensor ctx, torch::Tensor freq,
                             double mult) {
  CHECK_INTS(ctx);
  CHECK_DEV(freq); CHECK_CONT(freq);
  TORCH_CHECK(freq.scalar_type() == at::kDouble, "freq must be f64");
  const long M = ctx.numel(), P = freq.numel();
  auto t = torch::empty({M, P, 2}, ctx.options().dtype(at::kFloat));
  if (M * P > 0)
    launch_rotation_table(ctx.data_ptr<int>(), freq.data_ptr<double>(),
                          (float)mult, t.data_ptr<float>(), M, P,
                          cur_stream());
  return t;
}

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("sandwich_norm", &sandwich_norm);
  m.def("embed_positions", &embed_positions);
  m.def("layer_norm_add", &layer_norm_add);
  m.def("residual_step", &residual_step);
  m.def("stream_step", &stream_step);
  m.def("rotation_table", &rotation_table);
}
