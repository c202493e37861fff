// Sublayer boundaries of decoders with an fp32 residual stream x.
//
// RMS norms before and after each sublayer ("sandwich"):
//   embed_norm:      x = E[token];            h = rms(x) * w_next
//   post_norm_add:   x += rms(y) * w_post;    h = rms(x) * w_next
// Layer norm of the sublayer's output only:
//   embed_positions: x = E[token] + P[pos];   h = x
//   layer_norm_add:  x += ln(y) * w + b;      h = x, or ln(x) * wf + bf
// where y may be a weighted sum of several rows (routed experts).
// Pre-norm streams with an elementwise activation in the norm's place:
//   residual_step:   x += y + bias, or x += rms(y) * w;  x += scale E[token];
//                    x += vec;  h = x, or tanh(alpha x) * w + b
//
// One launch per boundary: the sublayer output y is normed and added and
// the next sublayer's input is produced while the row is still in
// registers. Statistics are over the first n columns; rows are padded
// with zeros to W columns. T is the type of y, h and E (bf16 or fp32).
#include "common.h"

// sum over the TPR threads (one or four waves) that share a row
template <int TPR>
__device__ __forceinline__ float row_sum(float v, float* scratch) {
  v = wave_reduce_sum(v);
  if (TPR == 64) return v;
  const int wid = threadIdx.x >> 6;
  __syncthreads();  // the previous use of scratch is over
  if ((threadIdx.x & 63) == 0) scratch[wid] = v;
  __syncthreads();
  return scratch[0] + scratch[1] + scratch[2] + scratch[3];
}

template <typename T, int NC, int TPR, bool EMBED>
__global__ void __launch_bounds__(256)
sandwich_norm_kernel(const T* __restrict__ y, const long* __restrict__ tokens,
                     float* __restrict__ x, const float* __restrict__ w_post,
                     const float* __restrict__ w_next, T* __restrict__ h,
                     int M, int W, int n, float eps) {
  __shared__ float scratch[4];
  const int sub = threadIdx.x % TPR;
  const int row = blockIdx.x * (256 / TPR) + threadIdx.x / TPR;
  if (row >= M) return;  // whole waves; whole blocks when TPR == 256
  const T* yr = y + (EMBED ? tokens[row] : (long)row) * W;
  float* xr = x + (long)row * W;

  float v[NC][8];
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < NC; ++k) {
    const int c = (sub + k * TPR) * 8;
#pragma unroll
    for (int i = 0; i < 8; ++i) v[k][i] = 0.f;
    if (c < W) load8<T>(yr + c, v[k]);
#pragma unroll
    for (int i = 0; i < 8; ++i) ss += v[k][i] * v[k][i];
  }
  ss = row_sum<TPR>(ss, scratch);
  if (!EMBED) {
    const float inv = 1.f / sqrtf(ss / n + eps);
    ss = 0.f;
#pragma unroll
    for (int k = 0; k < NC; ++k) {
      const int c = (sub + k * TPR) * 8;
      if (c < W) {
        float xv[8], wv[8];
        load8<float>(xr + c, xv);
        load8<float>(w_post + c, wv);
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          v[k][i] = xv[i] + v[k][i] * inv * wv[i];
          ss += v[k][i] * v[k][i];
        }
      }
    }
    ss = row_sum<TPR>(ss, scratch);
  }
  const float inv = 1.f / sqrtf(ss / n + eps);
#pragma unroll
  for (int k = 0; k < NC; ++k) {
    const int c = (sub + k * TPR) * 8;
    if (c < W) {
      float wv[8], o[8];
      load8<float>(w_next + c, wv);
#pragma unroll
      for (int i = 0; i < 8; ++i) o[i] = v[k][i] * inv * wv[i];
      store8(xr + c, v[k]);
      store8(h + (long)row * W + c, o);
    }
  }
}

extern "C" void launch_sandwich_norm(const void* y, const long* tokens,
                                     float* x, const float* w_post,
                                     const float* w_next, void* h, int M,
                                     int W, int n, float eps, bool fp32,
                                     hipStream_t stream) {
  // a wave per row up to 1024 columns, a workgroup per row above
  const int tpr = W <= 1024 ? 64 : 256;
  const int rows = 256 / tpr;
  const dim3 grid((M + rows - 1) / rows);
  const int nc = (W / 8 + tpr - 1) / tpr;
#define SN(T, NC, TPR, EM)                                                    \
  hipLaunchKernelGGL((sandwich_norm_kernel<T, NC, TPR, EM>), grid, dim3(256), \
                     0, stream, (const T*)y, tokens, x, w_post, w_next,       \
                     (T*)h, M, W, n, eps)
#define SN_E(T, NC, TPR)                       \
  do {                                         \
    if (tokens != nullptr) SN(T, NC, TPR, true); \
    else SN(T, NC, TPR, false);                \
  } while (0)
#define SN_N(T)                              \
  do {                                       \
    if (tpr == 64 && nc == 1) SN_E(T, 1, 64);  \
    else if (tpr == 64) SN_E(T, 2, 64);      \
    else if (nc == 1) SN_E(T, 1, 256);       \
    else if (nc == 2) SN_E(T, 2, 256);       \
    else if (nc <= 4) SN_E(T, 4, 256);       \
    else SN_E(T, 8, 256);                    \
  } while (0)
  if (fp32) SN_N(float);
  else SN_N(unsigned short);
#undef SN_N
#undef SN_E
#undef SN
}

template <typename T>
__global__ void __launch_bounds__(256)
embed_positions_kernel(const T* __restrict__ table,
                       const T* __restrict__ pos_table,
                       const long* __restrict__ tokens,
                       const int* __restrict__ ctx, float* __restrict__ x,
                       T* __restrict__ h, int M, int W, int max_pos) {
  const int vec = W / 8;
  const long i = (long)blockIdx.x * 256 + threadIdx.x;
  if (i >= (long)M * vec) return;
  const int row = (int)(i / vec), c = (int)(i % vec) * 8;
  const int pos = min(max(ctx[row] - 1, 0), max_pos - 1);
  float a[8], b[8];
  load8<T>(table + tokens[row] * W + c, a);
  load8<T>(pos_table + (long)pos * W + c, b);
#pragma unroll
  for (int k = 0; k < 8; ++k) a[k] += b[k];
  store8(x + (long)row * W + c, a);
  store8(h + (long)row * W + c, a);
}

extern "C" void launch_embed_positions(const void* table, const void* pos,
                                       const long* tokens, const int* ctx,
                                       float* x, void* h, int M, int W,
                                       int max_pos, bool fp32,
                                       hipStream_t stream) {
  const dim3 grid(((long)M * (W / 8) + 255) / 256);
#define EP(T)                                                               \
  hipLaunchKernelGGL((embed_positions_kernel<T>), grid, dim3(256), 0,       \
                     stream, (const T*)table, (const T*)pos, tokens, ctx, x, \
                     (T*)h, M, W, max_pos)
  if (fp32) EP(float);
  else EP(unsigned short);
#undef EP
}

// (v - mean) / sqrt(var + eps) over the first n columns, in place
template <int NC, int TPR>
__device__ __forceinline__ void center_scale(float v[NC][8], int sub, int n,
                                             float eps, float* scratch) {
  float s = 0.f;
#pragma unroll
  for (int k = 0; k < NC; ++k)
#pragma unroll
    for (int i = 0; i < 8; ++i) s += v[k][i];
  const float mean = row_sum<TPR>(s, scratch) / n;
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < NC; ++k) {
    const int c = (sub + k * TPR) * 8;
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      v[k][i] = c + i < n ? v[k][i] - mean : 0.f;
      ss += v[k][i] * v[k][i];
    }
  }
  const float inv = 1.f / sqrtf(row_sum<TPR>(ss, scratch) / n + eps);
#pragma unroll
  for (int k = 0; k < NC; ++k)
#pragma unroll
    for (int i = 0; i < 8; ++i) v[k][i] *= inv;
}

// mix == nullptr: y [M, W]; else y [M * top, W] with weights mix [M, top]
template <typename T, int NC, int TPR>
__global__ void __launch_bounds__(256)
layer_norm_add_kernel(const T* __restrict__ y, const float* __restrict__ mix,
                      int top, float* __restrict__ x,
                      const float* __restrict__ w,
                      const float* __restrict__ b,
                      const float* __restrict__ wf,
                      const float* __restrict__ bf, T* __restrict__ h, int M,
                      int W, int n, float eps) {
  __shared__ float scratch[4];
  const int sub = threadIdx.x % TPR;
  const int row = blockIdx.x * (256 / TPR) + threadIdx.x / TPR;
  if (row >= M) return;  // whole waves; whole blocks when TPR == 256
  float* xr = x + (long)row * W;

  float v[NC][8];
#pragma unroll
  for (int k = 0; k < NC; ++k)
#pragma unroll
    for (int i = 0; i < 8; ++i) v[k][i] = 0.f;
  if (mix == nullptr) {
#pragma unroll
    for (int k = 0; k < NC; ++k) {
      const int c = (sub + k * TPR) * 8;
      if (c < W) load8<T>(y + (long)row * W + c, v[k]);
    }
  } else {
    for (int e = 0; e < top; ++e) {
      const float m = mix[(long)row * top + e];
      if (m == 0.f) continue;  // no expert: its row was never written
      const T* yr = y + ((long)row * top + e) * W;
#pragma unroll
      for (int k = 0; k < NC; ++k) {
        const int c = (sub + k * TPR) * 8;
        if (c < W) {
          float t[8];
          load8<T>(yr + c, t);
#pragma unroll
          for (int i = 0; i < 8; ++i) v[k][i] += m * t[i];
        }
      }
    }
  }
  center_scale<NC, TPR>(v, sub, n, eps, scratch);
#pragma unroll
  for (int k = 0; k < NC; ++k) {
    const int c = (sub + k * TPR) * 8;
    if (c < W) {
      float xv[8], wv[8], bv[8];
      load8<float>(xr + c, xv);
      load8<float>(w + c, wv);
      load8<float>(b + c, bv);
#pragma unroll
      for (int i = 0; i < 8; ++i)
        v[k][i] = xv[i] + v[k][i] * wv[i] + bv[i];
      store8(xr + c, v[k]);
    }
  }
  if (wf != nullptr) {
    center_scale<NC, TPR>(v, sub, n, eps, scratch);
#pragma unroll
    for (int k = 0; k < NC; ++k) {
      const int c = (sub + k * TPR) * 8;
      if (c < W) {
        float wv[8], bv[8];
        load8<float>(wf + c, wv);
        load8<float>(bf + c, bv);
#pragma unroll
        for (int i = 0; i < 8; ++i) v[k][i] = v[k][i] * wv[i] + bv[i];
      }
    }
  }
#pragma unroll
  for (int k = 0; k < NC; ++k) {
    const int c = (sub + k * TPR) * 8;
    if (c < W) store8(h + (long)row * W + c, v[k]);
  }
}

extern "C" void launch_layer_norm_add(const void* y, const float* mix,
                                      int top, float* x, const float* w,
                                      const float* b, const float* wf,
                                      const float* bf, void* h, int M, int W,
                                      int n, float eps, bool fp32,
                                      hipStream_t stream) {
  const int tpr = W <= 1024 ? 64 : 256;
  const int rows = 256 / tpr;
  const dim3 grid((M + rows - 1) / rows);
  const int nc = (W / 8 + tpr - 1) / tpr;
#define LN(T, NC, TPR)                                                    \
  hipLaunchKernelGGL((layer_norm_add_kernel<T, NC, TPR>), grid, dim3(256), \
                     0, stream, (const T*)y, mix, top, x, w, b, wf, bf,   \
                     (T*)h, M, W, n, eps)
#define LN_N(T)                            \
  do {                                     \
    if (tpr == 64 && nc == 1) LN(T, 1, 64); \
    else if (tpr == 64) LN(T, 2, 64);      \
    else if (nc == 1) LN(T, 1, 256);       \
    else if (nc == 2) LN(T, 2, 256);       \
    else if (nc <= 4) LN(T, 4, 256);       \
    else LN(T, 8, 256);                    \
  } while (0)
  if (fp32) LN_N(float);
  else LN_N(unsigned short);
#undef LN_N
#undef LN
}

// tanh to a relative error of about 1e-6, also near 0
__device__ __forceinline__ float tanh_near(float u) {
  const float s = u * u;
  const float p =
      u + u * s *
              (-0.33333333f +
               s * (0.13333333f + s * (-0.05396825f + s * 0.02186949f)));
  return fabsf(u) < 0.3f ? p : fast_tanh(u);
}

struct ResidualArgs {
  const float* bias;
  const float* w_rms;   // null: y is added as it is
  int n;                // columns of the rms statistics
  float eps;
  const long* tokens;   // null: no table row
  float scale;
  const float* vec;
  const float *w, *b, *alpha;  // w null: h = x
  bool fresh, store;    // x starts from zeros; x changes
};

template <typename T, int NC, int TPR>
__global__ void __launch_bounds__(256)
residual_step_kernel(const T* __restrict__ y, const T* __restrict__ table,
                     float* __restrict__ x, const ResidualArgs a,
                     T* __restrict__ h, int M, int W) {
  __shared__ float scratch[4];
  const int sub = threadIdx.x % TPR;
  const int row = blockIdx.x * (256 / TPR) + threadIdx.x / TPR;
  if (row >= M) return;  // whole waves; whole blocks when TPR == 256
  float* xr = x + (long)row * W;

  float v[NC][8];
#pragma unroll
  for (int k = 0; k < NC; ++k) {
    const int c = (sub + k * TPR) * 8;
#pragma unroll
    for (int i = 0; i < 8; ++i) v[k][i] = 0.f;
    if (y != nullptr && c < W) load8<T>(y + (long)row * W + c, v[k]);
  }
  float inv = 1.f;
  if (a.w_rms != nullptr) {
    float ss = 0.f;
#pragma unroll
    for (int k = 0; k < NC; ++k)
#pragma unroll
      for (int i = 0; i < 8; ++i) ss += v[k][i] * v[k][i];
    inv = 1.f / sqrtf(row_sum<TPR>(ss, scratch) / a.n + a.eps);
  }
  const T* er =
      a.tokens != nullptr ? table + a.tokens[row] * (long)W : nullptr;
  const float alpha = a.w != nullptr ? *a.alpha : 0.f;
#pragma unroll
  for (int k = 0; k < NC; ++k) {
    const int c = (sub + k * TPR) * 8;
    if (c >= W) continue;
    float t[8];
    if (a.w_rms != nullptr) {
      load8<float>(a.w_rms + c, t);
#pragma unroll
      for (int i = 0; i < 8; ++i) v[k][i] *= inv * t[i];
    }
    if (a.bias != nullptr) {
      load8<float>(a.bias + c, t);
#pragma unroll
      for (int i = 0; i < 8; ++i) v[k][i] += t[i];
    }
    if (!a.fresh) {
      load8<float>(xr + c, t);
#pragma unroll
      for (int i = 0; i < 8; ++i) v[k][i] += t[i];
    }
    if (er != nullptr) {
      load8<T>(er + c, t);
#pragma unroll
      for (int i = 0; i < 8; ++i) v[k][i] += t[i] * a.scale;
    }
    if (a.vec != nullptr) {
      load8<float>(a.vec + c, t);
#pragma unroll
      for (int i = 0; i < 8; ++i) v[k][i] += t[i];
    }
    if (a.store) store8(xr + c, v[k]);
    if (a.w != nullptr) {
      float w[8];
      load8<float>(a.w + c, w);
      load8<float>(a.b + c, t);
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const float u = alpha * v[k][i];
        v[k][i] = (sizeof(T) == 2 ? tanh_near(u) : tanhf(u)) * w[i] + t[i];
      }
    }
    store8(h + (long)row * W + c, v[k]);
  }
}

extern "C" void launch_residual_step(
    const void* y, const void* table, float* x, const float* bias,
    const float* w_rms, int n, float eps, const long* tokens, float scale,
    const float* vec, const float* w, const float* b, const float* alpha,
    bool fresh, void* h, int M, int W, bool fp32, hipStream_t stream) {
  const ResidualArgs a{bias, w_rms, n, eps, tokens, scale, vec, w, b, alpha,
                       fresh,
                       y != nullptr || tokens != nullptr || vec != nullptr ||
                           fresh};
  const int tpr = W <= 1024 ? 64 : 256;
  const int rows = 256 / tpr;
  const dim3 grid((M + rows - 1) / rows);
  const int nc = (W / 8 + tpr - 1) / tpr;
#define RS(T, NC, TPR)                                                      \
  hipLaunchKernelGGL((residual_step_kernel<T, NC, TPR>), grid, dim3(256), 0, \
                     stream, (const T*)y, (const T*)table, x, a, (T*)h, M, W)
#define RS_N(T)                            \
  do {                                     \
    if (tpr == 64 && nc == 1) RS(T, 1, 64); \
    else if (tpr == 64) RS(T, 2, 64);      \
    else if (nc == 1) RS(T, 1, 256);       \
    else if (nc == 2) RS(T, 2, 256);       \
    else if (nc <= 4) RS(T, 4, 256);       \
    else RS(T, 8, 256);                    \
  } while (0)
  if (fp32) RS_N(float);
  else RS_N(unsigned short);
#undef RS_N
#undef RS
}
