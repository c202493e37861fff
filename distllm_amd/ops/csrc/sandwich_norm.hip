// RMS norms of a "sandwich" decoder layer (a norm before and after each
// sublayer) on an fp32 residual stream.
//
//   embed_norm:    x = E[token];            h = rms(x) * w_next
//   post_norm_add: x += rms(y) * w_post;    h = rms(x) * w_next
//
// One launch per sublayer boundary: the sublayer output y is normed and
// added and the next sublayer's input is produced while the row is still
// in registers. Statistics are over the first n columns; rows are padded
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
