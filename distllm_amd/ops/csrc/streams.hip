// Boundary of several fp32 residual streams x_1 .. x_S (see models/streams.py):
//   x_t <- sum_s mix[s, t] x_s + out[t] y     (with a sublayer's output y)
//   h    = rms(sum_s read[s] x_s) * w         (read null: the plain sum)
// in one launch, y being a row or a weighted sum of the rows of routed and
// shared experts. Statistics are over the first n columns; rows are padded
// with zeros to W columns. With tokens, every old stream is the token's row
// of the table. T is the type of y, h and the table.
#include "common.h"

// sum over the TPR threads (one or four waves) that share a row
template <int TPR>
__device__ __forceinline__ float row_sum(float v, float* scratch) {
  v = wave_reduce_sum(v);
  if (TPR == 64) return v;
  if ((threadIdx.x & 63) == 0) scratch[threadIdx.x >> 6] = v;
  __syncthreads();
  return scratch[0] + scratch[1] + scratch[2] + scratch[3];
}

template <typename T>
struct StreamArgs {
  const T* y;            // null: nothing is written
  const T* shared;
  const float* mix;      // weights of y's rows, then of shared
  int top;
  const long* tokens;    // null: old streams are x
  const T* table;
  const float* writes;   // out [S], mix [S, S] (from, to)
  const float* read;
  const float* w;
  int n;
  float eps;
  bool store;
};

// CAP: number of streams up to 4, else the most there may be
template <typename T, int CAP, int NC, int TPR>
__global__ void __launch_bounds__(256)
stream_step_kernel(const StreamArgs<T> a, float* __restrict__ x,
                   T* __restrict__ h, int M, int streams, int W) {
  __shared__ float scratch[4];
  const int S = CAP <= 4 ? CAP : streams;
  const int sub = threadIdx.x % TPR;
  const int row = blockIdx.x * (256 / TPR) + threadIdx.x / TPR;
  if (row >= M) return;  // whole waves; whole blocks when TPR == 256
  float* xr = x + (long)row * S * W;
  const T* er =
      a.tokens != nullptr ? a.table + a.tokens[row] * (long)W : nullptr;
  const int cols = a.top + (a.shared != nullptr);
  const float* mixr = a.mix != nullptr ? a.mix + (long)row * cols : nullptr;

  float u[NC][8];
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < NC; ++k) {
    const int c = (sub + k * TPR) * 8;
#pragma unroll
    for (int i = 0; i < 8; ++i) u[k][i] = 0.f;
    if (c >= W) continue;
    float old[CAP][8];
#pragma unroll
    for (int s = 0; s < CAP; ++s) {
      if (s < S) {
        if (er == nullptr) load8<float>(xr + (long)s * W + c, old[s]);
        else if (s == 0) load8<T>(er + c, old[0]);
        else
#pragma unroll
          for (int i = 0; i < 8; ++i) old[s][i] = old[0][i];
      }
    }
    if (a.y != nullptr) {
      float v[8];
      if (mixr == nullptr) {
        load8<T>(a.y + (long)row * W + c, v);
      } else {
#pragma unroll
        for (int i = 0; i < 8; ++i) v[i] = 0.f;
#pragma unroll 4
        for (int e = 0; e < a.top; ++e) {
          const float m = mixr[e];
          float t[8];
          load8<T>(a.y + ((long)row * a.top + e) * W + c, t);
#pragma unroll
          for (int i = 0; i < 8; ++i)  // weight 0: nothing was written there
            v[i] += m == 0.f ? 0.f : m * t[i];
        }
        if (a.shared != nullptr) {
          const float m = mixr[a.top];
          float t[8];
          load8<T>(a.shared + (long)row * W + c, t);
#pragma unroll
          for (int i = 0; i < 8; ++i) v[i] += m * t[i];
        }
      }
#pragma unroll
      for (int t = 0; t < CAP; ++t) {
        if (t < S) {
          float z[8];
          const float o = a.writes[t];
#pragma unroll
          for (int i = 0; i < 8; ++i) z[i] = o * v[i];
#pragma unroll
          for (int s = 0; s < CAP; ++s)
            if (s < S) {
              const float m = a.writes[S + s * S + t];
#pragma unroll
              for (int i = 0; i < 8; ++i) z[i] += m * old[s][i];
            }
          if (a.store) store8(xr + (long)t * W + c, z);
          const float r = a.read != nullptr ? a.read[t] : 1.f;
#pragma unroll
          for (int i = 0; i < 8; ++i) u[k][i] += r * z[i];
        }
      }
    } else {
#pragma unroll
      for (int s = 0; s < CAP; ++s)
        if (s < S) {
          const float r = a.read != nullptr ? a.read[s] : 1.f;
#pragma unroll
          for (int i = 0; i < 8; ++i) u[k][i] += r * old[s][i];
        }
    }
#pragma unroll
    for (int i = 0; i < 8; ++i) ss += u[k][i] * u[k][i];
  }
  const float inv = 1.f / sqrtf(row_sum<TPR>(ss, scratch) / a.n + a.eps);
#pragma unroll
  for (int k = 0; k < NC; ++k) {
    const int c = (sub + k * TPR) * 8;
    if (c < W) {
      float wv[8];
      load8<float>(a.w + c, wv);
#pragma unroll
      for (int i = 0; i < 8; ++i) u[k][i] *= inv * wv[i];
      store8(h + (long)row * W + c, u[k]);
    }
  }
}

extern "C" void launch_stream_step(
    const void* y, const void* shared, const float* mix, int top,
    const long* tokens, const void* table, float* x, const float* writes,
    const float* read, const float* w, int n, float eps, bool store, void* h,
    int M, int S, int W, bool fp32, hipStream_t stream) {
  const int tpr = W <= 1024 ? 64 : 256;
  const int rows = 256 / tpr;
  const dim3 grid((M + rows - 1) / rows);
  const int nc = (W / 8 + tpr - 1) / tpr;
#define ST(T, CAP, NC, TPR)                                                  \
  hipLaunchKernelGGL(                                                        \
      (stream_step_kernel<T, CAP, NC, TPR>), grid, dim3(256), 0, stream,     \
      (StreamArgs<T>{(const T*)y, (const T*)shared, mix, top, tokens,        \
                     (const T*)table, writes, read, w, n, eps, store}),      \
      x, (T*)h, M, S, W)
#define ST_N(T, CAP)                            \
  do {                                          \
    if (tpr == 64 && nc == 1) ST(T, CAP, 1, 64); \
    else if (tpr == 64) ST(T, CAP, 2, 64);      \
    else if (nc == 1) ST(T, CAP, 1, 256);       \
    else if (nc == 2) ST(T, CAP, 2, 256);       \
    else if (nc <= 4) ST(T, CAP, 4, 256);       \
    else ST(T, CAP, 8, 256);                    \
  } while (0)
#define ST_S(T)                \
  do {                         \
    if (S == 1) ST_N(T, 1);    \
    else if (S == 2) ST_N(T, 2); \
    else if (S == 3) ST_N(T, 3); \
    else if (S == 4) ST_N(T, 4); \
    else if (S <= 8) ST_N(T, 8); \
    else ST_N(T, 16);          \
  } while (0)
  if (fp32) ST_S(float);
  else ST_S(unsigned short);
#undef ST_S
#undef ST_N
#undef ST
}
