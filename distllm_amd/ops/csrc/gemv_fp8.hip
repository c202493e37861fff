// W8A16 projection GEMV for the interactive-decode regime:
//   out[M, N] = x[M, K] (bf16) @ (W_q[N, K] (fp8 e4m3) * scale[N])^T
// with optional bf16 bias. M <= 8 (per-token decode batches).
//
// The M=1 decode step is weight-stream bound (profiles/RESULTS.md "B=1
// interactive decode"): fp8 weights halve the HBM bytes per step, and
// a GEMV shape (one wave per output column, lanes striding K in
// 16-byte chunks, fully coalesced) wastes none of the stream on the
// MFMA tiling a 1-row GEMM can't fill. Scales are per output channel
// and applied after the fp32 dot: dot(w_q*s, x) == s * dot(w_q, x), so
// quantization only rounds the weights, never the accumulation.
// Reference anchor: the vLLM latency role the reference delegated
// (distllm/generate/generators/vllm_backend.py:62-93).
#include <hip/hip_fp8.h>

#include "common.h"

#define GV_MAXM 8

__device__ __forceinline__ float gv_fp8(unsigned char u) {
  __hip_fp8_e4m3 v;
  v.__x = u;
  return float(v);
}

__global__ void __launch_bounds__(512)
gemv_fp8_kernel(const unsigned short* __restrict__ X,
                const unsigned char* __restrict__ W,
                const float* __restrict__ scale,
                const unsigned short* __restrict__ bias,
                unsigned short* __restrict__ OUT, int M, int N, long K) {
  const int lane = threadIdx.x & (WAVE - 1);
  const int wid = threadIdx.x >> 6;
  const int n = blockIdx.x * 8 + wid;  // one wave per output column
  if (n >= N) return;
  const unsigned char* w = W + (long)n * K;
  float acc[GV_MAXM];
#pragma unroll
  for (int m = 0; m < GV_MAXM; ++m) acc[m] = 0.f;

  const int niter = (int)((K + 1023) >> 10);  // K % 16 enforced host-side
  for (int it = 0; it < niter; ++it) {
    const long off = (long)it * 1024 + lane * 16;  // fp8-element offset
    if (off >= K) break;  // tail chunk: inactive lanes
    const uint4 wb = *reinterpret_cast<const uint4*>(w + off);
    const unsigned char* wp =
        reinterpret_cast<const unsigned char*>(&wb);
    float wf[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) wf[i] = gv_fp8(wp[i]);
    for (int m = 0; m < M; ++m) {
      const unsigned short* xr = X + (long)m * K + off;
      const uint4 xa = *reinterpret_cast<const uint4*>(xr);
      const uint4 xb = *reinterpret_cast<const uint4*>(xr + 8);
      const unsigned short* xp =
          reinterpret_cast<const unsigned short*>(&xa);
      const unsigned short* xq =
          reinterpret_cast<const unsigned short*>(&xb);
      float s = 0.f;
#pragma unroll
      for (int i = 0; i < 8; ++i) s += wf[i] * bf2f(xp[i]);
#pragma unroll
      for (int i = 0; i < 8; ++i) s += wf[8 + i] * bf2f(xq[i]);
      acc[m] += s;
    }
  }
  const float sc = scale[n];
  for (int m = 0; m < M; ++m) {
    float v = wave_reduce_sum(acc[m]) * sc;
    if (lane == 0) {
      if (bias != nullptr) v += bf2f(bias[n]);
      OUT[(long)m * N + n] = f2bf(v);
    }
  }
}

extern "C" void launch_gemv_fp8(const void* X, const void* W,
                                const float* scale, const void* bias,
                                void* out, int M, int N, long K,
                                hipStream_t stream) {
  const int grid = (N + 7) / 8;
  hipLaunchKernelGGL(gemv_fp8_kernel, dim3(grid), dim3(512), 0, stream,
                     (const unsigned short*)X, (const unsigned char*)W,
                     scale, (const unsigned short*)bias,
                     (unsigned short*)out, M, N, K);
}
