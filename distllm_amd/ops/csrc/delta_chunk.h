// Shared by the chunked forms of the delta rule: sizes, the fp32 product and
// the triangular system of a chunk.
#pragma once
#include "common.h"

#define CH 32        // rows of a chunk
#define TROW 36      // padded LDS row of a chunk x chunk matrix

extern __shared__ __attribute__((aligned(16))) char smem[];

// Operands of the 16 x 16 x 4 product: lane group g = lane / 16 holds inner
// index 4 j + g for step j as the instruction has it; here step r of a block
// of 16 takes inner indices g * 4 + r instead, which lets a lane read both
// operands as float4 and lets an accumulator (rows g * 4 + r) be the right
// operand of the next product as it is.
__device__ __forceinline__ f32x4 mfma4(float a, float b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

// Column j of (I + A)^-1, A strictly lower triangular in LDS.
__device__ __forceinline__ void inverse_column(const float* A, int j,
                                               float* x) {
#pragma unroll
  for (int i = 0; i < CH; ++i) {
    float v = i == j ? 1.f : 0.f;
#pragma unroll
    for (int s4 = 0; s4 < i; s4 += 4) {
      const f32x4 a = *reinterpret_cast<const f32x4*>(A + i * TROW + s4);
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (s4 + e < i) v -= a[e] * x[s4 + e];
    }
    x[i] = v;
  }
}

extern "C" void launch_delta_norm(const float* o, const void* gate,
                                  int ld_gate, const float* o_norm,
                                  float out_scale, void* y, long ld_y, int M,
                                  int H, int vp, int vdim, float eps,
                                  int max_rows, const int* seg_rows,
                                  const int* row_seq, const int* ctx,
                                  bool sigmoid, hipStream_t stream);
