#include "common.h"

// ---- cos and sin of every row's position ------------------------------------
__global__ void __launch_bounds__(256)
rotation_table_kernel(const int* __restrict__ ctx,
                      const double* __restrict__ freq, float mult,
                      float* __restrict__ table, int M, int pairs) {
  const long i = (long)blockIdx.x * 256 + threadIdx.x;
  if (i >= (long)M * pairs) return;
  const double a = (double)max(ctx[i / pairs] - 1, 0) * freq[i % pairs];
  // to [-pi, pi] before the angle becomes 32 bits wide
  const double turns = a * 0.15915494309189535;
  float s, c;
  sincosf((float)((turns - rint(turns)) * 6.283185307179586), &s, &c);
  table[i * 2] = c * mult;
  table[i * 2 + 1] = s * mult;
}

extern "C" void launch_rotation_table(const int* ctx, const double* freq,
                                      float mult, float* table, int M,
                                      int pairs, hipStream_t stream) {
  hipLaunchKernelGGL(rotation_table_kernel,
                     dim3(((long)M * pairs + 255) / 256), dim3(256), 0,
                     stream, ctx, freq, mult, table, M, pairs);
}
