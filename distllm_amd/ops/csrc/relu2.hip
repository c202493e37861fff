// relu(z)^2 on a product's output.
#include "common.h"

template <typename T>
__global__ void __launch_bounds__(256)
relu2_kernel(const T* __restrict__ z, T* __restrict__ out, long n8) {
  const long stride = (long)gridDim.x * 256;
  for (long i = (long)blockIdx.x * 256 + threadIdx.x; i < n8; i += stride) {
    float v[8];
    load8<T>(z + i * 8, v);
#pragma unroll
    for (int k = 0; k < 8; ++k) v[k] = relu2(v[k]);
    store8(out + i * 8, v);
  }
}

extern "C" void launch_relu2(const void* z, void* out, long n, bool fp32,
                             hipStream_t stream) {
  const long n8 = n / 8;
  const int blocks = (int)min((n8 + 255) / 256, (long)8192);
#define R2(T)                                                              \
  hipLaunchKernelGGL((relu2_kernel<T>), dim3(blocks), dim3(256), 0, stream, \
                     (const T*)z, (T*)out, n8)
  if (fp32) R2(float);
  else R2(unsigned short);
#undef R2
}
