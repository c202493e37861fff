// xIELU on a product's output: for z > 0, ap z^2 + z / 2; for z <= 0,
// (an + 1/2) (exp(z) - 1 - z) + z / 2, with ap, an the softplus of the two
// raw numbers act[0], act[1].
#include "common.h"

template <typename T>
__global__ void __launch_bounds__(256)
xielu_kernel(const T* __restrict__ z, const float* __restrict__ act,
             T* __restrict__ out, long n8) {
  const float ap = softplus_exact(act[0]), an = softplus_exact(act[1]);
  const long stride = (long)gridDim.x * 256;
  for (long i = (long)blockIdx.x * 256 + threadIdx.x; i < n8; i += stride) {
    float v[8];
    load8<T>(z + i * 8, v);
#pragma unroll
    for (int k = 0; k < 8; ++k)
      v[k] = sizeof(T) == 2 ? xielu(v[k], ap, an) : xielu_exact(v[k], ap, an);
    store8(out + i * 8, v);
  }
}

extern "C" void launch_xielu(const void* z, const float* act, void* out,
                             long n, bool fp32, hipStream_t stream) {
  const long n8 = n / 8;
  const int blocks = (int)min((n8 + 255) / 256, (long)8192);
#define XI(T)                                                              \
  hipLaunchKernelGGL((xielu_kernel<T>), dim3(blocks), dim3(256), 0, stream, \
                     (const T*)z, act, (T*)out, n8)
  if (fp32) XI(float);
  else XI(unsigned short);
#undef XI
}
