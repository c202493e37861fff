// Gated unit with clamped halves on a packed [R, 2F] gate|up product:
//   g = min(gate, limit)            u = clamp(up, -limit, limit)
//   out = g * sigmoid(alpha * g) * (u + shift)
#include "common.h"

template <typename T>
__global__ void __launch_bounds__(256)
clamped_glu_kernel(const T* __restrict__ gu, T* __restrict__ out, long R,
                   int F, float limit, float alpha, float shift) {
  constexpr int V = 16 / sizeof(T);
  typedef __attribute__((ext_vector_type(V))) T vec;
  const long n_vec = R * F / V;
  const long stride = (long)gridDim.x * blockDim.x;
  const int fv = F / V;
  for (long v = (long)blockIdx.x * blockDim.x + threadIdx.x; v < n_vec;
       v += stride) {
    const long r = v / fv;
    const int c = (int)(v % fv);
    const T* row = gu + r * (2L * F);
    const vec gv = *reinterpret_cast<const vec*>(row + c * V);
    const vec uv = *reinterpret_cast<const vec*>(row + F + c * V);
    vec ov;
#pragma unroll
    for (int i = 0; i < V; ++i) {
      if constexpr (sizeof(T) == 2)
        ov[i] = f2bf(clamped_glu(bf2f(gv[i]), bf2f(uv[i]), limit, alpha,
                                 shift));
      else
        ov[i] = clamped_glu_exact(gv[i], uv[i], limit, alpha, shift);
    }
    *reinterpret_cast<vec*>(out + r * F + c * V) = ov;
  }
}

extern "C" void launch_clamped_glu(const void* gu, void* out, long R, int F,
                                   float limit, float alpha, float shift,
                                   bool fp32, hipStream_t stream) {
  const long n_vec = R * F / (fp32 ? 4 : 8);
  const int blocks = (int)min((n_vec + 255) / 256, (long)4096);
#define CG(T)                                                             \
  hipLaunchKernelGGL((clamped_glu_kernel<T>), dim3(blocks), dim3(256), 0, \
                     stream, (const T*)gu, (T*)out, R, F, limit, alpha, shift)
  if (fp32) CG(float);
  else CG(unsigned short);
#undef CG
}
