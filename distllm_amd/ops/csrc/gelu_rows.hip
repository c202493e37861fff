// out = gelu(z) * e, e being a part of a table's row (gelu_rows.h); columns
// of z behind that part become zeros.
#include "common.h"
#include "gelu_rows.h"

template <typename T>
__global__ void __launch_bounds__(256)
gelu_rows_kernel(const T* __restrict__ z, T* __restrict__ out, long M, int N,
                 const RowsArgs r) {
  const long i = (long)blockIdx.x * 256 + threadIdx.x;
  if (i >= M * N) return;
  const long row = i / N;
  const int col = (int)(i % N);
  float v = 0.f;
  if (col < r.n) {
    const float x = to_f(z[i]);
    v = (sizeof(T) == 2 ? fast_gelu(x) : gelu_exact(x)) *
        to_f(((const T*)r.table)[r.tokens[row] * r.ld + r.col0 + col]);
  }
  from_f(out + i, v);
}

extern "C" void launch_gelu_rows(const void* z, void* out, long M, int N,
                                 const RowsArgs* r, bool fp32,
                                 hipStream_t stream) {
  const dim3 grid((M * N + 255) / 256);
  if (fp32)
    hipLaunchKernelGGL(gelu_rows_kernel<float>, grid, dim3(256), 0, stream,
                       (const float*)z, (float*)out, M, N, *r);
  else
    hipLaunchKernelGGL(gelu_rows_kernel<unsigned short>, grid, dim3(256), 0,
                       stream, (const unsigned short*)z, (unsigned short*)out,
                       M, N, *r);
}
