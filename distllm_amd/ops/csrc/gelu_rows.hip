// out = gelu(z) * e, e being a part of a table's row (gelu_rows.h); columns
// of z behind that part become zeros.
#include "common.h"
#include "gelu_rows.h"

// a thread: eight columns; WHOLE: the part is made of whole eights
template <typename T, bool WHOLE>
__global__ void __launch_bounds__(256)
gelu_rows_kernel(const T* __restrict__ z, T* __restrict__ out, long M, int N,
                 const RowsArgs r) {
  const long i = (long)blockIdx.x * 256 + threadIdx.x;
  const int vec = N / 8;
  const long row = i / vec;
  const int col = (int)(i % vec) * 8;
  if (row >= M) return;
  float x[8], e[8];
  load8<T>(z + row * N + col, x);
  const T* t = (const T*)r.table + r.tokens[row] * r.ld + r.col0 + col;
  if (WHOLE) {
    if (col < r.n) load8<T>(t, e);
  } else {
#pragma unroll
    for (int k = 0; k < 8; ++k) e[k] = col + k < r.n ? to_f(t[k]) : 0.f;
  }
#pragma unroll
  for (int k = 0; k < 8; ++k)
    x[k] = col + k < r.n
               ? (sizeof(T) == 2 ? fast_gelu(x[k]) : gelu_exact(x[k])) * e[k]
               : 0.f;
  store8(out + row * N + col, x);
}

extern "C" void launch_gelu_rows(const void* z, void* out, long M, int N,
                                 const RowsArgs* r, bool fp32,
                                 hipStream_t stream) {
  const dim3 grid((M * (N / 8) + 255) / 256);
  const bool whole = r->n % 8 == 0 && r->col0 % 8 == 0 && r->ld % 8 == 0;
#define GR(T, W)                                                            \
  hipLaunchKernelGGL((gelu_rows_kernel<T, W>), grid, dim3(256), 0, stream,  \
                     (const T*)z, (T*)out, M, N, *r)
  if (fp32 && whole) GR(float, true);
  else if (fp32) GR(float, false);
  else if (whole) GR(unsigned short, true);
  else GR(unsigned short, false);
#undef GR
}
