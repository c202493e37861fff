// Grouped products of routed experts for many rows per expert (see
// experts.hip for the plan): 256 x 256 x 64 tiles on the deep-pipelined
// main loop of gemm16.hip, with gathered rows and silu(gate) * up or
// relu(up)^2, or scattered rows. N % 256 == 0, K % 128 == 0.
#include "gemm16_core.h"

template <int UNIT>
__global__ void __launch_bounds__(512, 2)
expert_gemm16_kernel(const unsigned short* __restrict__ x,
                     const unsigned short* __restrict__ W,
                     unsigned short* __restrict__ out,
                     const int* __restrict__ perm,
                     const int* __restrict__ tiles,
                     const int* __restrict__ ntiles, int N, int K, int top) {
  constexpr bool GLU = UNIT == 1, UP = UNIT != 0;
  const int ncol = N / G16_BN;
  // contiguous runs of (tile, column block) per XCD, columns fastest: they
  // share the rows of x
  const int total = *ntiles * ncol;
  const int per = (total + 7) / 8;
  const int j8 = blockIdx.x / 8;
  const int bid = blockIdx.x % 8 * per + j8;
  if (j8 >= per || bid >= total) return;
  const int* tile = tiles + (long)(bid / ncol) * 4;
  const int e = tile[0], s0 = tile[1], cnt = tile[2];
  const int n0 = bid % ncol * G16_BN;
  const int lane = threadIdx.x & 63;
  const int wid = threadIdx.x >> 6;
  const int mw = wid >> 2, nw = wid & 3;

  // this lane's row of its two pieces of each half of A
  const int r_in = lane >> 3, c_src = ((lane & 7) ^ r_in) * 8;
  const unsigned short* xs[2][2];
#pragma unroll
  for (int half = 0; half < 2; ++half)
#pragma unroll
    for (int pp = 0; pp < 2; ++pp) {
      const int r = half * 128 + (wid * 2 + pp) * 8 + r_in;
      const int s = s0 + min(r, cnt - 1);
      xs[half][pp] = x + (long)(UP ? perm[s] / top : s) * K + c_src;
    }
  const unsigned short* wb =
      W + ((long)e * N + n0 + wid * 16 + r_in) * K + c_src;

  f32x4 acc[8][4];
  g16_mainloop(
      [&](long k0, int buf, int half) {
#pragma unroll
        for (int pp = 0; pp < 2; ++pp)
          g16_stage(xs[half][pp] + k0, 0, buf, half, pp, wid, lane);
      },
      [&](long k0, int buf, int half) {
#pragma unroll
        for (int pp = 0; pp < 2; ++pp)
          g16_stage(wb + (long)(half * 128 + pp * 8) * K + k0, 1, buf, half,
                    pp, wid, lane);
      },
      K, lane, mw, nw, acc);

  // per-wave transpose slab, 16 rows at a time, 16-byte stores
  constexpr int SLAB_W = 68;
  float* slab = reinterpret_cast<float*>(smem16) + wid * 16 * SLAB_W;
#pragma unroll
  for (int rd = 0; rd < 8; ++rd) {
    const int row0 = mw * 128 + rd * 16;
    if (row0 >= cnt) break;
#pragma unroll
    for (int ni = 0; ni < 4; ++ni)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        slab[((lane >> 4) * 4 + r) * SLAB_W + ni * 16 + (lane & 15)] =
            acc[rd][ni][r];
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    if (GLU) {
      const int r = lane >> 2, c8 = lane & 3;  // 32 columns of output
      const float* p = slab + r * SLAB_W + (c8 >> 1) * 32 + (c8 & 1) * 8;
      float o[8];
#pragma unroll
      for (int i = 0; i < 8; ++i) o[i] = silu(p[i]) * p[16 + i];
      if (row0 + r < cnt)
        store8(out + (long)(s0 + row0 + r) * (N / 2) + n0 / 2 + nw * 32 +
                   c8 * 8,
               o);
    } else {
#pragma unroll
      for (int p = 0; p < 2; ++p) {
        const int r = p * 8 + (lane >> 3), c8 = lane & 7;
        float o[8];
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          o[i] = slab[r * SLAB_W + c8 * 8 + i];
          if (UNIT == 2) o[i] = relu2(o[i]);
        }
        if (row0 + r < cnt) {
          const long row = UP ? s0 + row0 + r : perm[s0 + row0 + r];
          store8(out + row * N + n0 + nw * 64 + c8 * 8, o);
        }
      }
    }
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  }
}

extern "C" bool expert_gemm16_covers(int N, int K) {
  return N % G16_BN == 0 && K % 128 == 0;
}

extern "C" void launch_expert_gemm16(const void* x, const void* W, void* out,
                                     const int* perm, const int* tiles,
                                     const int* ntiles, int max_tiles, int N,
                                     int K, int top, int unit,
                                     hipStream_t stream) {
  typedef unsigned short u16;
  const long wgs = ((long)max_tiles * (N / G16_BN) + 7) / 8 * 8;
#define EG(GL)                                                               \
  hipLaunchKernelGGL((expert_gemm16_kernel<GL>), dim3(wgs), dim3(512),       \
                     G16_LDS, stream, (const u16*)x, (const u16*)W,          \
                     (u16*)out, perm, tiles, ntiles, N, K, top)
  if (unit == 1) EG(1);
  else if (unit == 2) EG(2);
  else EG(0);
#undef EG
}
