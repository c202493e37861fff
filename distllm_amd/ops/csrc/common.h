// Common device helpers for distllm-amd CDNA4 (gfx950) kernels.
// Hardware model per /opt/skills/guides/cdna_hip_programming.md:
//   wave = 64 lanes, 4 SIMD-32/CU, 160 KiB LDS/CU, MFMA bf16 K=16/32.
#pragma once

#include <hip/hip_runtime.h>
#include <hip/hip_bf16.h>
#include <stdint.h>

#define WAVE 64

// ---- vector types -------------------------------------------------------
typedef __attribute__((ext_vector_type(2))) float  f32x2;
typedef __attribute__((ext_vector_type(4))) float  f32x4;
typedef __attribute__((ext_vector_type(16))) float f32x16;
typedef __attribute__((ext_vector_type(4))) short  s16x4;
typedef __attribute__((ext_vector_type(8))) short  s16x8;
typedef __attribute__((ext_vector_type(2))) int    i32x2;
typedef __attribute__((ext_vector_type(4))) int    i32x4;

// bf16 <-> f32 (scalar); use __hip_bfloat16 for storage only.
__device__ __forceinline__ float bf2f(unsigned short u) {
  union { float f; unsigned int i; } c;
  c.i = ((unsigned int)u) << 16;
  return c.f;
}
__device__ __forceinline__ unsigned short f2bf(float f) {
  // hardware RTNE converter (v_cvt_*_bf16_f32 on gfx950) — far cheaper
  // than the 5-op manual rounding sequence.
  __bf16 h = (__bf16)f;
  union { __bf16 h; unsigned short u; } c;
  c.h = h;
  return c.u;
}

// Convert 8 bf16 (s16x8) to 8 f32.
__device__ __forceinline__ void bf8_to_f32(const s16x8 v, float* out) {
#pragma unroll
  for (int i = 0; i < 8; ++i) out[i] = bf2f((unsigned short)v[i]);
}

// ---- wave reductions (64-wide) -----------------------------------------
__device__ __forceinline__ float wave_reduce_sum(float v) {
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) v += __shfl_xor(v, off, WAVE);
  return v;
}
__device__ __forceinline__ float wave_reduce_max(float v) {
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) v = fmaxf(v, __shfl_xor(v, off, WAVE));
  return v;
}

// Order one wave's LDS accesses across its lanes.
__device__ __forceinline__ void wave_sync() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
  __builtin_amdgcn_wave_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
}

// Workgroups go round the eight XCDs one by one: number b of n such that
// each XCD (an L2 cache of its own) gets a contiguous run of numbers.
__device__ __forceinline__ int xcd_run(int b, int n) {
  const int per = n / 8, rem = n % 8, xcd = b % 8;
  return (xcd < rem ? xcd * (per + 1) : rem * (per + 1) + (xcd - rem) * per) +
         b / 8;
}

// Block-level reduce across NW waves using LDS scratch (NW <= 16).
template <int NW>
__device__ __forceinline__ float block_reduce_sum(float v, float* lds_scratch) {
  const int lane = threadIdx.x & (WAVE - 1);
  const int wid = threadIdx.x / WAVE;
  v = wave_reduce_sum(v);
  if (lane == 0) lds_scratch[wid] = v;
  __syncthreads();
  float r = (lane < NW) ? lds_scratch[lane] : 0.f;
  r = wave_reduce_sum(r);
  // broadcast via readfirstlane semantics: all lanes of wave 0 now agree
  if (threadIdx.x == 0) lds_scratch[0] = r;
  __syncthreads();
  float out = lds_scratch[0];
  __syncthreads();
  return out;
}

#define HIP_CHECK_KERNEL()                                                    \
  do {                                                                        \
    hipError_t e = hipGetLastError();                                         \
    if (e != hipSuccess) {                                                    \
      printf("HIP kernel launch error: %s\n", hipGetErrorString(e));          \
    }                                                                         \
  } while (0)

// Branch-free transcendentals on the native v_exp_f32 / v_rcp_f32
// instructions. libm tanhf/erff/expf compile to branchy range-checked
// slow paths (one s_and_saveexec waterfall per element — measured 37%
// of a fused-GELU GEMM's time); these stay straight-line VALU.
__device__ __forceinline__ float fast_exp(float x) {
  return __builtin_amdgcn_exp2f(x * 1.4426950408889634f);
}
__device__ __forceinline__ float fast_rcp(float x) {
  return __builtin_amdgcn_rcpf(x);  // ~1 ulp: plenty for bf16 outputs
}
__device__ __forceinline__ float fast_tanh(float u) {
  // 1 - 2/(e^{2u}+1); exp2 under/overflow saturates to +-1 gracefully
  const float e = __builtin_amdgcn_exp2f(u * 2.885390081777927f);
  return 1.f - 2.f * fast_rcp(e + 1.f);
}
__device__ __forceinline__ float fast_erf(float z) {
  // Abramowitz-Stegun 7.1.26 (max abs err 1.5e-7), branch-free
  const float a = fabsf(z);
  const float t = fast_rcp(fmaf(0.3275911f, a, 1.f));
  float p = fmaf(1.061405429f, t, -1.453152027f);
  p = fmaf(p, t, 1.421413741f);
  p = fmaf(p, t, -0.284496736f);
  p = fmaf(p, t, 0.254829592f);
  const float y = 1.f - p * t * fast_exp(-a * a);
  return copysignf(y, z);
}
__device__ __forceinline__ float fast_gelu(float x) {
  // tanh approximation (matches BERT/HF "gelu_new" semantics)
  const float k0 = 0.7978845608028654f;  // sqrt(2/pi)
  const float k1 = 0.044715f;
  return 0.5f * x * (1.f + fast_tanh(k0 * (x + k1 * x * x * x)));
}
// the same on library functions
__device__ __forceinline__ float gelu_exact(float x) {
  return 0.5f * x *
         (1.f + tanhf(0.7978845608028654f * (x + 0.044715f * x * x * x)));
}
__device__ __forceinline__ float gelu_erf(float x) {
  return 0.5f * x * (1.f + fast_erf(x * 0.70710678118654752f));
}
__device__ __forceinline__ float silu(float x) {
  return x * fast_rcp(1.f + fast_exp(-x));
}
// Clamped gated unit (see clamped_glu.hip): the fast form for 16-bit
// outputs and the form on library functions for 32-bit ones.
__device__ __forceinline__ float clamped_glu(float gate, float up,
                                             float limit, float alpha,
                                             float shift) {
  const float g = fminf(gate, limit);
  const float u = fminf(fmaxf(up, -limit), limit);
  return g * fast_rcp(1.f + fast_exp(-alpha * g)) * (u + shift);
}
__device__ __forceinline__ float clamped_glu_exact(float gate, float up,
                                                   float limit, float alpha,
                                                   float shift) {
  const float g = fminf(gate, limit);
  const float u = fminf(fmaxf(up, -limit), limit);
  return g / (1.f + expf(-alpha * g)) * (u + shift);
}

// xIELU with ap = softplus(p), an = softplus(q): the fast form for 16-bit
// outputs and the form on library functions for 32-bit ones.
__device__ __forceinline__ float softplus_exact(float z) {
  return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z)));
}
__device__ __forceinline__ float xielu(float z, float ap, float an) {
  const float neg = (0.5f + an) * (fast_exp(fminf(z, 0.f)) - 1.f - z);
  return 0.5f * z + (z > 0.f ? ap * z * z : neg);
}
__device__ __forceinline__ float xielu_exact(float z, float ap, float an) {
  const float neg = (0.5f + an) * (expm1f(fminf(z, 0.f)) - z);
  return 0.5f * z + (z > 0.f ? ap * z * z : neg);
}
__device__ __forceinline__ float relu2(float z) {
  const float r = fmaxf(z, 0.f);
  return r * r;
}
__device__ __forceinline__ float sigmoid_exact(float z) {
  return 1.f / (1.f + expf(-z));
}

// Scalars of the two tensor types as fp32.
__device__ __forceinline__ float to_f(unsigned short v) { return bf2f(v); }
__device__ __forceinline__ float to_f(float v) { return v; }
__device__ __forceinline__ void from_f(unsigned short* p, float v) {
  *p = f2bf(v);
}
__device__ __forceinline__ void from_f(float* p, float v) { *p = v; }

// Eight consecutive numbers of a bf16 or fp32 array, as fp32.
template <typename T>
__device__ __forceinline__ void load8(const T* p, float* f);
template <>
__device__ __forceinline__ void load8<unsigned short>(const unsigned short* p,
                                                      float* f) {
  bf8_to_f32(*reinterpret_cast<const s16x8*>(p), f);
}
template <>
__device__ __forceinline__ void load8<float>(const float* p, float* f) {
  const f32x4 a = *reinterpret_cast<const f32x4*>(p);
  const f32x4 b = *reinterpret_cast<const f32x4*>(p + 4);
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    f[i] = a[i];
    f[4 + i] = b[i];
  }
}
__device__ __forceinline__ void store8(unsigned short* p, const float* f) {
  s16x8 v;
#pragma unroll
  for (int i = 0; i < 8; ++i) v[i] = (short)f2bf(f[i]);
  *reinterpret_cast<s16x8*>(p) = v;
}
__device__ __forceinline__ void store8(float* p, const float* f) {
  f32x4 a, b;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    a[i] = f[i];
    b[i] = f[4 + i];
  }
  *reinterpret_cast<f32x4*>(p) = a;
  *reinterpret_cast<f32x4*>(p + 4) = b;
}
