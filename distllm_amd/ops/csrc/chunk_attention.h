// Softmax attention over paged keys and values. What a score is and what
// becomes of the output is a policy of the kernels:
//   CappedScore  s_ij = softcap * tanh(scale * q_i . k_j / softcap)
//                       - r1 * ln(1 + r2 (i-j)), output * sigmoid(gate)
//   SinkScore    s_ij = scale * q_i . k_j, exp(sink) of the head in the
//                softmax's denominator, output * a constant
// for j <= i in the same chunk (i / chunk == j / chunk).
//
// Key pages are [num_blocks, G, PBLK, DK], value pages are transposed:
// [num_blocks, G, DV, PBLK], so that both are read from memory in the
// operand order of the MFMA products. block_table [S, max_blocks] int32.
// A row of the output holds DV numbers per head, rows are ld_out apart.
#pragma once
#include "common.h"

#define PBLK 16  // tokens per cache block
#define LOG2E 1.4426950408889634f

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;

// A policy has, for a head: score() in units of log2 and its form on library
// functions exact_score(); for the end of a row: the sink, if there is one
// (-inf: none), and finish() for N consecutive output numbers.
struct CappedScore {
  float scale, softcap;
  float c_in, c_out;  // 2 scale / softcap * log2(e), softcap * log2(e)
  const float* dist;  // r1 [H], r2 [H]
  const void* gate;
  int ld_gate;

  struct Head {
    float r1, r2;
  };
  __device__ __forceinline__ Head head(int h, int H) const {
    return {dist[h], dist[H + h]};
  }
  // distance >= 0 for visible keys
  __device__ __forceinline__ float score(float s, const Head& h,
                                         float distance) const {
    const float e = __builtin_amdgcn_exp2f(s * c_in);
    const float t = c_out - 2.f * c_out * fast_rcp(e + 1.f);
    return t - h.r1 * __builtin_amdgcn_logf(fmaf(h.r2, distance, 1.f));
  }
  __device__ __forceinline__ float exact_score(float s, const Head& h,
                                               float distance) const {
    return softcap * tanhf(s * scale / softcap) -
           h.r1 * log1pf(h.r2 * distance);
  }
  static constexpr bool SINK = false;
  __device__ __forceinline__ float sink_of(int) const { return -INFINITY; }
  // N numbers of a head from column c on
  template <typename T, int N>
  __device__ __forceinline__ void finish(long row, long head, int DV, int c,
                                         float* v) const {
    const T* g = (const T*)gate + row * ld_gate + head * DV + c;
    if constexpr (N == 4 && sizeof(T) == 2) {
      const s16x4 gv = *reinterpret_cast<const s16x4*>(g);
#pragma unroll
      for (int i = 0; i < 4; ++i)
        v[i] *= fast_rcp(1.f + fast_exp(-bf2f((unsigned short)gv[i])));
    } else {
#pragma unroll
      for (int i = 0; i < N; ++i) v[i] *= sigmoid_exact(to_f(g[i]));
    }
  }
};

struct SinkScore {
  float scale;
  float c;  // scale * log2(e)
  const float* sink;
  float out_scale;

  struct Head {};
  __device__ __forceinline__ Head head(int, int) const { return {}; }
  __device__ __forceinline__ float score(float s, const Head&, float) const {
    return s * c;
  }
  __device__ __forceinline__ float exact_score(float s, const Head&,
                                               float) const {
    return s * scale;
  }
  static constexpr bool SINK = true;
  __device__ __forceinline__ float sink_of(int h) const { return sink[h]; }
  template <typename T, int N>
  __device__ __forceinline__ void finish(long, long, int, int,
                                         float* v) const {
#pragma unroll
    for (int i = 0; i < N; ++i) v[i] *= out_scale;
  }
};

// Factor on an output whose weights exp2(s - m) sum to l; with a sink, its
// weight is part of the sum. 0 for a row that sees nothing.
template <typename P>
__device__ __forceinline__ float softmax_factor(const P& p, int head, float m,
                                                float l) {
  if (!(l > 0.f)) return 0.f;
  if (!P::SINK) return 1.f / l;
  const float s = p.sink_of(head) * LOG2E;
  const float top = fmaxf(m, s);
  const float a = __builtin_amdgcn_exp2f(m - top);
  return a / (l * a + __builtin_amdgcn_exp2f(s - top));
}
