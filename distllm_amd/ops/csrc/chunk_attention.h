// Softmax attention over paged keys and values with chunk-wise visibility,
// capped scores and a logarithmic distance bias:
//   s_ij = softcap * tanh(scale * q_i . k_j / softcap) - r1 * ln(1 + r2 (i-j))
// for j <= i in the same chunk (i / chunk == j / chunk), softmax over j,
// output times sigmoid(gate).
//
// Key pages are [num_blocks, G, PBLK, DK], value pages are transposed:
// [num_blocks, G, DV, PBLK], so that both are read from memory in the
// operand order of the MFMA products. block_table [S, max_blocks] int32.
#pragma once
#include "common.h"

#define PBLK 16  // tokens per cache block
#define LOG2E 1.4426950408889634f

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;

// a score in units of log2: c_in = 2 scale / softcap * log2(e), c_out =
// softcap * log2(e). dist >= 0 for visible keys.
__device__ __forceinline__ float capped_score(float s, float c_in,
                                              float c_out, float r1, float r2,
                                              float dist) {
  const float e = __builtin_amdgcn_exp2f(s * c_in);
  const float t = c_out - 2.f * c_out * fast_rcp(e + 1.f);
  return t - r1 * __builtin_amdgcn_logf(fmaf(r2, dist, 1.f));
}
