// Causal convolutions of a few taps over the rows of a ragged step, one per
// channel. A segment is the consecutive rows of one sequence; its slot holds
// the taps - 1 inputs before its first row. A sequence that starts in the
// step (ctx 1 in its first row) starts from zeros.
#pragma once
#include "common.h"

// rb: rows that a thread goes through. shift: every segment has one row, and
// the thread renews its channels of the convolution slot itself (else
// conv_state_kernel does).
template <typename T>
struct ConvArgs {
  const T* ab;
  int ld, M, C, taps, rb;
  const float* w;
  T* conv;
  const int *seg_row0, *seg_slot, *row_seq, *ctx;
  bool shift;
};

// input j rows before `row`, as fp32; zeros before the start
template <typename T>
__device__ __forceinline__ void conv_input(const ConvArgs<T>& a, int row,
                                           int pos, int o, const T* slot,
                                           int ch, int j, float* x) {
#pragma unroll
  for (int i = 0; i < 8; ++i) x[i] = 0.f;
  if (pos < j) return;
  load8<T>(o >= j ? a.ab + (long)(row - j) * a.ld + ch
                  : slot + (long)(a.taps - 1 + o - j) * a.C,
           x);
}

// the slot of a segment of one row takes that row's eight inputs in
template <typename T>
__device__ __forceinline__ void conv_shift(const ConvArgs<T>& a, int row,
                                           T* slot, int ch) {
  float t[8];
  for (int j = 0; j < a.taps - 2; ++j) {
    load8<T>(slot + (long)(j + 1) * a.C, t);
    store8(slot + (long)j * a.C, t);
  }
  load8<T>(a.ab + (long)row * a.ld + ch, t);
  store8(slot + (long)(a.taps - 2) * a.C, t);
}

// last taps - 1 inputs of every segment -> its slot; a thread owns a channel
template <typename T>
__global__ void __launch_bounds__(256)
conv_state_kernel(const T* __restrict__ ab, int ld, int C, int taps,
                  T* __restrict__ conv, const int* __restrict__ seg_row0,
                  const int* __restrict__ seg_rows,
                  const int* __restrict__ seg_slot,
                  const int* __restrict__ ctx) {
  const int seg = blockIdx.y;
  const int ch = blockIdx.x * 256 + threadIdx.x;
  const int n = seg_rows[seg];
  if (ch >= C || n == 0) return;
  const int row0 = seg_row0[seg];
  const bool fresh = ctx[row0] <= 1;
  T* slot = conv + (long)seg_slot[seg] * (taps - 1) * C + ch;
  for (int i = 0; i < taps - 1; ++i) {  // ascending: old entries move down
    const int o = n - (taps - 1) + i;   // offset in the segment
    T x = (T)0;
    if (o >= 0) x = ab[(long)(row0 + o) * ld + ch];
    else if (!fresh) x = slot[(long)(i + n) * C];
    slot[(long)i * C] = x;
  }
}
