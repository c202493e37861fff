// Gated delta rule of a ragged step, per head with state S [dim, vdim]:
//   S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
//
// The fused projection ab of a row holds G query heads, G key heads (dp
// numbers each), H value heads, H gate heads (vp each), then b and a of
// every head. delta_prep runs the short convolutions and makes what enters
// the recurrence, in fp32; a scan kernel runs the recurrence. A segment is
// the consecutive rows of one sequence; a sequence that starts in the step
// (ctx 1 in its first row) starts from zeros, whatever its slot holds.
#include "common.h"

extern __shared__ __attribute__((aligned(16))) char smem[];

template <typename T>
__device__ __forceinline__ float act_silu(float z) {
  if constexpr (sizeof(T) == 2) return silu(z);
  else return z * sigmoid_exact(z);
}

// ---- convolutions, unit queries and keys, decays ---------------------------
// One wave per (run of `rb` rows, unit); units: 2G query/key heads, H value
// heads, one for all scalars. A lane owns CPL channels of its head. shift:
// every segment has one row, and the wave renews its channels of the
// convolution slot itself (else conv_state_kernel does).
template <typename T, int CPL>
__device__ __forceinline__ void conv_unit(
    const T* __restrict__ ab, int ld, int M, int C, int ch0, int unit_kind,
    int unit, int G, int dp, int vp, const float* __restrict__ conv_w,
    int taps, float q_scale, float unit_eps, float* __restrict__ qk,
    T* __restrict__ v, int H, T* __restrict__ conv,
    const int* __restrict__ seg_row0, const int* __restrict__ seg_slot,
    const int* __restrict__ row_seq, const int* __restrict__ ctx, int r0,
    int rb, bool shift, int lane) {
  const int ch = ch0 + lane * CPL;
  for (int row = r0; row < min(r0 + rb, M); ++row) {
    const int pos = ctx[row] - 1;
    if (pos < 0) continue;
    const int seg = row_seq[row];
    const int o = row - seg_row0[seg];  // offset in its segment
    T* slot = conv + (long)seg_slot[seg] * (taps - 1) * C + ch;
    float z[CPL];
#pragma unroll
    for (int i = 0; i < CPL; ++i) z[i] = 0.f;
    // tap `taps - 1 - j` meets the input j rows back
    for (int j = taps - 1; j >= 0; --j) {
      if (pos - j < 0) continue;  // before the start
      const T* src = o >= j ? ab + (long)(row - j) * ld + ch
                            : slot + (long)(taps - 1 + o - j) * C;
      const float* w = conv_w + (long)(taps - 1 - j) * C + ch;
#pragma unroll
      for (int i = 0; i < CPL; ++i) z[i] += to_f(src[i]) * w[i];
    }
    if (shift) {
      for (int j = 0; j < taps - 2; ++j)
#pragma unroll
        for (int i = 0; i < CPL; ++i)
          slot[(long)j * C + i] = slot[(long)(j + 1) * C + i];
      if (taps > 1)
#pragma unroll
        for (int i = 0; i < CPL; ++i)
          slot[(long)(taps - 2) * C + i] = ab[(long)row * ld + ch + i];
    }
#pragma unroll
    for (int i = 0; i < CPL; ++i) z[i] = act_silu<T>(z[i]);
    if (unit_kind == 0) {  // query or key head
      float ss = 0.f;
#pragma unroll
      for (int i = 0; i < CPL; ++i) ss += z[i] * z[i];
      ss = wave_reduce_sum(ss);
      const float inv =
          (unit < G ? q_scale : 1.f) / sqrtf(ss + unit_eps);
      float* dst = qk + ((long)row * 2 * G + unit) * dp + lane * CPL;
#pragma unroll
      for (int i = 0; i < CPL; ++i) dst[i] = z[i] * inv;
    } else {
      T* dst = v + ((long)row * H + unit) * vp + lane * CPL;
#pragma unroll
      for (int i = 0; i < CPL; ++i) from_f(dst + i, z[i]);
    }
  }
}

template <typename T>
__global__ void __launch_bounds__(256)
delta_prep_kernel(const T* __restrict__ ab, int ld, int M, int H, int G,
                  int dp, int vp, const float* __restrict__ conv_w, int taps,
                  const float* __restrict__ decay, float q_scale,
                  float unit_eps, float* __restrict__ qk, T* __restrict__ v,
                  float* __restrict__ gb, T* __restrict__ conv,
                  const int* __restrict__ seg_row0,
                  const int* __restrict__ seg_slot,
                  const int* __restrict__ row_seq,
                  const int* __restrict__ ctx, int rb, bool shift) {
  const int lane = threadIdx.x & 63;
  const int units = 2 * G + H + 1;
  const long w = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
  const int unit = (int)(w % units);
  const int r0 = (int)(w / units) * rb;
  if (r0 >= M) return;
  const int C = 2 * G * dp + H * vp;
  if (unit == units - 1) {
    const int ba = C + H * vp;
    for (int row = r0; row < min(r0 + rb, M); ++row) {
      if (ctx[row] <= 0) continue;
      for (int h = lane; h < H; h += 64) {
        const float b = to_f(ab[(long)row * ld + ba + h]);
        const float a = to_f(ab[(long)row * ld + ba + H + h]);
        // log of the decay, and the step size
        gb[((long)row * H + h) * 2] =
            -expf(decay[h]) * softplus_exact(a + decay[H + h]);
        gb[((long)row * H + h) * 2 + 1] = sigmoid_exact(b);
      }
    }
    return;
  }
  const bool head_qk = unit < 2 * G;
  const int u = head_qk ? unit : unit - 2 * G;
  const int ch0 = head_qk ? u * dp : 2 * G * dp + u * vp;
  const int cpl = (head_qk ? dp : vp) / 64;
#define CONV(N)                                                              \
  conv_unit<T, N>(ab, ld, M, C, ch0, head_qk ? 0 : 1, u, G, dp, vp, conv_w,  \
                  taps, q_scale, unit_eps, qk, v, H, conv, seg_row0,         \
                  seg_slot, row_seq, ctx, r0, rb, shift, lane)
  if (cpl == 1) CONV(1);
  else if (cpl == 2) CONV(2);
  else CONV(4);
#undef CONV
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

extern "C" void launch_delta_prep(
    const void* ab, int ld, int M, int H, int G, int dp, int vp,
    const float* conv_w, int taps, const float* decay, float q_scale,
    float unit_eps, float* qk, void* v, float* gb, void* conv,
    const int* seg_row0, const int* seg_rows, const int* seg_slot, int nseg,
    int longest, const int* row_seq, const int* ctx, bool fp32,
    hipStream_t stream) {
  const bool shift = longest <= 1;
  const int rb = M > 2048 ? 8 : 1;
  const int C = 2 * G * dp + H * vp;
  const long waves = (long)((M + rb - 1) / rb) * (2 * G + H + 1);
#define DP(T)                                                                 \
  do {                                                                        \
    hipLaunchKernelGGL((delta_prep_kernel<T>), dim3((waves + 3) / 4),         \
                       dim3(256), 0, stream, (const T*)ab, ld, M, H, G, dp,   \
                       vp, conv_w, taps, decay, q_scale, unit_eps, qk, (T*)v, \
                       gb, (T*)conv, seg_row0, seg_slot, row_seq, ctx, rb,    \
                       shift);                                                \
    if (!shift && taps > 1)                                                   \
      hipLaunchKernelGGL((conv_state_kernel<T>),                              \
                         dim3((C + 255) / 256, nseg), dim3(256), 0, stream,   \
                         (const T*)ab, ld, C, taps, (T*)conv, seg_row0,       \
                         seg_rows, seg_slot, ctx);                            \
  } while (0)
  if (fp32) DP(float);
  else DP(unsigned short);
#undef DP
}

// ---- recurrence, token by token ---------------------------------------------
// One workgroup per (segment, head). LPC lanes share a value column, each
// with 16 entries of the state's column in registers (float4 number i of
// lane `part` is float4 i * LPC + part of the column); a thread has NCOL
// columns. The output is normed over vdim and gated in place.
template <typename T, int LPC, int NCOL>
__global__ void __launch_bounds__(1024)
delta_scan_kernel(const float* __restrict__ qk, const T* __restrict__ v,
                  const float* __restrict__ gb, const T* __restrict__ gate,
                  int ld_gate, const float* __restrict__ o_norm,
                  float* __restrict__ state, T* __restrict__ y, int H, int G,
                  int vp, int vdim, float eps,
                  const int* __restrict__ seg_row0,
                  const int* __restrict__ seg_rows,
                  const int* __restrict__ seg_slot,
                  const int* __restrict__ ctx) {
  constexpr int dp = LPC * 16;
  __shared__ float red[2][16];
  const int seg = blockIdx.x / H, head = blockIdx.x % H;
  const int n = seg_rows[seg];
  if (n == 0) return;
  const int row0 = seg_row0[seg];
  const int part = threadIdx.x % LPC;
  const int col0 = threadIdx.x / LPC, cstep = blockDim.x / LPC;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int nwave = blockDim.x >> 6;
  const int kvh = head / (H / G);
  float* st = state + ((long)seg_slot[seg] * H + head) * vp * dp + part * 4;

  float S[NCOL][16];
  const bool fresh = ctx[row0] <= 1;
#pragma unroll
  for (int c = 0; c < NCOL; ++c)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      f32x4 x = {0.f, 0.f, 0.f, 0.f};
      if (!fresh)
        x = *reinterpret_cast<const f32x4*>(
            st + (long)(col0 + c * cstep) * dp + i * LPC * 4);
#pragma unroll
      for (int e = 0; e < 4; ++e) S[c][i * 4 + e] = x[e];
    }
  float w[NCOL];
#pragma unroll
  for (int c = 0; c < NCOL; ++c) w[c] = o_norm[col0 + c * cstep];

  for (int t = 0; t < n; ++t) {
    const long row = row0 + t;
    const float* qr = qk + (row * 2 * G + kvh) * dp + part * 4;
    const float* kr = qr + (long)G * dp;
    float q[16], k[16];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const f32x4 a = *reinterpret_cast<const f32x4*>(qr + i * LPC * 4);
      const f32x4 b = *reinterpret_cast<const f32x4*>(kr + i * LPC * 4);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        q[i * 4 + e] = a[e];
        k[i * 4 + e] = b[e];
      }
    }
    const float g = expf(gb[(row * H + head) * 2]);
    const float beta = gb[(row * H + head) * 2 + 1];
    float o[NCOL];
    float ss = 0.f;
#pragma unroll
    for (int c = 0; c < NCOL; ++c) {
      float dot = 0.f;
#pragma unroll
      for (int e = 0; e < 16; ++e) {
        S[c][e] *= g;
        dot += S[c][e] * k[e];
      }
#pragma unroll
      for (int off = LPC / 2; off > 0; off >>= 1)
        dot += __shfl_xor(dot, off, 64);
      const float u =
          beta *
          (to_f(v[(row * H + head) * vp + col0 + c * cstep]) - dot);
      float r = 0.f;
#pragma unroll
      for (int e = 0; e < 16; ++e) {
        S[c][e] += k[e] * u;
        r += S[c][e] * q[e];
      }
#pragma unroll
      for (int off = LPC / 2; off > 0; off >>= 1)
        r += __shfl_xor(r, off, 64);
      o[c] = r;
      ss += part == 0 ? r * r : 0.f;
    }
    ss = wave_reduce_sum(ss);
    if (lane == 0) red[t & 1][wid] = ss;
    __syncthreads();
    float tot = 0.f;
    for (int i = 0; i < nwave; ++i) tot += red[t & 1][i];
    const float inv = 1.f / sqrtf(tot / vdim + eps);
    if (part == 0) {
#pragma unroll
      for (int c = 0; c < NCOL; ++c) {
        const int j = col0 + c * cstep;
        const float gt = to_f(gate[row * ld_gate + (long)head * vp + j]);
        from_f(y + (row * H + head) * vp + j,
               o[c] * inv * w[c] * act_silu<T>(gt));
      }
    }
  }
#pragma unroll
  for (int c = 0; c < NCOL; ++c)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      f32x4 x;
#pragma unroll
      for (int e = 0; e < 4; ++e) x[e] = S[c][i * 4 + e];
      *reinterpret_cast<f32x4*>(st + (long)(col0 + c * cstep) * dp +
                                i * LPC * 4) = x;
    }
}

extern "C" void launch_delta_scan(
    const float* qk, const void* v, const float* gb, const void* gate,
    int ld_gate, const float* o_norm, float* state, void* y, int H, int G,
    int dp, int vp, int vdim, float eps, const int* seg_row0,
    const int* seg_rows, const int* seg_slot, int nseg, const int* ctx,
    bool fp32, hipStream_t stream) {
  const int lpc = dp / 16;
  const int threads = min(1024, lpc * vp);
  const int ncol = lpc * vp / threads;
#define DS(T, L, N)                                                          \
  hipLaunchKernelGGL((delta_scan_kernel<T, L, N>), dim3(nseg * H),           \
                     dim3(threads), 0, stream, qk, (const T*)v, gb,          \
                     (const T*)gate, ld_gate, o_norm, state, (T*)y, H, G,    \
                     vp, vdim, eps, seg_row0, seg_rows, seg_slot, ctx)
#define DS_N(T)                                \
  do {                                         \
    if (lpc == 4) DS(T, 4, 1);                 \
    else if (lpc == 8 && ncol == 1) DS(T, 8, 1); \
    else if (lpc == 8) DS(T, 8, 2);            \
    else if (ncol == 1) DS(T, 16, 1);          \
    else if (ncol == 2) DS(T, 16, 2);          \
    else DS(T, 16, 4);                         \
  } while (0)
  if (fp32) DS_N(float);
  else DS_N(unsigned short);
#undef DS_N
#undef DS
}
