// Gated delta rule of a ragged step, per head with state S [dim, vdim]:
//   S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
//
// The fused projection ab of a row holds G query heads, G key heads (dp
// numbers each) and H value heads (vp each). Decays are one number per head,
// g = exp(-exp(A) softplus(a + dt)) with the step sizes' b and the a of every
// head side by side and an output gate silu(.), or (CHAN) one per head and
// key channel, with an output gate sigmoid(.) times a constant. delta_prep runs the short convolutions and makes what enters
// the recurrence, in fp32; a scan kernel runs the recurrence. A segment is
// the consecutive rows of one sequence; a sequence that starts in the step
// (ctx 1 in its first row) starts from zeros, whatever its slot holds.
#include "short_conv.h"

extern __shared__ __attribute__((aligned(16))) char smem[];

template <typename T>
__device__ __forceinline__ float act_silu(float z) {
  if constexpr (sizeof(T) == 2) return silu(z);
  else return z * sigmoid_exact(z);
}

// ---- convolutions, unit queries and keys, decays ---------------------------
// A unit is a query, key or value head over a run of `rb` rows; LPH lanes of
// eight channels each share it. The window of inputs stays in registers
// from row to row. TAPS: 0 for any number, at the price of reading every
// input of every row.
template <typename T, int LPH, int TAPS, bool QK>
__device__ __forceinline__ void conv_unit(const ConvArgs<T>& a, int unit,
                                          int r0, int sub, int ch0, int G,
                                          int H, float q_scale,
                                          float unit_eps, float* qk, T* v) {
  constexpr int D = LPH * 8;
  constexpr int NT = TAPS > 0 ? TAPS : 1;
  const int ch = ch0 + sub * 8;
  float w[NT][8], x[NT][8];  // x[j]: the input j rows back
  if (TAPS > 0)
#pragma unroll
    for (int j = 0; j < NT; ++j)
      load8<float>(a.w + (long)(NT - 1 - j) * a.C + ch, w[j]);
  int before = -1;  // sequence of the previous row
  for (int row = r0; row < min(r0 + a.rb, a.M); ++row) {
    const int pos = a.ctx[row] - 1;
    if (pos < 0) {
      before = -1;
      continue;
    }
    const int seg = a.row_seq[row];
    const int o = row - a.seg_row0[seg];  // offset in its segment
    T* slot = a.conv + (long)a.seg_slot[seg] * (a.taps - 1) * a.C + ch;
    float z[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) z[i] = 0.f;
    if (TAPS > 0) {
#pragma unroll
      for (int j = NT - 1; j > 0; --j) {
        if (seg == before)
#pragma unroll
          for (int i = 0; i < 8; ++i) x[j][i] = x[j - 1][i];
        else
          conv_input(a, row, pos, o, slot, ch, j, x[j]);
      }
      load8<T>(a.ab + (long)row * a.ld + ch, x[0]);
#pragma unroll
      for (int j = NT - 1; j >= 0; --j)
#pragma unroll
        for (int i = 0; i < 8; ++i) z[i] += x[j][i] * w[j][i];
    } else {
      for (int j = a.taps - 1; j >= 0; --j) {
        conv_input(a, row, pos, o, slot, ch, j, x[0]);
        load8<float>(a.w + (long)(a.taps - 1 - j) * a.C + ch, w[0]);
#pragma unroll
        for (int i = 0; i < 8; ++i) z[i] += x[0][i] * w[0][i];
      }
    }
    before = seg;
    if (a.shift && a.taps > 1) conv_shift(a, row, slot, ch);
#pragma unroll
    for (int i = 0; i < 8; ++i) z[i] = act_silu<T>(z[i]);
    if (QK) {
      float ss = 0.f;
#pragma unroll
      for (int i = 0; i < 8; ++i) ss += z[i] * z[i];
#pragma unroll
      for (int off = LPH / 2; off > 0; off >>= 1)
        ss += __shfl_xor(ss, off, 64);
      const float inv = (unit < G ? q_scale : 1.f) / sqrtf(ss + unit_eps);
#pragma unroll
      for (int i = 0; i < 8; ++i) z[i] *= inv;
      store8(qk + ((long)row * 2 * G + unit) * D + sub * 8, z);
    } else {
      store8(v + ((long)row * H + unit) * D + sub * 8, z);
    }
  }
}

// What decays and step sizes come from.
template <typename T>
struct DecayArgs {
  const T* ba;         // b of every head (CHAN false: then a), rows a.ld apart
  const float* a_log;  // [H]
  const float* dt;     // [H], CHAN: [H * dp]
  const T* ag;         // CHAN: a [H * dp], rows ld_ag apart
  int ld_ag;
  const int* seg_rows;
  int max_rows;        // CHAN: decays are for segments of up to this many
};

// workgroups: first those of query and key heads, then of value heads, then
// one thread per (row, head) for decays and step sizes -> gb [M, H, 2]: log
// of the decay, step size. CHAN: one thread per (row, head, 8 channels) ->
// gb [M, H]: step size, gc [M, H, dp]: decay.
template <typename T, int LQ, int LV, int TAPS, bool CHAN>
__global__ void __launch_bounds__(256)
delta_prep_kernel(ConvArgs<T> a, DecayArgs<T> d, int H, int G, float q_scale,
                  float unit_eps, float* __restrict__ qk, T* __restrict__ v,
                  float* __restrict__ gb, float* __restrict__ gc, int wg_qk,
                  int wg_v) {
  const int runs = (a.M + a.rb - 1) / a.rb;
  int wg = blockIdx.x;
  if (wg < wg_qk) {
    const long u = (long)wg * (256 / LQ) + threadIdx.x / LQ;
    if (u >= (long)runs * 2 * G) return;  // whole units
    const int unit = (int)(u % (2 * G));
    conv_unit<T, LQ, TAPS, true>(a, unit, (int)(u / (2 * G)) * a.rb,
                                 threadIdx.x % LQ, unit * LQ * 8, G, H,
                                 q_scale, unit_eps, qk, v);
    return;
  }
  wg -= wg_qk;
  if (wg < wg_v) {
    const long u = (long)wg * (256 / LV) + threadIdx.x / LV;
    if (u >= (long)runs * H) return;
    const int unit = (int)(u % H);
    conv_unit<T, LV, TAPS, false>(
        a, unit, (int)(u / H) * a.rb, threadIdx.x % LV,
        2 * G * LQ * 8 + unit * LV * 8, G, H, q_scale, unit_eps, qk, v);
    return;
  }
  wg -= wg_v;
  const long u = (long)wg * 256 + threadIdx.x;
  const long i = CHAN ? u / LQ : u;
  if (i >= (long)a.M * H) return;
  const int row = (int)(i / H), h = (int)(i % H);
  if (a.ctx[row] <= 0) return;
  const T* ba = d.ba + (long)row * a.ld;
  if constexpr (CHAN) {
    const int c = (int)(u % LQ) * 8;
    if (c == 0) gb[i] = sigmoid_exact(to_f(ba[h]));
    if (d.seg_rows[a.row_seq[row]] > d.max_rows) return;
    float x[8], t[8];
    load8<T>(d.ag + (long)row * d.ld_ag + h * LQ * 8 + c, x);
    load8<float>(d.dt + h * LQ * 8 + c, t);
    const float rate = -expf(d.a_log[h]);
#pragma unroll
    for (int k = 0; k < 8; ++k) x[k] = expf(rate * softplus_exact(x[k] + t[k]));
    store8(gc + i * LQ * 8 + c, x);
  } else {
    gb[i * 2] =
        -expf(d.a_log[h]) * softplus_exact(to_f(ba[H + h]) + d.dt[h]);
    gb[i * 2 + 1] = sigmoid_exact(to_f(ba[h]));
  }
}

// chan: decays per channel from ag, a_log [H] and dt [H * dp]; else from the
// columns behind H gates of vp numbers in ab, a_log [H] and dt [H]
extern "C" void launch_delta_prep(
    const void* ab, int ld, const void* ag, int ld_ag, int M, int H, int G,
    int dp, int vp, const float* conv_w, int taps, const float* a_log,
    const float* dt, float q_scale, float unit_eps, float* qk, void* v,
    float* gb, float* gc, void* conv, const int* seg_row0,
    const int* seg_rows, const int* seg_slot, int nseg, int longest,
    int max_rows, const int* row_seq, const int* ctx, bool chan, bool fp32,
    hipStream_t stream) {
  const bool shift = longest <= 1;
  const int rb = M >= 8192 ? 8 : M >= 2048 ? 4 : 1;
  const int C = 2 * G * dp + H * vp;
  const long runs = (M + rb - 1) / rb;
  const int lq = dp / 8, lv = vp / 8;
  const long wg_qk = (runs * 2 * G + 256 / lq - 1) / (256 / lq);
  const long wg_v = (runs * H + 256 / lv - 1) / (256 / lv);
  const long wg_s = ((long)M * H * (chan ? lq : 1) + 255) / 256;
  const int ba_at = chan ? C : C + H * vp;
#define DP_C(T, LQ, LV, TAPS, CH)                                            \
  do {                                                                       \
    const ConvArgs<T> a{(const T*)ab, ld, M, C, taps, rb, conv_w,            \
                        (T*)conv, seg_row0, seg_slot, row_seq, ctx, shift};  \
    const DecayArgs<T> d{(const T*)ab + ba_at, a_log, dt, (const T*)ag,      \
                         ld_ag, seg_rows, max_rows};                         \
    hipLaunchKernelGGL((delta_prep_kernel<T, LQ, LV, TAPS, CH>),             \
                       dim3(wg_qk + wg_v + wg_s), dim3(256), 0, stream, a,   \
                       d, H, G, q_scale, unit_eps, qk, (T*)v, gb, gc,        \
                       (int)wg_qk, (int)wg_v);                               \
    if (!shift && taps > 1)                                                  \
      hipLaunchKernelGGL((conv_state_kernel<T>),                             \
                         dim3((C + 255) / 256, nseg), dim3(256), 0, stream,  \
                         (const T*)ab, ld, C, taps, (T*)conv, seg_row0,      \
                         seg_rows, seg_slot, ctx);                           \
  } while (0)
#define DP(T, LQ, LV, TAPS)                 \
  do {                                      \
    if (chan) DP_C(T, LQ, LV, TAPS, true);  \
    else DP_C(T, LQ, LV, TAPS, false);      \
  } while (0)
#define DP_T(T, LQ, LV)              \
  do {                               \
    if (taps == 4) DP(T, LQ, LV, 4); \
    else DP(T, LQ, LV, 0);           \
  } while (0)
#define DP_V(T, LQ)              \
  do {                           \
    if (lv == 8) DP_T(T, LQ, 8); \
    else if (lv == 16) DP_T(T, LQ, 16); \
    else DP_T(T, LQ, 32);        \
  } while (0)
#define DP_Q(T)                  \
  do {                           \
    if (lq == 8) DP_V(T, 8);     \
    else if (lq == 16) DP_V(T, 16); \
    else DP_V(T, 32);            \
  } while (0)
  if (fp32) DP_Q(float);
  else DP_Q(unsigned short);
#undef DP_Q
#undef DP_V
#undef DP_T
#undef DP
#undef DP_C
}

// ---- recurrence, token by token ---------------------------------------------
// One workgroup per (segment, head). LPC lanes share a value column, each
// with 16 entries of the state's column in registers (float4 number i of
// lane `part` is float4 i * LPC + part of the column); a thread has NCOL
// columns. The output is normed over vdim and gated in place; rows of y are
// ld_y apart. Segments of more than max_rows rows are left to the chunked
// forms (delta_chunk.hip, delta_channel.hip).
template <typename T, int LPC, int NCOL, bool CHAN>
__global__ void __launch_bounds__(1024)
delta_scan_kernel(const float* __restrict__ qk, const T* __restrict__ v,
                  const float* __restrict__ gb, const float* __restrict__ gc,
                  const T* __restrict__ gate, int ld_gate,
                  const float* __restrict__ o_norm, float out_scale,
                  float* __restrict__ state, T* __restrict__ y, long ld_y,
                  int H, int G, int vp, int vdim, float eps,
                  const int* __restrict__ seg_row0,
                  const int* __restrict__ seg_rows,
                  const int* __restrict__ seg_slot,
                  const int* __restrict__ ctx, int max_rows) {
  constexpr int dp = LPC * 16;
  __shared__ float red[2][16];
  const int seg = blockIdx.x / H, head = blockIdx.x % H;
  const int n = seg_rows[seg];
  if (n == 0 || n > max_rows) return;
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
    float g[CHAN ? 16 : 1], beta;
    if constexpr (CHAN) {
      beta = gb[row * H + head];
      const float* gr = gc + (row * H + head) * dp + part * 4;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const f32x4 a = *reinterpret_cast<const f32x4*>(gr + i * LPC * 4);
#pragma unroll
        for (int e = 0; e < 4; ++e) g[i * 4 + e] = a[e];
      }
    } else {
      g[0] = expf(gb[(row * H + head) * 2]);
      beta = gb[(row * H + head) * 2 + 1];
    }
    float o[NCOL];
    float ss = 0.f;
#pragma unroll
    for (int c = 0; c < NCOL; ++c) {
      float dot = 0.f;
#pragma unroll
      for (int e = 0; e < 16; ++e) {
        S[c][e] *= g[CHAN ? e : 0];
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
    const float inv = 1.f / sqrtf(tot / vdim + eps) * (CHAN ? out_scale : 1.f);
    if (part == 0) {
#pragma unroll
      for (int c = 0; c < NCOL; ++c) {
        const int j = col0 + c * cstep;
        const float gt = to_f(gate[row * ld_gate + (long)head * vp + j]);
        from_f(y + row * ld_y + (long)head * vp + j,
               o[c] * inv * w[c] *
                   (CHAN ? sigmoid_exact(gt) : act_silu<T>(gt)));
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
    const float* qk, const void* v, const float* gb, const float* gc,
    const void* gate, int ld_gate, const float* o_norm, float out_scale,
    float* state, void* y, long ld_y, int H, int G, int dp, int vp, int vdim,
    float eps, const int* seg_row0, const int* seg_rows, const int* seg_slot,
    int nseg, const int* ctx, int max_rows, bool chan, bool fp32,
    hipStream_t stream) {
  const int lpc = dp / 16;
  const int threads = min(1024, lpc * vp);
  const int ncol = lpc * vp / threads;
#define DS_C(T, L, N, CH)                                                    \
  hipLaunchKernelGGL((delta_scan_kernel<T, L, N, CH>), dim3(nseg * H),       \
                     dim3(threads), 0, stream, qk, (const T*)v, gb, gc,      \
                     (const T*)gate, ld_gate, o_norm, out_scale, state,      \
                     (T*)y, ld_y, H, G, vp, vdim, eps, seg_row0, seg_rows,   \
                     seg_slot, ctx, max_rows)
#define DS(T, L, N)                  \
  do {                               \
    if (chan) DS_C(T, L, N, true);   \
    else DS_C(T, L, N, false);       \
  } while (0)
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
#undef DS_C
}
