// Gated delta rule of long segments, in chunks of 32 rows. With b the log
// of the decay summed from the chunk's start, S the state before the chunk
// and A_ts = beta_t exp(b_t - b_s) k_t.k_s for s < t (rows t, s):
//   (I + A) U = beta (V - exp(b) K S)         rows u_t of the updates
//   o_t = exp(b_t) S^T q_t + sum_{s<=t} exp(b_t - b_s) (q_t.k_s) u_s
//   S  <- exp(b_last) S + sum_s exp(b_last - b_s) k_s u_s^T
// Every exponent is <= 0.
//
//   delta_chunk_kernel  T = (I + A)^-1 beta and P = tril(exp(b_t - b_s)
//                       q_t.k_s) of every chunk, all chunks at once
//   delta_carry_kernel  the rest, chunk after chunk, a wave per 16 value
//                       columns
//   delta_norm_kernel   gated output norm
// All of it in fp32, the products on the fp32 MFMA.
#include "delta_chunk.h"

// ---- T and P: one wave per (chunk, key head) -------------------------------
template <int DP>
__global__ void __launch_bounds__(256)
delta_chunk_kernel(const float* __restrict__ qk, const float* __restrict__ gb,
                   int H, int G, const int* __restrict__ chunks, int nchunks,
                   const int* __restrict__ seg_row0,
                   const int* __restrict__ seg_rows, float* __restrict__ T,
                   float* __restrict__ P, float* __restrict__ bsum) {
  __shared__ __attribute__((aligned(16))) float A_lds[4][CH * TROW];
  __shared__ float b_lds[4][CH], beta_lds[4][CH];
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int i16 = lane & 15, g = lane >> 4;
  const long w = (long)blockIdx.x * 4 + wid;
  if (w >= (long)nchunks * G) return;
  const int ch = (int)(w / G), kvh = (int)(w % G);
  const int seg = chunks[ch * 2], c = chunks[ch * 2 + 1];
  const int cnt = min(CH, seg_rows[seg] - c * CH);
  const long r0 = seg_row0[seg] + c * CH;
  float* A = A_lds[wid];
  float *bl = b_lds[wid], *betal = beta_lds[wid];

  // q_t.k_s and k_t.k_s: tiles (0, 0), (1, 0), (1, 1)
  f32x4 kk[3], pq[3];
#pragma unroll
  for (int i = 0; i < 3; ++i) kk[i] = pq[i] = {0.f, 0.f, 0.f, 0.f};
  const float *qr[2], *kr[2];
#pragma unroll
  for (int m = 0; m < 2; ++m) {
    const long row = r0 + min(m * 16 + i16, cnt - 1);
    qr[m] = qk + (row * 2 * G + kvh) * DP + g * 4;
    kr[m] = qr[m] + (long)G * DP;
  }
#pragma unroll 2
  for (int kt = 0; kt < DP; kt += 16) {
    f32x4 q[2], k[2];
#pragma unroll
    for (int m = 0; m < 2; ++m) {
      q[m] = *reinterpret_cast<const f32x4*>(qr[m] + kt);
      k[m] = *reinterpret_cast<const f32x4*>(kr[m] + kt);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      kk[0] = mfma4(k[0][r], k[0][r], kk[0]);
      kk[1] = mfma4(k[1][r], k[0][r], kk[1]);
      kk[2] = mfma4(k[1][r], k[1][r], kk[2]);
      pq[0] = mfma4(q[0][r], k[0][r], pq[0]);
      pq[1] = mfma4(q[1][r], k[0][r], pq[1]);
      pq[2] = mfma4(q[1][r], k[1][r], pq[2]);
    }
  }

  const int j = lane & 31;
  for (int head = kvh * (H / G); head < (kvh + 1) * (H / G); ++head) {
    float b = 0.f, beta = 0.f;
    if (j < cnt) {
      b = gb[((r0 + j) * H + head) * 2];
      beta = gb[((r0 + j) * H + head) * 2 + 1];
    }
#pragma unroll
    for (int off = 1; off < CH; off <<= 1) {
      const float x = __shfl_up(b, off, CH);
      if (j >= off) b += x;
    }
    wave_sync();  // the previous head's matrix is consumed
    if (lane < CH) {
      bl[j] = b;
      betal[j] = beta;
      if (j < cnt) bsum[(r0 + j) * H + head] = b;
    }
    wave_sync();
    float* Pg = P + ((long)ch * H + head) * CH * CH;
#pragma unroll
    for (int i = 0; i < 3; ++i) {
      const int m = i > 0, n = i > 1;
      const int s = n * 16 + i16;
      const float bs = bl[s];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = m * 16 + g * 4 + r;
        const bool row = t < cnt;
        const float d = expf(fminf(bl[t] - bs, 0.f));
        A[t * TROW + s] = row && s < t ? betal[t] * d * kk[i][r] : 0.f;
        Pg[t * CH + s] = row && s <= t ? d * pq[i][r] : 0.f;
      }
    }
    wave_sync();
    float x[CH];
    inverse_column(A, j, x);
    if (lane < CH) {
      float* Tg = T + ((long)ch * H + head) * CH * CH + j;
#pragma unroll
      for (int i = 0; i < CH; ++i) Tg[i * CH] = x[i] * beta;
    }
  }
}

// ---- the state from chunk to chunk ------------------------------------------
// A workgroup of NW waves serves one head of one segment, 16 value columns a
// wave: the wave's part of the state [DP x 16] is DP / 16 accumulators. K, Q,
// T and P of a chunk are staged in LDS; those of the next chunk are on their
// way in registers meanwhile.
template <int DP, int NW>
__global__ void __launch_bounds__(NW * 64)
delta_carry_kernel(const float* __restrict__ qk,
                   const unsigned short* __restrict__ v,
                   const float* __restrict__ bsum,
                   const float* __restrict__ T, const float* __restrict__ P,
                   float* __restrict__ state, float* __restrict__ o, int H,
                   int G, int vp, const int* __restrict__ longs, int nlong,
                   const int* __restrict__ seg_row0,
                   const int* __restrict__ seg_rows,
                   const int* __restrict__ seg_slot,
                   const int* __restrict__ ctx) {
  constexpr int ROW = DP + 4;
  constexpr int NT = NW * 64;
  constexpr int NKQ = CH * DP / 4 / NT;          // float4 per thread, K or Q
  constexpr int NTP = (CH * CH / 4 + NT - 1) / NT;
  constexpr int KT = DP / 16;
  float* Kl = reinterpret_cast<float*>(smem);
  float* Ql = Kl + CH * ROW;
  float* Tl = Ql + CH * ROW;
  float* Pl = Tl + CH * TROW;

  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
  const int i16 = lane & 15, g = lane >> 4;
  const int heads = nlong * H;
  const int lh = blockIdx.x % heads;
  const int col = (blockIdx.x / heads * NW + wid) * 16 + i16;
  const int head = lh % H, seg = longs[lh / H * 2];
  const long chunk0 = longs[lh / H * 2 + 1];
  const int kvh = head / (H / G);
  const int n = seg_rows[seg];
  const long row0 = seg_row0[seg];
  const int nch = (n + CH - 1) / CH;

  f32x4 kq[2][NKQ], tp[2][NTP];
  unsigned short vr[2][4];
  float br[2][4], blast = 0.f;
  // rows behind the segment's end repeat its last one: their rows and
  // columns of T and P are zero. (Nothing here may use what it loads: that
  // would wait for it.)
  auto fetch = [&](int c) {
    const int cnt = min(CH, n - c * CH);
    const long r0 = row0 + c * CH;
#pragma unroll
    for (int i = 0; i < NKQ; ++i) {
      const int x = tid + i * NT, row = x / (DP / 4), e = x % (DP / 4) * 4;
      const float* src =
          qk + ((r0 + min(row, cnt - 1)) * 2 * G + kvh) * DP + e;
      kq[0][i] = *reinterpret_cast<const f32x4*>(src + (long)G * DP);
      kq[1][i] = *reinterpret_cast<const f32x4*>(src);
    }
    const long tile = ((chunk0 + c) * H + head) * CH * CH;
#pragma unroll
    for (int i = 0; i < NTP; ++i) {
      const int x = tid + i * NT;
      if (x < CH * CH / 4) {
        tp[0][i] = *reinterpret_cast<const f32x4*>(T + tile + x * 4);
        tp[1][i] = *reinterpret_cast<const f32x4*>(P + tile + x * 4);
      }
    }
    blast = bsum[(r0 + cnt - 1) * H + head];
#pragma unroll
    for (int m = 0; m < 2; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const long rh =
            (r0 + min(m * 16 + g * 4 + r, cnt - 1)) * H + head;
        vr[m][r] = v[rh * vp + col];
        br[m][r] = bsum[rh];
      }
  };

  f32x4 S[KT];
  float* st =
      state + (((long)seg_slot[seg] * H + head) * vp + col) * DP + g * 4;
  const bool fresh = ctx[row0] <= 1;
#pragma unroll
  for (int k = 0; k < KT; ++k) {
    S[k] = (f32x4)0.f;
    if (!fresh) S[k] = *reinterpret_cast<const f32x4*>(st + k * 16);
  }

  fetch(0);
  for (int c = 0; c < nch; ++c) {
    __syncthreads();  // the previous chunk is consumed
#pragma unroll
    for (int i = 0; i < NKQ; ++i) {
      const int x = tid + i * NT, row = x / (DP / 4), e = x % (DP / 4) * 4;
      *reinterpret_cast<f32x4*>(Kl + row * ROW + e) = kq[0][i];
      *reinterpret_cast<f32x4*>(Ql + row * ROW + e) = kq[1][i];
    }
#pragma unroll
    for (int i = 0; i < NTP; ++i) {
      const int x = tid + i * NT;
      if (x < CH * CH / 4) {
        const int at = x / (CH / 4) * TROW + x % (CH / 4) * 4;
        *reinterpret_cast<f32x4*>(Tl + at) = tp[0][i];
        *reinterpret_cast<f32x4*>(Pl + at) = tp[1][i];
      }
    }
    float vc[2][4], eb[2][4], es[2][4];
    const float elast = expf(blast);
#pragma unroll
    for (int m = 0; m < 2; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        vc[m][r] = bf2f(vr[m][r]);
        eb[m][r] = expf(br[m][r]);
        es[m][r] = expf(blast - br[m][r]);
      }
    __syncthreads();
    if (c + 1 < nch) fetch(c + 1);

    // K S and Q S
    f32x4 ks[2], qs[2];
#pragma unroll
    for (int m = 0; m < 2; ++m) ks[m] = qs[m] = (f32x4)0.f;
#pragma unroll
    for (int k = 0; k < KT; ++k) {
      f32x4 a[2], b[2];
#pragma unroll
      for (int m = 0; m < 2; ++m) {
        const int at = (m * 16 + i16) * ROW + k * 16 + g * 4;
        a[m] = *reinterpret_cast<const f32x4*>(Kl + at);
        b[m] = *reinterpret_cast<const f32x4*>(Ql + at);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r)
#pragma unroll
        for (int m = 0; m < 2; ++m) {
          ks[m] = mfma4(a[m][r], S[k][r], ks[m]);
          qs[m] = mfma4(b[m][r], S[k][r], qs[m]);
        }
    }
    // U = T (V - exp(b) K S), out = exp(b) Q S + P U
    f32x4 R[2], U[2], out[2];
#pragma unroll
    for (int m = 0; m < 2; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        R[m][r] = vc[m][r] - eb[m][r] * ks[m][r];
        out[m][r] = eb[m][r] * qs[m][r];
        U[m][r] = 0.f;
      }
#pragma unroll
    for (int m = 0; m < 2; ++m)
#pragma unroll
      for (int k = 0; k <= m; ++k) {
        const f32x4 a = *reinterpret_cast<const f32x4*>(
            Tl + (m * 16 + i16) * TROW + k * 16 + g * 4);
#pragma unroll
        for (int r = 0; r < 4; ++r) U[m] = mfma4(a[r], R[k][r], U[m]);
      }
#pragma unroll
    for (int m = 0; m < 2; ++m)
#pragma unroll
      for (int k = 0; k <= m; ++k) {
        const f32x4 a = *reinterpret_cast<const f32x4*>(
            Pl + (m * 16 + i16) * TROW + k * 16 + g * 4);
#pragma unroll
        for (int r = 0; r < 4; ++r) out[m] = mfma4(a[r], U[k][r], out[m]);
      }
    // S = exp(b_last) S + K^T exp(b_last - b) U
#pragma unroll
    for (int m = 0; m < 2; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) U[m][r] *= es[m][r];
#pragma unroll
    for (int k = 0; k < KT; ++k)
#pragma unroll
      for (int e = 0; e < 4; ++e) S[k][e] *= elast;
#pragma unroll
    for (int m = 0; m < 2; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float* kc = Kl + (m * 16 + g * 4 + r) * ROW + i16;
#pragma unroll
        for (int k = 0; k < KT; ++k)
          S[k] = mfma4(kc[k * 16], U[m][r], S[k]);
      }
    const int cnt = min(CH, n - c * CH);
#pragma unroll
    for (int m = 0; m < 2; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = m * 16 + g * 4 + r;
        if (t < cnt)
          o[((row0 + c * CH + t) * H + head) * vp + col] = out[m][r];
      }
  }
#pragma unroll
  for (int k = 0; k < KT; ++k) *reinterpret_cast<f32x4*>(st + k * 16) = S[k];
}

// ---- output norm and gate, silu(gate) or sigmoid(gate) * out_scale; LV lanes
// share a head of a row ---------------------------------------------------------
template <int LV, bool SIGMOID>
__global__ void __launch_bounds__(256)
delta_norm_kernel(const float* __restrict__ o,
                  const unsigned short* __restrict__ gate, int ld_gate,
                  const float* __restrict__ o_norm,
                  float out_scale, unsigned short* __restrict__ y, long ld_y,
                  int M, int H, int vdim, float eps, int max_rows, const int* __restrict__ seg_rows,
                  const int* __restrict__ row_seq,
                  const int* __restrict__ ctx) {
  constexpr int VP = LV * 8;
  const int sub = threadIdx.x % LV;
  const long u = (long)blockIdx.x * (256 / LV) + threadIdx.x / LV;
  if (u >= (long)M * H) return;  // whole heads
  const int row = (int)(u / H), head = (int)(u % H);
  if (ctx[row] <= 0 || seg_rows[row_seq[row]] <= max_rows) return;
  float x[8], w[8], gt[8];
  load8<float>(o + u * VP + sub * 8, x);
  load8<unsigned short>(gate + (long)row * ld_gate + head * VP + sub * 8, gt);
  load8<float>(o_norm + sub * 8, w);
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < 8; ++i) ss += x[i] * x[i];
#pragma unroll
  for (int off = LV / 2; off > 0; off >>= 1) ss += __shfl_xor(ss, off, 64);
  const float inv =
      1.f / sqrtf(ss / vdim + eps) * (SIGMOID ? out_scale : 1.f);
#pragma unroll
  for (int i = 0; i < 8; ++i)
    x[i] *= inv * w[i] *
            (SIGMOID ? fast_rcp(1.f + fast_exp(-gt[i])) : silu(gt[i]));
  store8(y + row * ld_y + head * VP + sub * 8, x);
}

// rows of y are ld_y apart; segments of more than max_rows rows only
extern "C" void launch_delta_norm(const float* o, const void* gate,
                                  int ld_gate, const float* o_norm,
                                  float out_scale, void* y, long ld_y, int M,
                                  int H, int vp, int vdim, float eps,
                                  int max_rows, const int* seg_rows,
                                  const int* row_seq, const int* ctx,
                                  bool sigmoid, hipStream_t stream) {
#define DN_G(L, S)                                                          \
  hipLaunchKernelGGL((delta_norm_kernel<L, S>),                             \
                     dim3(((long)M * H + 256 / L - 1) / (256 / L)),         \
                     dim3(256), 0, stream, o, (const unsigned short*)gate,  \
                     ld_gate, o_norm, out_scale, (unsigned short*)y, ld_y,  \
                     M, H, vdim, eps, max_rows, seg_rows, row_seq, ctx)
#define DN(L)                      \
  do {                             \
    if (sigmoid) DN_G(L, true);    \
    else DN_G(L, false);           \
  } while (0)
  if (vp == 64) DN(8);
  else if (vp == 128) DN(16);
  else DN(32);
#undef DN
#undef DN_G
}

// T, P [nchunks, H, 32, 32], bsum [M, H], o [M, H * vp]: scratch. longs
// [nlong, 2]: segment, its first chunk; chunks [nchunks, 2]: segment, number
// of the chunk in it. Long segments have more than max_rows rows.
extern "C" void launch_delta_chunks(
    const float* qk, const void* v, const float* gb, const void* gate,
    int ld_gate, const float* o_norm, float* state, void* y, float* T,
    float* P, float* bsum, float* o, int M, int H, int G, int dp, int vp,
    int vdim, float eps, const int* longs, int nlong, const int* chunks,
    int nchunks, int max_rows, const int* seg_row0, const int* seg_rows,
    const int* seg_slot, const int* row_seq, const int* ctx,
    hipStream_t stream) {
#define DC(D)                                                               \
  hipLaunchKernelGGL((delta_chunk_kernel<D>),                               \
                     dim3(((long)nchunks * G + 3) / 4), dim3(256), 0,       \
                     stream, qk, gb, H, G, chunks, nchunks, seg_row0,       \
                     seg_rows, T, P, bsum)
  if (dp == 64) DC(64);
  else if (dp == 128) DC(128);
  else DC(256);
#undef DC
  // fewer waves per workgroup while that fills more CUs
  int nw = vp >= 128 ? 8 : 4;
  while (nw > 2 && (long)nlong * H * vp / (16 * nw) < 256) nw /= 2;
  const long wgs = (long)nlong * H * (vp / (16 * nw));
#define DY(D, N)                                                            \
  hipLaunchKernelGGL((delta_carry_kernel<D, N>), dim3(wgs), dim3(N * 64),   \
                     (2 * CH * (D + 4) + 2 * CH * TROW) * 4, stream, qk,    \
                     (const unsigned short*)v, bsum, T, P, state, o, H, G,  \
                     vp, longs, nlong, seg_row0, seg_rows, seg_slot, ctx)
#define DY_N(D)                \
  do {                         \
    if (nw == 8) DY(D, 8);     \
    else if (nw == 4) DY(D, 4); \
    else DY(D, 2);             \
  } while (0)
  if (dp == 64) DY_N(64);
  else if (dp == 128) DY_N(128);
  else DY_N(256);
#undef DY_N
#undef DY
  launch_delta_norm(o, gate, ld_gate, o_norm, 1.f, y, (long)H * vp, M, H, vp,
                    vdim, eps, max_rows, seg_rows, row_seq, ctx, false,
                    stream);
}
