// Delta rule with a decay per key channel, long segments in chunks of 32
// rows. With b [rows, dim] the logs of the decays summed from the chunk's
// start, S the state before the chunk, products over channels c and
// A_ts = beta_t sum_c k_tc k_sc exp(b_tc - b_sc) for s < t:
//   (I + A) U = beta (V - (exp(b) K) S)
//   o_t = S^T (exp(b_t) q_t) + sum_{s<=t} (sum_c q_tc k_sc exp(b_tc - b_sc)) u_s
//   S  <- exp(b_last) S + sum_s (exp(b_last - b_s) k_s) u_s^T
//
//   channel_chunk_kernel  b, T = (I + A)^-1 beta and P (the sums over c of
//                         o) of every chunk, all chunks at once
//   channel_carry_kernel  the rest, chunk after chunk, a wave per 16 value
//                         columns
// followed by delta_norm_kernel. All of it in fp32, the products on the fp32
// MFMA.
#include "delta_chunk.h"

// Decays within a tile of 16 rows are split into exp(b_t - ref) exp(ref - b_s)
// as long as the second factor stays below e^RANGE; each term of a sum is then
// as exact as if it were formed at once.
#define RANGE 80.f

// log(1 + e^z) to a few units in the last place, also where it is tiny
__device__ __forceinline__ float softplus_near(float z) {
  const float e = fast_exp(-fabsf(z));
  const float w = 1.f + e;
  const float d = w - 1.f;
  const float l = __builtin_amdgcn_logf(w) * 0.6931471805599453f;
  return fmaxf(z, 0.f) + (d == 0.f ? e : l * e * fast_rcp(d));
}

__device__ __forceinline__ f32x4 exp4(f32x4 x) {
  f32x4 y;
#pragma unroll
  for (int i = 0; i < 4; ++i) y[i] = fast_exp(x[i]);
  return y;
}

// Pairs (t = g * 4 + r, s = i16) of the tile of rows row0 .. row0 + 15,
// channels c0 .. c1 - 1, every decay formed at once.
template <int ROW>
__device__ __forceinline__ void direct_tile(const float* K, const float* Q,
                                            const float* B, int row0, int c0,
                                            int c1, int i16, int g, f32x4* kk,
                                            f32x4* pq) {
  for (int c = c0; c < c1; c += 4) {
    const int as = (row0 + i16) * ROW + c;
    const f32x4 bs = *reinterpret_cast<const f32x4*>(B + as);
    const f32x4 ks = *reinterpret_cast<const f32x4*>(K + as);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int at = (row0 + g * 4 + r) * ROW + c;
      const f32x4 bt = *reinterpret_cast<const f32x4*>(B + at);
      const f32x4 kt = *reinterpret_cast<const f32x4*>(K + at);
      const f32x4 qt = *reinterpret_cast<const f32x4*>(Q + at);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float d = ks[e] * fast_exp(fminf(bt[e] - bs[e], 0.f));
        (*kk)[r] += kt[e] * d;
        (*pq)[r] += qt[e] * d;
      }
    }
  }
}

// LDS of the following kernel, in floats: K, Q and b; the waves' partial sums
// over K and Q, then A
#define PART (4 * 6 * 256)
constexpr int a_offset(int dp) {
  return 2 * CH * (dp + 4) > PART ? 2 * CH * (dp + 4) : PART;
}
constexpr int chunk_lds(int dp) {
  return a_offset(dp) + CH * TROW > 3 * CH * (dp + 4) ? a_offset(dp) + CH * TROW
                                                      : 3 * CH * (dp + 4);
}

// ---- b, T and P: one workgroup per (chunk, head) ------------------------------
// Each of the four waves sums over a quarter of the channels.
template <int DP>
__global__ void __launch_bounds__(256)
channel_chunk_kernel(const float* __restrict__ qk,
                     const float* __restrict__ beta,
                     const unsigned short* __restrict__ ag, int ld_ag,
                     const float* __restrict__ a_log,
                     const float* __restrict__ dt, int H, int G,
                     const int* __restrict__ chunks,
                     const int* __restrict__ seg_row0,
                     const int* __restrict__ seg_rows, float* __restrict__ T,
                     float* __restrict__ P, float* __restrict__ bsum) {
  constexpr int ROW = DP + 4;
  __shared__ float betal[CH];
  __shared__ int wide[2];
  float* Kl = reinterpret_cast<float*>(smem);
  float* Ql = Kl + CH * ROW;
  float* Bl = Ql + CH * ROW;
  float* part = Kl;               // [4][6][256], once all are consumed
  float* A = Kl + a_offset(DP);

  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
  const int i16 = lane & 15, g = lane >> 4;
  const int ch = blockIdx.x / H, head = blockIdx.x % H;
  const int kvh = head / (H / G);
  const int seg = chunks[ch * 2], c = chunks[ch * 2 + 1];
  const int cnt = min(CH, seg_rows[seg] - c * CH);
  const long r0 = seg_row0[seg] + c * CH;

  const float rate = -expf(a_log[head]);
#pragma unroll
  for (int i = 0; i < CH * DP / 4 / 256; ++i) {
    const int x = tid + i * 256, row = x / (DP / 4), e = x % (DP / 4) * 4;
    const long src = r0 + min(row, cnt - 1);
    const float* p = qk + (src * 2 * G + kvh) * DP + e;
    const f32x4 q = *reinterpret_cast<const f32x4*>(p);
    const f32x4 k = *reinterpret_cast<const f32x4*>(p + (long)G * DP);
    const s16x4 a =
        *reinterpret_cast<const s16x4*>(ag + src * ld_ag + head * DP + e);
    const f32x4 t = *reinterpret_cast<const f32x4*>(dt + head * DP + e);
    f32x4 b;
#pragma unroll
    for (int j = 0; j < 4; ++j)
      b[j] = row < cnt
                 ? rate * softplus_near(bf2f((unsigned short)a[j]) + t[j])
                 : 0.f;
    *reinterpret_cast<f32x4*>(Ql + row * ROW + e) = q;
    *reinterpret_cast<f32x4*>(Kl + row * ROW + e) = k;
    *reinterpret_cast<f32x4*>(Bl + row * ROW + e) = b;
  }
  if (tid < CH) betal[tid] = tid < cnt ? beta[(r0 + tid) * H + head] : 0.f;
  if (tid < 2) wide[tid] = 0;
  __syncthreads();
  if (tid < DP) {  // sums over the rows of a channel
    float b[CH];
#pragma unroll
    for (int t = 0; t < CH; ++t) b[t] = Bl[t * ROW + tid];
#pragma unroll
    for (int t = 1; t < CH; ++t) b[t] += b[t - 1];
    float* out = bsum + (r0 * H + head) * DP + tid;
#pragma unroll
    for (int t = 0; t < CH; ++t) {
      Bl[t * ROW + tid] = b[t];
      if (t < cnt) out[(long)t * H * DP] = b[t];
    }
    if (-b[15] > RANGE) wide[0] = 1;
    if (b[15] - b[31] > RANGE) wide[1] = 1;
  }
  __syncthreads();

  // tiles (0, 0), (1, 0), (1, 1): references are the chunk's start for the
  // first and row 15 for the others
  f32x4 kk[3], pq[3];
#pragma unroll
  for (int i = 0; i < 3; ++i) kk[i] = pq[i] = (f32x4)0.f;
  const bool wide0 = wide[0], wide1 = wide[1];
  const int q0 = wid * (DP / 4);
#pragma unroll
  for (int kt = 0; kt < DP / 4; kt += 16) {
    const int at = q0 + kt + g * 4;
    f32x4 k[2], q[2], b[2];
#pragma unroll
    for (int m = 0; m < 2; ++m) {
      const int row = (m * 16 + i16) * ROW + at;
      k[m] = *reinterpret_cast<const f32x4*>(Kl + row);
      q[m] = *reinterpret_cast<const f32x4*>(Ql + row);
      b[m] = *reinterpret_cast<const f32x4*>(Bl + row);
    }
    const f32x4 ref = *reinterpret_cast<const f32x4*>(Bl + 15 * ROW + at);
    const f32x4 off = k[0] * exp4(ref - b[0]);
    const f32x4 e1 = exp4(b[1] - ref);
    const f32x4 lk1 = k[1] * e1, lq1 = q[1] * e1;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      kk[1] = mfma4(lk1[r], off[r], kk[1]);
      pq[1] = mfma4(lq1[r], off[r], pq[1]);
    }
    if (!wide0) {
      const f32x4 e0 = exp4(b[0]);
      const f32x4 lk = k[0] * e0, lq = q[0] * e0;
      const f32x4 right = k[0] * exp4(-b[0]);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        kk[0] = mfma4(lk[r], right[r], kk[0]);
        pq[0] = mfma4(lq[r], right[r], pq[0]);
      }
    }
    if (!wide1) {
      const f32x4 right = k[1] * exp4(ref - b[1]);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        kk[2] = mfma4(lk1[r], right[r], kk[2]);
        pq[2] = mfma4(lq1[r], right[r], pq[2]);
      }
    }
  }
  if (wide0)
    direct_tile<ROW>(Kl, Ql, Bl, 0, q0, q0 + DP / 4, i16, g, &kk[0], &pq[0]);
  if (wide1)
    direct_tile<ROW>(Kl, Ql, Bl, 16, q0, q0 + DP / 4, i16, g, &kk[2], &pq[2]);

  __syncthreads();  // K, Q and b are consumed
#pragma unroll
  for (int i = 0; i < 3; ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int at = wid * 6 * 256 + (g * 4 + r) * 16 + i16;
      part[at + i * 256] = kk[i][r];
      part[at + (3 + i) * 256] = pq[i][r];
    }
  __syncthreads();
  float* Pg = P + ((long)ch * H + head) * CH * CH;
#pragma unroll
  for (int i = 0; i < 3; ++i) {
    const int t = (i > 0) * 16 + tid / 16, s = (i > 1) * 16 + tid % 16;
    float a = 0.f, p = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) {
      a += part[(w * 6 + i) * 256 + tid];
      p += part[(w * 6 + 3 + i) * 256 + tid];
    }
    A[t * TROW + s] = t < cnt && s < t ? betal[t] * a : 0.f;
    Pg[t * CH + s] = t < cnt && s <= t ? p : 0.f;
  }
  __syncthreads();
  if (wid == 0) {
    const int j = lane & 31;
    float x[CH];
    inverse_column(A, j, x);
    if (lane < CH) {
      float* Tg = T + ((long)ch * H + head) * CH * CH + j;
#pragma unroll
      for (int i = 0; i < CH; ++i) Tg[i * CH] = x[i] * betal[j];
    }
  }
}

// ---- the state from chunk to chunk ------------------------------------------
// As delta_carry_kernel (delta_chunk.hip), with decayed keys and queries
// formed on their way to LDS and rows of the state decaying one by one.
template <int DP, int NW>
__global__ void __launch_bounds__(NW * 64)
channel_carry_kernel(const float* __restrict__ qk,
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
  constexpr int NKQ = CH * DP / 4 / NT;          // float4 per thread, K, Q or b
  constexpr int NTP = (CH * CH / 4 + NT - 1) / NT;
  constexpr int KT = DP / 16;
  float* Kl = reinterpret_cast<float*>(smem);    // exp(b) k
  float* Ql = Kl + CH * ROW;                     // exp(b) q
  float* El = Ql + CH * ROW;                     // exp(b_last - b) k
  float* Tl = El + CH * ROW;
  float* Pl = Tl + CH * TROW;
  float* Dl = Pl + CH * TROW;                    // exp(b_last)

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
  const int ec = tid % (DP / 4) * 4;  // the thread's channels when staging

  f32x4 kr[NKQ], qr[NKQ], br[NKQ], tp[2][NTP], blast;
  unsigned short vr[2][4];
  // rows behind the segment's end repeat its last one: their rows and
  // columns of T and P are zero. (Nothing here may use what it loads: that
  // would wait for it.)
  auto fetch = [&](int c) {
    const int cnt = min(CH, n - c * CH);
    const long r0 = row0 + c * CH;
#pragma unroll
    for (int i = 0; i < NKQ; ++i) {
      const long row = r0 + min((tid + i * NT) / (DP / 4), cnt - 1);
      const float* src = qk + (row * 2 * G + kvh) * DP + ec;
      kr[i] = *reinterpret_cast<const f32x4*>(src + (long)G * DP);
      qr[i] = *reinterpret_cast<const f32x4*>(src);
      br[i] = *reinterpret_cast<const f32x4*>(bsum + (row * H + head) * DP +
                                              ec);
    }
    blast = *reinterpret_cast<const f32x4*>(
        bsum + ((r0 + cnt - 1) * H + head) * DP + ec);
    const long tile = ((chunk0 + c) * H + head) * CH * CH;
#pragma unroll
    for (int i = 0; i < NTP; ++i) {
      const int x = tid + i * NT;
      if (x < CH * CH / 4) {
        tp[0][i] = *reinterpret_cast<const f32x4*>(T + tile + x * 4);
        tp[1][i] = *reinterpret_cast<const f32x4*>(P + tile + x * 4);
      }
    }
#pragma unroll
    for (int m = 0; m < 2; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        vr[m][r] =
            v[((r0 + min(m * 16 + g * 4 + r, cnt - 1)) * H + head) * vp +
              col];
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
      const int at = (tid + i * NT) / (DP / 4) * ROW + ec;
      const f32x4 e = exp4(br[i]);
      *reinterpret_cast<f32x4*>(Kl + at) = kr[i] * e;
      *reinterpret_cast<f32x4*>(Ql + at) = qr[i] * e;
      *reinterpret_cast<f32x4*>(El + at) = kr[i] * exp4(blast - br[i]);
    }
    if (tid < DP / 4) *reinterpret_cast<f32x4*>(Dl + ec) = exp4(blast);
#pragma unroll
    for (int i = 0; i < NTP; ++i) {
      const int x = tid + i * NT;
      if (x < CH * CH / 4) {
        const int at = x / (CH / 4) * TROW + x % (CH / 4) * 4;
        *reinterpret_cast<f32x4*>(Tl + at) = tp[0][i];
        *reinterpret_cast<f32x4*>(Pl + at) = tp[1][i];
      }
    }
    float vc[2][4];
#pragma unroll
    for (int m = 0; m < 2; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) vc[m][r] = bf2f(vr[m][r]);
    __syncthreads();
    if (c + 1 < nch) fetch(c + 1);

    // K S and Q S
    f32x4 ks[2], out[2];
#pragma unroll
    for (int m = 0; m < 2; ++m) ks[m] = out[m] = (f32x4)0.f;
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
          out[m] = mfma4(b[m][r], S[k][r], out[m]);
        }
    }
    // U = T (V - K S), out = Q S + P U
    f32x4 R[2], U[2];
#pragma unroll
    for (int m = 0; m < 2; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        R[m][r] = vc[m][r] - ks[m][r];
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
    // S = exp(b_last) S + E^T U
#pragma unroll
    for (int k = 0; k < KT; ++k)
      S[k] *= *reinterpret_cast<const f32x4*>(Dl + k * 16 + g * 4);
#pragma unroll
    for (int m = 0; m < 2; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float* kc = El + (m * 16 + g * 4 + r) * ROW + i16;
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

// T, P [nchunks, H, 32, 32], bsum [M, H, dp], o [M, H * vp]: scratch. longs
// [nlong, 2]: segment, its first chunk; chunks [nchunks, 2]: segment, number
// of the chunk in it. Long segments have more than max_rows rows.
extern "C" void launch_channel_chunks(
    const float* qk, const void* v, const float* beta, const void* ag,
    int ld_ag, const float* a_log, const float* dt, const float* o_norm,
    float out_scale, float* state, void* y, long ld_y, float* T, float* P,
    float* bsum, float* o, int M, int H, int G, int dp, int vp, int vdim,
    float eps, const int* longs, int nlong, const int* chunks, int nchunks,
    int max_rows, const int* seg_row0, const int* seg_rows,
    const int* seg_slot, const int* row_seq, const int* ctx,
    hipStream_t stream) {
#define CC(D)                                                               \
  hipLaunchKernelGGL((channel_chunk_kernel<D>), dim3((long)nchunks * H),    \
                     dim3(256), chunk_lds(D) * 4, stream, qk, beta,         \
                     (const unsigned short*)ag, ld_ag, a_log, dt, H, G,     \
                     chunks, seg_row0, seg_rows, T, P, bsum)
  if (dp == 64) CC(64);
  else if (dp == 128) CC(128);
  else CC(256);
#undef CC
  // fewer waves per workgroup while that fills more CUs
  int nw = vp >= 128 ? 8 : 4;
  while (nw > 2 && (long)nlong * H * vp / (16 * nw) < 256) nw /= 2;
  const long wgs = (long)nlong * H * (vp / (16 * nw));
#define DY(D, N)                                                            \
  hipLaunchKernelGGL((channel_carry_kernel<D, N>), dim3(wgs), dim3(N * 64), \
                     (3 * CH * (D + 4) + 2 * CH * TROW + D) * 4, stream,    \
                     qk, (const unsigned short*)v, bsum, T, P, state, o, H, \
                     G, vp, longs, nlong, seg_row0, seg_rows, seg_slot, ctx)
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
  launch_delta_norm(
      o, (const unsigned short*)ag + (long)H * dp, ld_ag, o_norm, out_scale,
      y, ld_y, M, H, vp, vdim, eps, max_rows, seg_rows, row_seq, ctx, true,
      stream);
}
