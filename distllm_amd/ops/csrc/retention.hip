// Retention of a ragged step: linear attention with a fixed decay per head.
// Per head with state S [dim, vdim], decay g and rotated queries and keys
// (keys times kscale):
//   S <- g S + k v^T;  o = S^T q;  y = o / rms(o) * silu(gate)
//
// A row of the fused projection ab holds H query heads and H key heads (dp
// numbers each), H value heads and H gate heads (vp each). A segment is the
// consecutive rows of one sequence; a sequence that starts in the step (ctx 1
// in its first row) starts from zeros, whatever its slot holds. The state is
// kept as [slots, H, vp, dp] in fp32, and everything that enters it is fp32.
//
//   retention_scan_kernel   token by token, any type, short segments
//   retention_chunk_kernel  long segments, 32 rows at a time on the fp32 MFMA
//   retention_join_kernel   states between the pieces of a long segment
//
// With n the rows of a chunk and S the state before it (rows t, s from 0):
//   o_t = g^(t+1) S^T q_t + sum_{s<=t} g^(t-s) (q_t.k_s) v_s
//   S  <- g^n S + sum_s g^(n-1-s) k_s v_s^T
// A long segment may be cut into pieces that run side by side: first every
// piece but the last finds its state from zeros, then these are joined.
#include "common.h"

#define CH 32    // rows of a chunk
#define TROW 36  // padded row of a chunk x chunk matrix
#define PROW 20  // padded row of a 16 x 16 partial sum

extern __shared__ __attribute__((aligned(16))) char smem[];

template <typename T>
struct RetentionArgs {
  const T* ab;
  int ld, H, vp, vdim;
  float kscale, eps;
  const float* decay;   // [2, H]: decay, its base-2 logarithm
  const float* table;   // [M, half, 2]
  int half;
  float* state;
  T* y;                 // [M, H * vp]
  const int *seg_row0, *seg_rows, *seg_slot, *ctx;
};

template <typename T>
__device__ __forceinline__ float gate_silu(float z) {
  if constexpr (sizeof(T) == 2) return silu(z);
  else return z * sigmoid_exact(z);
}

// number c of a head at src, rotated by cs
template <typename T>
__device__ __forceinline__ float rotated(const T* src, int c, int half,
                                         const float* cs) {
  const float x = to_f(src[c]);
  if (c >= 2 * half) return x;
  const bool low = c < half;
  const int i = low ? c : c - half;
  const float y = to_f(src[low ? c + half : i]);
  return x * cs[i * 2] + (low ? -y : y) * cs[i * 2 + 1];
}

// ---- token by token -----------------------------------------------------------
// One workgroup per (segment, head). LPC lanes share a value column, each
// with 16 entries of the state's column in registers (float4 number i of
// lane `part` is float4 i * LPC + part of the column); a thread has NCOL
// columns. Rotated queries and keys of up to TT rows are staged in LDS.
// Segments of more than max_rows rows are left to the chunks.
#define TT 16

template <typename T, int LPC, int NCOL>
__global__ void __launch_bounds__(1024)
retention_scan_kernel(const RetentionArgs<T> a, int max_rows) {
  constexpr int dp = LPC * 16;
  __shared__ float red[2][16];
  __shared__ __attribute__((aligned(16))) float qk[TT][2][dp];
  const int seg = blockIdx.x / a.H, head = blockIdx.x % a.H;
  const int n = a.seg_rows[seg];
  if (n == 0 || n > max_rows) return;
  const int row0 = a.seg_row0[seg];
  const int part = threadIdx.x % LPC;
  const int col0 = threadIdx.x / LPC, cstep = blockDim.x / LPC;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int nwave = blockDim.x >> 6;
  const float g = a.decay[head];
  float* st = a.state + ((long)a.seg_slot[seg] * a.H + head) * a.vp * dp +
              part * 4;

  float S[NCOL][16];
  const bool fresh = a.ctx[row0] <= 1;
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

  for (int t0 = 0; t0 < n; t0 += TT) {
    const int cnt = min(TT, n - t0);
    if (t0 > 0) __syncthreads();  // the rows before are consumed
    for (int u = threadIdx.x; u < cnt * 2 * dp; u += blockDim.x) {
      const int t = u / (2 * dp), which = u / dp % 2, c = u % dp;
      const long row = row0 + t0 + t;
      const float x = rotated(a.ab + row * a.ld + (which * a.H + head) * dp,
                              c, a.half, a.table + row * a.half * 2);
      qk[t][which][c] = which == 1 ? x * a.kscale : x;
    }
    __syncthreads();
    for (int t = 0; t < cnt; ++t) {
      const long row = row0 + t0 + t;
      const T* vr = a.ab + row * a.ld + 2 * a.H * dp + head * a.vp;
      float v[NCOL], o[NCOL];
#pragma unroll
      for (int c = 0; c < NCOL; ++c) v[c] = to_f(vr[col0 + c * cstep]);
      float q[16], k[16];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int at = (i * LPC + part) * 4;
        const f32x4 x = *reinterpret_cast<const f32x4*>(&qk[t][0][at]);
        const f32x4 z = *reinterpret_cast<const f32x4*>(&qk[t][1][at]);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          q[i * 4 + e] = x[e];
          k[i * 4 + e] = z[e];
        }
      }
      float ss = 0.f;
#pragma unroll
      for (int c = 0; c < NCOL; ++c) {
        float r = 0.f;
#pragma unroll
        for (int e = 0; e < 16; ++e) {
          S[c][e] = g * S[c][e] + k[e] * v[c];
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
      const float inv = 1.f / sqrtf(tot / a.vdim + a.eps);
      if (part == 0) {
#pragma unroll
        for (int c = 0; c < NCOL; ++c) {
          const int j = col0 + c * cstep;
          const float gt = to_f(vr[a.H * a.vp + j]);
          from_f(a.y + (row * a.H + head) * a.vp + j,
                 o[c] * inv * gate_silu<T>(gt));
        }
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

// ---- long segments --------------------------------------------------------------
// Operands of the 16 x 16 x 4 product: step r of a block of 16 inner indices
// takes those with number g * 4 + r (g = lane / 16), which lets a lane read
// operands as float4 and lets an accumulator (rows g * 4 + r) be the right
// operand of the next product as it is.
__device__ __forceinline__ f32x4 mfma4(float a, float b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

__device__ __forceinline__ float exp2_of(float x) {
  return __builtin_amdgcn_exp2f(x);
}

// pieces [P, 5]: segment, first row in it, rows, number, pieces of the
// segment. One workgroup per (piece, head), a wave for each 16 value columns
// (its part of the state, DP x 16, is DP / 16 accumulators).
//   LOCAL  the piece's state from zeros, to between[piece]; not for the last
//          piece of a segment
//   else   the outputs, from the slot's state or (several pieces) from
//          between[piece]; the last piece writes the slot
// Rotated queries and keys of a chunk are staged in LDS, those of the next
// chunk are on their way in registers meanwhile. For the scores the waves
// split the inner dimension; their sums meet in LDS. VEC: half is a multiple
// of 8, so that rotation partners are eight in a row, too.
template <int DP, int NW, bool LOCAL, bool VEC>
__global__ void __launch_bounds__(NW * 64, NW >= 8 ? 4 : 2)
retention_chunk_kernel(const RetentionArgs<unsigned short> a,
                       const int* __restrict__ pieces,
                       float* __restrict__ between) {
  typedef unsigned short T;
  constexpr int VP = NW * 16, NT = NW * 64;
  constexpr int ROW = DP + 4, OROW = VP + 4;
  constexpr int KT = DP / 16;
  constexpr int NP = NW < KT ? NW : KT;       // waves that form scores
  constexpr int WHICH = LOCAL ? 1 : 2;        // keys, then queries
  constexpr int SLOTS = CH * WHICH * KT;      // of 16 numbers
  constexpr int NS = (SLOTS + NT - 1) / NT;
  float* Kl = reinterpret_cast<float*>(smem);
  float* Ql = Kl + CH * ROW;
  float* Pl = Ql + CH * ROW;                  // [CH][TROW]
  float* part = Pl + CH * TROW;               // [NP][3][16][PROW]
  float* Ol = part;                           // [CH][OROW], later

  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
  const int i16 = lane & 15, g = lane >> 4;
  const int piece = blockIdx.x / a.H, head = blockIdx.x % a.H;
  const int* pc = pieces + piece * 5;
  const int seg = pc[0], n = pc[2], number = pc[3], count = pc[4];
  if (LOCAL && number + 1 == count) return;
  const long row0 = a.seg_row0[seg] + pc[1];
  const int nch = (n + CH - 1) / CH;
  const int col = wid * 16 + i16;
  const float lg = a.decay[a.H + head];
  const int at_q = head * DP, at_k = (a.H + head) * DP;
  const int at_v = 2 * a.H * DP + head * VP, at_g = at_v + a.H * VP;

  // slot number u: 16 numbers of a row of keys or queries, as two groups of
  // eight that rotate with each other, or two that do not rotate
  s16x8 ra[NS], rb[NS];
  float cs[NS][VEC ? 16 : 1];
  unsigned short vr[2][4];
  s16x8 gr;
  auto fetch = [&](int c) {
    const int cnt = min(CH, n - c * CH);
    const long r0 = row0 + c * CH;
    if constexpr (VEC) {
#pragma unroll
      for (int i = 0; i < NS; ++i) {
        const int u = tid + i * NT;
        if (SLOTS % NT != 0 && u >= SLOTS) break;
        const int j = u % KT, which = u / KT % WHICH;
        const long row = r0 + min(u / (KT * WHICH), cnt - 1);
        const T* src = a.ab + row * a.ld + (which == 0 ? at_k : at_q);
        const bool turn = j * 8 < a.half;
        const int x = turn ? j * 8 : j * 16;
        ra[i] = *reinterpret_cast<const s16x8*>(src + x);
        rb[i] = *reinterpret_cast<const s16x8*>(src + x +
                                                (turn ? a.half : 8));
        if (turn) {
          const float* t = a.table + (row * a.half + j * 8) * 2;
          load8<float>(t, cs[i]);
          load8<float>(t + 8, cs[i] + 8);
        }
      }
    }
#pragma unroll
    for (int m = 0; m < 2; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        vr[m][r] = a.ab[(r0 + min(m * 16 + g * 4 + r, cnt - 1)) * a.ld +
                        at_v + col];
    if (!LOCAL)
      gr = *reinterpret_cast<const s16x8*>(
          a.ab + (r0 + min(tid / (VP / 8), cnt - 1)) * a.ld + at_g +
          tid % (VP / 8) * 8);
  };
  auto stage = [&](int c) {
    const int cnt = min(CH, n - c * CH);
#pragma unroll
    for (int i = 0; i < NS; ++i) {
      const int u = tid + i * NT;
      if (SLOTS % NT != 0 && u >= SLOTS) break;
      const int j = u % KT, which = u / KT % WHICH, t = u / (KT * WHICH);
      float* dst = (which == 0 ? Kl : Ql) + t * ROW;
      float z[16];
      int x = j * 16, y = j * 16 + 8;
      if constexpr (VEC) {
        bf8_to_f32(ra[i], z);
        bf8_to_f32(rb[i], z + 8);
        if (j * 8 < a.half) {
          x = j * 8;
          y = x + a.half;
#pragma unroll
          for (int e = 0; e < 8; ++e) {
            const float p = z[e], q = z[8 + e];
            z[e] = p * cs[i][2 * e] - q * cs[i][2 * e + 1];
            z[8 + e] = q * cs[i][2 * e] + p * cs[i][2 * e + 1];
          }
        }
      } else {
        const long row = row0 + c * CH + min(t, cnt - 1);
        const T* src = a.ab + row * a.ld + (which == 0 ? at_k : at_q);
#pragma unroll
        for (int e = 0; e < 16; ++e)
          z[e] = rotated(src, x + e, a.half, a.table + row * a.half * 2);
      }
      // rows behind the end count for nothing
      const float f = t >= cnt ? 0.f : which == 0 ? a.kscale : 1.f;
#pragma unroll
      for (int e = 0; e < 16; ++e) z[e] *= f;
#pragma unroll
      for (int e = 0; e < 8; e += 4) {
        *reinterpret_cast<f32x4*>(dst + x + e) =
            f32x4{z[e], z[e + 1], z[e + 2], z[e + 3]};
        *reinterpret_cast<f32x4*>(dst + y + e) =
            f32x4{z[8 + e], z[9 + e], z[10 + e], z[11 + e]};
      }
    }
  };

  f32x4 S[KT];
  const long own = ((long)piece * a.H + head) * VP + col;
  float* slot =
      a.state + (((long)a.seg_slot[seg] * a.H + head) * VP + col) * DP + g * 4;
  const float* from = count > 1 ? between + own * DP + g * 4 : slot;
  const bool zero = LOCAL || (count == 1 && a.ctx[row0] <= 1);
#pragma unroll
  for (int k = 0; k < KT; ++k) {
    S[k] = (f32x4)0.f;
    if (!zero) S[k] = *reinterpret_cast<const f32x4*>(from + k * 16);
  }
  // weights of this lane's rows m * 16 + g * 4 + r (chunks of 32 rows)
  const float glast = exp2_of(lg * CH);

  fetch(0);
  for (int c = 0; c < nch; ++c) {
    const int cnt = min(CH, n - c * CH);
    if (LOCAL && c > 0) __syncthreads();  // the chunk before is consumed
    stage(c);
    float v[2][4], gt[8];
#pragma unroll
    for (int m = 0; m < 2; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) v[m][r] = bf2f(vr[m][r]);
    if (!LOCAL) bf8_to_f32(gr, gt);
    __syncthreads();
    if (c + 1 < nch) fetch(c + 1);

    f32x4 out[2];
    if constexpr (!LOCAL) {
      // my part of q_t.k_s: tiles (0, 0), (1, 0), (1, 1)
      if (wid < NP) {
        f32x4 p[3];
#pragma unroll
        for (int i = 0; i < 3; ++i) p[i] = (f32x4)0.f;
#pragma unroll
        for (int kt = 0; kt < KT / NP; ++kt) {
          f32x4 q[2], k[2];
#pragma unroll
          for (int m = 0; m < 2; ++m) {
            const int at = (m * 16 + i16) * ROW + (kt * NP + wid) * 16 + g * 4;
            q[m] = *reinterpret_cast<const f32x4*>(Ql + at);
            k[m] = *reinterpret_cast<const f32x4*>(Kl + at);
          }
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            p[0] = mfma4(q[0][r], k[0][r], p[0]);
            p[1] = mfma4(q[1][r], k[0][r], p[1]);
            p[2] = mfma4(q[1][r], k[1][r], p[2]);
          }
        }
#pragma unroll
        for (int i = 0; i < 3; ++i)
#pragma unroll
          for (int r = 0; r < 4; ++r)
            part[((wid * 3 + i) * 16 + g * 4 + r) * PROW + i16] = p[i][r];
      }
      // Q S
#pragma unroll
      for (int m = 0; m < 2; ++m) out[m] = (f32x4)0.f;
#pragma unroll
      for (int k = 0; k < KT; ++k) {
        f32x4 q[2];
#pragma unroll
        for (int m = 0; m < 2; ++m)
          q[m] = *reinterpret_cast<const f32x4*>(
              Ql + (m * 16 + i16) * ROW + k * 16 + g * 4);
#pragma unroll
        for (int r = 0; r < 4; ++r)
#pragma unroll
          for (int m = 0; m < 2; ++m)
            out[m] = mfma4(q[m][r], S[k][r], out[m]);
      }
      __syncthreads();
      for (int e = tid; e < 3 * 256; e += NT) {
        const int i = e / 256, x = e / 16 % 16, z = e % 16;
        const int t = (i > 0) * 16 + x, s = (i > 1) * 16 + z;
        float p = 0.f;
#pragma unroll
        for (int w = 0; w < NP; ++w) p += part[((w * 3 + i) * 16 + x) * PROW + z];
        Pl[t * TROW + s] = s <= t ? p * exp2_of(lg * (t - s)) : 0.f;
      }
      __syncthreads();
#pragma unroll
      for (int m = 0; m < 2; ++m) {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          out[m][r] *= exp2_of(lg * (m * 16 + g * 4 + r + 1));
#pragma unroll
        for (int k = 0; k <= m; ++k) {
          const f32x4 p = *reinterpret_cast<const f32x4*>(
              Pl + (m * 16 + i16) * TROW + k * 16 + g * 4);
#pragma unroll
          for (int r = 0; r < 4; ++r) out[m] = mfma4(p[r], v[k][r], out[m]);
        }
#pragma unroll
        for (int r = 0; r < 4; ++r)
          Ol[(m * 16 + g * 4 + r) * OROW + col] = out[m][r];
      }
    }
    // S <- g^n S + K^T (g^(n-1-s) V); rows behind the end have zero keys
    const float decay = cnt == CH ? glast : exp2_of(lg * cnt);
#pragma unroll
    for (int k = 0; k < KT; ++k)
#pragma unroll
      for (int e = 0; e < 4; ++e) S[k][e] *= decay;
#pragma unroll
    for (int m = 0; m < 2; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int s = m * 16 + g * 4 + r;
        const float w = v[m][r] * exp2_of(lg * max(cnt - 1 - s, 0));
        const float* kc = Kl + s * ROW + i16;
#pragma unroll
        for (int k = 0; k < KT; ++k) S[k] = mfma4(kc[k * 16], w, S[k]);
      }
    if constexpr (!LOCAL) {
      __syncthreads();
      const int t = tid / (VP / 8), c8 = tid % (VP / 8) * 8;
      float x[8];
      load8<float>(Ol + t * OROW + c8, x);
      float ss = 0.f;
#pragma unroll
      for (int i = 0; i < 8; ++i) ss += x[i] * x[i];
#pragma unroll
      for (int off = VP / 16; off > 0; off >>= 1)
        ss += __shfl_xor(ss, off, 64);
      const float inv = 1.f / sqrtf(ss / a.vdim + a.eps);
#pragma unroll
      for (int i = 0; i < 8; ++i) x[i] *= inv * silu(gt[i]);
      if (t < cnt)
        store8(a.y + ((row0 + c * CH + t) * a.H + head) * VP + c8, x);
    }
  }
  if (LOCAL || number + 1 == count) {
    float* to = LOCAL ? between + own * DP + g * 4 : slot;
#pragma unroll
    for (int k = 0; k < KT; ++k) *reinterpret_cast<f32x4*>(to + k * 16) = S[k];
  }
}

// The state before every piece of a segment in place of the pieces' own ones.
// longs [L, 2]: segment, its first piece.
__global__ void __launch_bounds__(256)
retention_join_kernel(const RetentionArgs<unsigned short> a,
                      const int* __restrict__ longs,
                      const int* __restrict__ pieces,
                      float* __restrict__ between, int numel) {
  const int lh = blockIdx.y, head = lh % a.H;
  const int seg = longs[lh / a.H * 2], first = longs[lh / a.H * 2 + 1];
  const int count = pieces[first * 5 + 4];
  const int e = (blockIdx.x * 256 + threadIdx.x) * 4;
  if (count == 1 || e >= numel) return;
  const float lg = a.decay[a.H + head];
  f32x4 run = (f32x4)0.f;
  if (a.ctx[a.seg_row0[seg]] > 1)
    run = *reinterpret_cast<const f32x4*>(
        a.state + ((long)a.seg_slot[seg] * a.H + head) * numel + e);
  float* b = between + ((long)first * a.H + head) * numel + e;
  for (int p = 0; p < count; ++p) {
    float* at = b + (long)p * a.H * numel;
    f32x4 own = (f32x4)0.f;
    if (p + 1 < count) own = *reinterpret_cast<const f32x4*>(at);
    *reinterpret_cast<f32x4*>(at) = run;
    const float decay = exp2_of(lg * pieces[(first + p) * 5 + 2]);
#pragma unroll
    for (int i = 0; i < 4; ++i) run[i] = decay * run[i] + own[i];
  }
}

extern "C" void launch_retention_scan(
    const void* ab, int ld, int H, int dp, int vp, int vdim, float kscale,
    float eps, const float* decay, const float* table, int half, float* state,
    void* y, const int* seg_row0, const int* seg_rows, const int* seg_slot,
    const int* ctx, int nseg, int max_rows, bool fp32, hipStream_t stream) {
  const int lpc = dp / 16;
  const int threads = min(1024, lpc * vp);
  const int ncol = lpc * vp / threads;
#define RS(T, L, N)                                                          \
  hipLaunchKernelGGL((retention_scan_kernel<T, L, N>), dim3(nseg * H),       \
                     dim3(threads), 0, stream,                               \
                     (RetentionArgs<T>{(const T*)ab, ld, H, vp, vdim, kscale, \
                                       eps, decay, table, half, state,       \
                                       (T*)y, seg_row0, seg_rows, seg_slot,  \
                                       ctx}),                                \
                     max_rows)
#define RS_N(T)                                \
  do {                                         \
    if (lpc == 4) RS(T, 4, 1);                 \
    else if (lpc == 8 && ncol == 1) RS(T, 8, 1); \
    else if (lpc == 8) RS(T, 8, 2);            \
    else if (ncol == 1) RS(T, 16, 1);          \
    else if (ncol == 2) RS(T, 16, 2);          \
    else RS(T, 16, 4);                         \
  } while (0)
  if (fp32) RS_N(float);
  else RS_N(unsigned short);
#undef RS_N
#undef RS
}

// several: some segment has more than one piece; between [npieces, H, vp, dp]
extern "C" void launch_retention_chunks(
    const void* ab, int ld, int H, int dp, int vp, int vdim, float kscale,
    float eps, const float* decay, const float* table, int half, float* state,
    void* y, const int* seg_row0, const int* seg_rows, const int* seg_slot,
    const int* ctx, const int* longs, int nlong, const int* pieces,
    int npieces, bool several, float* between, hipStream_t stream) {
  typedef unsigned short T;
  const RetentionArgs<T> a{(const T*)ab, ld,    H,    vp,    vdim,
                           kscale,       eps,   decay, table, half,
                           state,        (T*)y, seg_row0, seg_rows, seg_slot,
                           ctx};
#define RC(D, N, LOC, V)                                                     \
  do {                                                                       \
    constexpr int np = N < D / 16 ? N : D / 16;                              \
    constexpr int p = np * 3 * 16 * PROW, o = CH * (N * 16 + 4);             \
    const int lds =                                                          \
        (LOC ? CH * (D + 4)                                                  \
             : 2 * CH * (D + 4) + CH * TROW + (p > o ? p : o)) * 4;          \
    hipLaunchKernelGGL((retention_chunk_kernel<D, N, LOC, V>),               \
                       dim3(npieces * H), dim3(N * 64), lds, stream, a,      \
                       pieces, between);                                     \
  } while (0)
#define RC_V(D, N, LOC)              \
  do {                               \
    if (half % 8 == 0) RC(D, N, LOC, true); \
    else RC(D, N, LOC, false);       \
  } while (0)
#define RC_N(D, LOC)                   \
  do {                                 \
    if (vp == 64) RC_V(D, 4, LOC);     \
    else if (vp == 128) RC_V(D, 8, LOC); \
    else RC_V(D, 16, LOC);             \
  } while (0)
#define RC_D(LOC)                 \
  do {                            \
    if (dp == 64) RC_N(64, LOC);  \
    else if (dp == 128) RC_N(128, LOC); \
    else RC_N(256, LOC);          \
  } while (0)
  if (several) {
    RC_D(true);
    hipLaunchKernelGGL(retention_join_kernel,
                       dim3((dp * vp / 4 + 255) / 256, nlong * H), dim3(256),
                       0, stream, a, longs, pieces, between, dp * vp);
  }
  RC_D(false);
#undef RC_D
#undef RC_N
#undef RC_V
#undef RC
}
