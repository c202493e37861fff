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
//   retention_chunk_kernel  long segments, 32 rows at a time on the MFMA
//   retention_join_kernel   states between the pieces of a long segment
//   retention_wide_kernel   token by token, heads of more than 256 numbers
//
// With n the rows of a chunk and S the state before it (rows t, s from 0):
//   o_t = g^(t+1) S^T q_t + sum_{s<=t} g^(t-s) (q_t.k_s) v_s
//   S  <- g^n S + sum_s g^(n-1-s) k_s v_s^T
// A long segment may be cut into pieces that run side by side: first every
// piece but the last finds its state from zeros, then these are joined.
#include "common.h"

#define CH 32    // rows of a chunk
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
  const bool turn = c < 2 * half, low = c < half;
  const int i = !turn ? 0 : low ? c : c - half;  // its pair
  const float x = to_f(src[c]), y = to_f(src[low ? c + half : i]);
  const float2 t = reinterpret_cast<const float2*>(cs)[i];
  return turn ? x * t.x + (low ? -y : y) * t.y : x;
}

// ---- token by token -----------------------------------------------------------
// One workgroup per (segment, head). LPC lanes share a value column, each
// with 16 entries of the state's column in registers (float4 number i of
// lane `part` is float4 i * LPC + part of the column); a thread has NCOL
// columns. Rotated queries and keys of up to TT rows are staged in LDS.
// Segments of more than max_rows rows are left to the chunks.
#define TT 16

template <typename T, int LPC, int NCOL>
__global__ void __launch_bounds__(1024, 4)
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

  // number u of the queries and keys of rows t0 ..
  auto input = [&](int t0, int u) {
    const long row = row0 + t0 + u / (2 * dp);
    const int which = u / dp % 2;
    const float x = rotated(a.ab + row * a.ld + (which * a.H + head) * dp,
                            u % dp, a.half, a.table + row * a.half * 2);
    return which == 1 ? x * a.kscale : x;
  };
  // the first inputs are on their way before the state
  const int first = min(TT, n) * 2 * dp;
  const float x0 = (int)threadIdx.x < first ? input(0, threadIdx.x) : 0.f;
  float S[NCOL][16];
  const bool fresh = a.ctx[row0] <= 1;
#pragma unroll
  for (int c = 0; c < NCOL; ++c)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const f32x4 x = *reinterpret_cast<const f32x4*>(
          st + (long)(col0 + c * cstep) * dp + i * LPC * 4);
#pragma unroll
      for (int e = 0; e < 4; ++e) S[c][i * 4 + e] = fresh ? 0.f : x[e];
    }
  if ((int)threadIdx.x < first) (&qk[0][0][0])[threadIdx.x] = x0;

  for (int t0 = 0; t0 < n; t0 += TT) {
    const int cnt = min(TT, n - t0);
    if (t0 > 0) __syncthreads();  // the rows before are consumed
    for (int u = threadIdx.x + (t0 == 0 ? blockDim.x : 0); u < cnt * 2 * dp;
         u += blockDim.x)
      (&qk[0][0][0])[u] = input(t0, u);
    __syncthreads();
    for (int t = 0; t < cnt; ++t) {
      const long row = row0 + t0 + t;
      const T* vr = a.ab + row * a.ld + 2 * a.H * dp + head * a.vp;
      float v[NCOL], o[NCOL], gt[NCOL];
#pragma unroll
      for (int c = 0; c < NCOL; ++c) {
        v[c] = to_f(vr[col0 + c * cstep]);
        gt[c] = to_f(vr[a.H * a.vp + col0 + c * cstep]);
        o[c] = 0.f;
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int at = (i * LPC + part) * 4;
        const f32x4 q = *reinterpret_cast<const f32x4*>(&qk[t][0][at]);
        const f32x4 k = *reinterpret_cast<const f32x4*>(&qk[t][1][at]);
#pragma unroll
        for (int c = 0; c < NCOL; ++c)
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            float& s = S[c][i * 4 + e];
            s = g * s + k[e] * v[c];
            o[c] += s * q[e];
          }
      }
      float ss = 0.f;
#pragma unroll
      for (int c = 0; c < NCOL; ++c) {
#pragma unroll
        for (int off = LPC / 2; off > 0; off >>= 1)
          o[c] += __shfl_xor(o[c], off, 64);
        ss += part == 0 ? o[c] * o[c] : 0.f;
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
          from_f(a.y + (row * a.H + head) * a.vp + col0 + c * cstep,
                 o[c] * inv * gate_silu<T>(gt[c]));
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
// The products run on the bf16 MFMA without giving up fp32: a number is the
// sum of three bf16 numbers, its leading bits, the next and the last eight of
// 24 (values are bf16 already). A product of two such sums takes the six
// products of parts that reach beyond the last bit.
typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;

struct Parts {
  unsigned int p[3];
};

// two neighbours; every part is packed like two bf16 in memory
__device__ __forceinline__ Parts split2(float x0, float x1) {
  Parts out;
#pragma unroll
  for (int i = 0; i < 3; ++i) {
    const unsigned int u0 = __float_as_uint(x0), u1 = __float_as_uint(x1);
    out.p[i] = __builtin_amdgcn_perm(u1, u0, 0x07060302);
    x0 -= __uint_as_float(u0 & 0xffff0000u);
    x1 -= __uint_as_float(u1 & 0xffff0000u);
  }
  return out;
}

__device__ __forceinline__ f32x4 mfma_bf(bf16x8 a, bf16x8 b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}

// a . b of two numbers in parts, smallest terms first
__device__ __forceinline__ f32x4 mfma_parts(const bf16x8 (&a)[3],
                                            const bf16x8 (&b)[3], f32x4 c) {
  c = mfma_bf(a[2], b[0], c);
  c = mfma_bf(a[0], b[2], c);
  c = mfma_bf(a[1], b[1], c);
  c = mfma_bf(a[1], b[0], c);
  c = mfma_bf(a[0], b[1], c);
  return mfma_bf(a[0], b[0], c);
}

__device__ __forceinline__ float exp2_of(float x) {
  return __builtin_amdgcn_exp2f(x);
}

// Place of number d of a row of keys or queries in LDS: within 32 numbers,
// those that a lane group g finds in two accumulators of the state (4 g ..
// 4 g + 3 and 16 + 4 g ..) are neighbours, so that the state's accumulators
// are the right operand of the next product as they are.
__device__ __forceinline__ int lds_place(int d) {
  const int w = d & 31, h = w >> 4;
  return (d & ~31) + ((w & 15) >> 2) * 8 + h * 4 + (w & 3);
}

// pieces [P, 5]: segment, first row in it, rows, number, pieces of the
// segment. One workgroup per (piece, head), a wave for each 32 value columns
// (its part of the state, DP x 32, is DP / 8 accumulators).
//   LOCAL  the piece's state from zeros, to between[piece]; not for the last
//          piece of a segment
//   else   the outputs, from the slot's state or (several pieces) from
//          between[piece]; the last piece writes the slot
// The rotated queries and keys of a chunk are kept in parts in LDS, by rows
// and, weighted with their decay to the chunk's end, keys by numbers; the
// next chunk is on its way in registers meanwhile. For the scores the waves
// split the inner dimension; their sums meet in LDS.
//
// A thread's unit of keys and queries is four rows by four numbers: two
// neighbours and their rotation partners, or four that do not rotate. VEC:
// half is even; else units are read number by number.
template <int DP, int VP>
struct ChunkLds {
  static constexpr int NW = VP / 32;
  static constexpr int KJ = DP / 32;
  static constexpr int NP = NW < KJ ? NW : KJ;  // waves that form scores
  static constexpr int ROW_B = DP * 2 + 16;     // a row of one part
  static constexpr int Q_B = 3 * CH * ROW_B;
  static constexpr int T_B = 3 * DP * CH * 2;   // by numbers
  static constexpr int K_B = Q_B > T_B ? Q_B : T_B;
  static constexpr int P_ROW = CH * 2 + 16;
  static constexpr int P_B = 3 * CH * P_ROW;
  static constexpr int O_ROW = VP + 4;          // floats
  static constexpr int S_B = NP * 3 * 16 * PROW * 4;
  static constexpr int O_B = CH * O_ROW * 4;
  static constexpr int BYTES = Q_B + K_B + P_B + (S_B > O_B ? S_B : O_B);
};

template <int DP, int VP, bool LOCAL, bool VEC>
__global__ void __launch_bounds__(VP * 2, DP <= 128 && VP > 64 ? 2 : 1)
retention_chunk_kernel(const RetentionArgs<unsigned short> a,
                       const int* __restrict__ pieces,
                       float* __restrict__ between) {
  typedef unsigned short T;
  typedef ChunkLds<DP, VP> L;
  constexpr int NW = L::NW, NT = NW * 64, KT = DP / 16, KJ = L::KJ;
  constexpr int NP = L::NP;
  constexpr int UNITS = CH / 4 * (DP / 4);
  constexpr int NS = (UNITS + NT - 1) / NT;
  constexpr int LPR = VP / 16;   // lanes that share an output row
  char* Kl = smem;               // rows [3][CH], then numbers [3][DP]
  char* Ql = Kl + (LOCAL ? L::T_B : L::K_B);
  char* Pl = Ql + L::Q_B;
  float* part = reinterpret_cast<float*>(Pl + L::P_B);  // [NP][3][16][PROW]
  float* Ol = part;                                     // later

  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
  const int i16 = lane & 15, g = lane >> 4;
  const int piece = blockIdx.x / a.H, head = blockIdx.x % a.H;
  const int* pc = pieces + piece * 5;
  const int seg = pc[0], n = pc[2], number = pc[3], count = pc[4];
  if (LOCAL && number + 1 == count) return;
  const long row0 = a.seg_row0[seg] + pc[1];
  const int nch = (n + CH - 1) / CH;
  const float lg = a.decay[a.H + head];
  const int at_q = head * DP, at_k = (a.H + head) * DP;
  const int at_v = 2 * a.H * DP + head * VP, at_g = at_v + a.H * VP;

  // numbers d[0], d[0] + 1, d[1], d[1] + 1 of rows t .. t + 3 of the chunk
  struct Unit {
    int d[2], t;
    bool turn, live;
  };
  auto unit = [&](int i) {
    const int u = tid + i * NT, q = u % (DP / 4) * 2;
    Unit x;
    x.t = u / (DP / 4) * 4;
    x.live = UNITS % NT == 0 || u < UNITS;
    if constexpr (VEC) {
      x.turn = q < a.half;
      x.d[0] = x.turn ? q : q + a.half;
      x.d[1] = x.turn ? q + a.half : q + DP / 2;
    } else {
      x.turn = true;
      x.d[0] = q;
      x.d[1] = q + DP / 2;
    }
    return x;
  };
  unsigned int rk[NS][4][2], rq[NS][4][2];
  f32x4 cs[NS][4];
  auto fetch = [&](int c) {
    if constexpr (VEC) {
      const int cnt = min(CH, n - c * CH);
#pragma unroll
      for (int i = 0; i < NS; ++i) {
        const Unit x = unit(i);
        if (!x.live) break;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const long row = row0 + c * CH + min(x.t + e, cnt - 1);
          const T* src = a.ab + row * a.ld;
#pragma unroll
          for (int j = 0; j < 2; ++j) {
            rk[i][e][j] = *reinterpret_cast<const unsigned int*>(
                src + at_k + x.d[j]);
            if (!LOCAL)
              rq[i][e][j] = *reinterpret_cast<const unsigned int*>(
                  src + at_q + x.d[j]);
          }
          if (x.turn)
            cs[i][e] = *reinterpret_cast<const f32x4*>(
                a.table + (row * a.half + x.d[0]) * 2);
        }
      }
    }
  };
  // row e of unit i, rotated; zeros behind the end
  auto turned = [&](int c, int i, const Unit& x, int e, bool key, float* z) {
    const int cnt = min(CH, n - c * CH);
    if constexpr (VEC) {
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        const unsigned int r = key ? rk[i][e][j] : rq[i][e][j];
        z[j * 2] = __uint_as_float(r << 16);
        z[j * 2 + 1] = __uint_as_float(r & 0xffff0000u);
      }
      if (x.turn)
#pragma unroll
        for (int j = 0; j < 2; ++j) {
          const float p = z[j], q = z[2 + j];
          const float cv = cs[i][e][2 * j], sv = cs[i][e][2 * j + 1];
          z[j] = p * cv - q * sv;
          z[2 + j] = q * cv + p * sv;
        }
    } else {
      const long row = row0 + c * CH + min(x.t + e, cnt - 1);
      const T* src = a.ab + row * a.ld + (key ? at_k : at_q);
#pragma unroll
      for (int j = 0; j < 4; ++j)
        z[j] = rotated(src, x.d[j >> 1] + (j & 1), a.half,
                       a.table + row * a.half * 2);
    }
    const float f = x.t + e >= cnt ? 0.f : key ? a.kscale : 1.f;
#pragma unroll
    for (int j = 0; j < 4; ++j) z[j] *= f;
  };
  float kz[NS][4][4];  // the chunk's keys
  auto stage = [&](int c) {
#pragma unroll
    for (int i = 0; i < NS; ++i) {
      const Unit x = unit(i);
      if (!x.live) break;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        turned(c, i, x, e, true, kz[i][e]);
        if constexpr (!LOCAL) {
          float z[4];
          turned(c, i, x, e, false, z);
#pragma unroll
          for (int j = 0; j < 2; ++j) {
            char* dst = Kl + (x.t + e) * L::ROW_B + lds_place(x.d[j]) * 2;
            const Parts k = split2(kz[i][e][j * 2], kz[i][e][j * 2 + 1]);
            const Parts q = split2(z[j * 2], z[j * 2 + 1]);
#pragma unroll
            for (int p = 0; p < 3; ++p) {
              const int at = p * CH * L::ROW_B;
              *reinterpret_cast<unsigned int*>(dst + at) = k.p[p];
              *reinterpret_cast<unsigned int*>(dst + (Ql - Kl) + at) = q.p[p];
            }
          }
        }
      }
    }
  };
  // keys by numbers, eight rows in a 16-byte piece, weighted with
  // g^(cnt-1-s)
  auto stage_numbers = [&](int cnt) {
#pragma unroll
    for (int i = 0; i < NS; ++i) {
      const Unit x = unit(i);
      if (!x.live) break;
      float w[4];
#pragma unroll
      for (int e = 0; e < 4; ++e)
        w[e] = exp2_of(lg * max(cnt - 1 - x.t - e, 0));
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int d = x.d[j >> 1] + (j & 1);
        const Parts lo = split2(kz[i][0][j] * w[0], kz[i][1][j] * w[1]);
        const Parts hi = split2(kz[i][2][j] * w[2], kz[i][3][j] * w[3]);
        char* dst = Kl + d * (CH * 2) +
                    (((x.t >> 3) ^ ((d >> 2) & 3)) * 16) + (x.t & 4) * 2;
#pragma unroll
        for (int p = 0; p < 3; ++p)
          *reinterpret_cast<i32x2*>(dst + p * DP * (CH * 2)) =
              i32x2{(int)lo.p[p], (int)hi.p[p]};
      }
    }
  };
  auto row_frags = [&](const char* base, int t, int j, bf16x8 (&f)[3]) {
#pragma unroll
    for (int p = 0; p < 3; ++p)
      f[p] = *reinterpret_cast<const bf16x8*>(
          base + (p * CH + t) * L::ROW_B + j * 64 + g * 16);
  };

  f32x4 S[KT][2];
  const long own = ((long)piece * a.H + head) * VP + wid * 32 + i16;
  float* slot = a.state +
                (((long)a.seg_slot[seg] * a.H + head) * VP + wid * 32 + i16) *
                    DP + g * 4;
  const float* from = count > 1 ? between + own * DP + g * 4 : slot;
  const bool zero = LOCAL || (count == 1 && a.ctx[row0] <= 1);
#pragma unroll
  for (int k = 0; k < KT; ++k)
#pragma unroll
    for (int ct = 0; ct < 2; ++ct) {
      S[k][ct] = (f32x4)0.f;
      if (!zero)
        S[k][ct] =
            *reinterpret_cast<const f32x4*>(from + ct * 16 * DP + k * 16);
    }

  fetch(0);
  for (int c = 0; c < nch; ++c) {
    const int cnt = min(CH, n - c * CH);
    if (LOCAL && c > 0) __syncthreads();  // the chunk before is consumed
    stage(c);
    if (LOCAL) stage_numbers(cnt);
    __syncthreads();
    T vr[2][8];  // values of my columns, rows g * 8 ..
#pragma unroll
    for (int ct = 0; ct < 2; ++ct)
#pragma unroll
      for (int e = 0; e < 8; ++e)
        vr[ct][e] = a.ab[(row0 + c * CH + min(g * 8 + e, cnt - 1)) * a.ld +
                         at_v + wid * 32 + ct * 16 + i16];
    if (c + 1 < nch) fetch(c + 1);

    s16x8 gr[2];
    f32x4 out[2][2];
    if constexpr (!LOCAL) {
      // my part of q_t.k_s: tiles (0, 0), (1, 0), (1, 1)
      if (wid < NP) {
        f32x4 p[3];
#pragma unroll
        for (int i = 0; i < 3; ++i) p[i] = (f32x4)0.f;
#pragma unroll
        for (int jj = 0; jj < KJ / NP; ++jj) {
          bf16x8 q[2][3], k[2][3];
#pragma unroll
          for (int m = 0; m < 2; ++m) {
            row_frags(Ql, m * 16 + i16, jj * NP + wid, q[m]);
            row_frags(Kl, m * 16 + i16, jj * NP + wid, k[m]);
          }
          p[0] = mfma_parts(q[0], k[0], p[0]);
          p[1] = mfma_parts(q[1], k[0], p[1]);
          p[2] = mfma_parts(q[1], k[1], p[2]);
        }
#pragma unroll
        for (int i = 0; i < 3; ++i)
#pragma unroll
          for (int r = 0; r < 4; ++r)
            part[((wid * 3 + i) * 16 + g * 4 + r) * PROW + i16] = p[i][r];
      }
      // Q S
#pragma unroll
      for (int m = 0; m < 2; ++m)
#pragma unroll
        for (int ct = 0; ct < 2; ++ct) out[m][ct] = (f32x4)0.f;
#pragma unroll
      for (int j = 0; j < KJ; ++j) {
        bf16x8 q[2][3], s[2][3];
#pragma unroll
        for (int m = 0; m < 2; ++m) row_frags(Ql, m * 16 + i16, j, q[m]);
#pragma unroll
        for (int ct = 0; ct < 2; ++ct) {
          i32x4 x[3];
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            const f32x4& t = S[2 * j + (e >> 1)][ct];
            const Parts y = split2(t[(e & 1) * 2], t[(e & 1) * 2 + 1]);
#pragma unroll
            for (int p = 0; p < 3; ++p) x[p][e] = (int)y.p[p];
          }
#pragma unroll
          for (int p = 0; p < 3; ++p)
            s[ct][p] = __builtin_bit_cast(bf16x8, x[p]);
        }
#pragma unroll
        for (int m = 0; m < 2; ++m)
#pragma unroll
          for (int ct = 0; ct < 2; ++ct)
            out[m][ct] = mfma_parts(q[m], s[ct], out[m][ct]);
      }
      const T* src = a.ab +
                     (row0 + c * CH + min(tid / LPR, cnt - 1)) * a.ld + at_g +
                     tid % LPR * 16;
      gr[0] = *reinterpret_cast<const s16x8*>(src);
      gr[1] = *reinterpret_cast<const s16x8*>(src + 8);
      __syncthreads();  // the keys' rows are consumed
      stage_numbers(cnt);
#pragma unroll 1
      for (int e0 = 0; e0 < CH * CH / 2; e0 += NT) {
        const int t = (e0 + tid) / 16, s = (e0 + tid) % 16 * 2;
        if (NT > CH * CH / 2 && t >= CH) break;
        float2 p = {0.f, 0.f};
        if (s <= t) {
          const int i = (t >> 4) + (s >> 4);
          const float* at = part + (i * 16 + (t & 15)) * PROW + (s & 15);
#pragma unroll
          for (int w = 0; w < NP; ++w) {
            const float2 x =
                *reinterpret_cast<const float2*>(at + w * 3 * 16 * PROW);
            p.x += x.x;
            p.y += x.y;
          }
          p.x *= exp2_of(lg * (t - s));
          p.y = s < t ? p.y * exp2_of(lg * (t - s - 1)) : 0.f;
        }
        const Parts x = split2(p.x, p.y);
#pragma unroll
        for (int i = 0; i < 3; ++i)
          *reinterpret_cast<unsigned int*>(Pl + (i * CH + t) * L::P_ROW +
                                           s * 2) = x.p[i];
      }
      __syncthreads();
    }
    bf16x8 v[2];
#pragma unroll
    for (int ct = 0; ct < 2; ++ct) {
      s16x8 x;
#pragma unroll
      for (int e = 0; e < 8; ++e) x[e] = (short)vr[ct][e];
      v[ct] = __builtin_bit_cast(bf16x8, x);
    }
    if constexpr (!LOCAL) {
#pragma unroll
      for (int m = 0; m < 2; ++m) {
        float w[4];
#pragma unroll
        for (int r = 0; r < 4; ++r)
          w[r] = exp2_of(lg * (m * 16 + g * 4 + r + 1));
        bf16x8 p[3];
#pragma unroll
        for (int i = 0; i < 3; ++i)
          p[i] = *reinterpret_cast<const bf16x8*>(
              Pl + (i * CH + m * 16 + i16) * L::P_ROW + g * 16);
#pragma unroll
        for (int ct = 0; ct < 2; ++ct) {
#pragma unroll
          for (int r = 0; r < 4; ++r) out[m][ct][r] *= w[r];
#pragma unroll
          for (int i = 2; i >= 0; --i)
            out[m][ct] = mfma_bf(p[i], v[ct], out[m][ct]);
#pragma unroll
          for (int r = 0; r < 4; ++r)
            Ol[(m * 16 + g * 4 + r) * L::O_ROW + wid * 32 + ct * 16 + i16] =
                out[m][ct][r];
        }
      }
    }
    // S <- g^n S + K^T V, keys weighted; rows behind the end have zero keys
    const float decay = exp2_of(lg * cnt);
#pragma unroll
    for (int k = 0; k < KT; ++k) {
      const int d = k * 16 + i16;
      bf16x8 x[3];
#pragma unroll
      for (int p = 0; p < 3; ++p)
        x[p] = *reinterpret_cast<const bf16x8*>(
            Kl + (p * DP + d) * (CH * 2) + ((g ^ ((d >> 2) & 3)) * 16));
#pragma unroll
      for (int ct = 0; ct < 2; ++ct) {
#pragma unroll
        for (int e = 0; e < 4; ++e) S[k][ct][e] *= decay;
#pragma unroll
        for (int p = 2; p >= 0; --p)
          S[k][ct] = mfma_bf(x[p], v[ct], S[k][ct]);
      }
    }
    if constexpr (!LOCAL) {
      __syncthreads();
      const int t = tid / LPR, c16 = tid % LPR * 16;
      float x[16], gate[16];
      load8<float>(Ol + t * L::O_ROW + c16, x);
      load8<float>(Ol + t * L::O_ROW + c16 + 8, x + 8);
      bf8_to_f32(gr[0], gate);
      bf8_to_f32(gr[1], gate + 8);
      float ss = 0.f;
#pragma unroll
      for (int i = 0; i < 16; ++i) ss += x[i] * x[i];
#pragma unroll
      for (int off = LPR / 2; off > 0; off >>= 1)
        ss += __shfl_xor(ss, off, 64);
      const float inv = 1.f / sqrtf(ss / a.vdim + a.eps);
#pragma unroll
      for (int i = 0; i < 16; ++i) x[i] *= inv * silu(gate[i]);
      if (t < cnt) {
        T* dst = a.y + ((row0 + c * CH + t) * a.H + head) * VP + c16;
        store8(dst, x);
        store8(dst + 8, x + 8);
      }
    }
  }
  if (LOCAL || number + 1 == count) {
    float* to = LOCAL ? between + own * DP + g * 4 : slot;
#pragma unroll
    for (int k = 0; k < KT; ++k)
#pragma unroll
      for (int ct = 0; ct < 2; ++ct)
        *reinterpret_cast<f32x4*>(to + ct * 16 * DP + k * 16) = S[k][ct];
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

// Any multiple of 64 as head size: one workgroup per (segment, head), the
// state stays in memory, a thread goes down the columns of its own.
template <typename T>
__global__ void __launch_bounds__(256)
retention_wide_kernel(const RetentionArgs<T> a, int dp) {
  __shared__ float scratch[4];
  float* q = reinterpret_cast<float*>(smem);  // [dp], then k [dp], o [vp]
  float *k = q + dp, *o = k + dp;
  const int seg = blockIdx.x / a.H, head = blockIdx.x % a.H;
  const int n = a.seg_rows[seg];
  if (n == 0) return;
  const int row0 = a.seg_row0[seg];
  const float g = a.decay[head];
  float* st =
      a.state + ((long)a.seg_slot[seg] * a.H + head) * a.vp * dp;
  const bool fresh = a.ctx[row0] <= 1;
  for (int t = 0; t < n; ++t) {
    const long row = row0 + t;
    const T* r = a.ab + row * a.ld;
    const float* cs = a.table + row * a.half * 2;
    __syncthreads();  // the row before is done
    for (int c = threadIdx.x; c < dp; c += 256) {
      q[c] = rotated(r + head * dp, c, a.half, cs);
      k[c] = rotated(r + (a.H + head) * dp, c, a.half, cs) * a.kscale;
    }
    __syncthreads();
    r += 2 * a.H * dp + head * a.vp;
    float ss = 0.f;
    for (int c = threadIdx.x; c < a.vp; c += 256) {
      float* s = st + (long)c * dp;
      const float v = to_f(r[c]);
      float x = 0.f;
      for (int d = 0; d < dp; d += 4) {
        f32x4 y = (f32x4)0.f;
        if (t > 0 || !fresh) y = *reinterpret_cast<const f32x4*>(s + d);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          y[e] = g * y[e] + k[d + e] * v;
          x += y[e] * q[d + e];
        }
        *reinterpret_cast<f32x4*>(s + d) = y;
      }
      o[c] = x;
      ss += x * x;
    }
    ss = block_reduce_sum<4>(ss, scratch);
    const float inv = 1.f / sqrtf(ss / a.vdim + a.eps);
    for (int c = threadIdx.x; c < a.vp; c += 256)
      from_f(a.y + (row * a.H + head) * a.vp + c,
             o[c] * inv * gate_silu<T>(to_f(r[a.H * a.vp + c])));
  }
}

extern "C" void launch_retention_wide(
    const void* ab, int ld, int H, int dp, int vp, int vdim, float kscale,
    float eps, const float* decay, const float* table, int half, float* state,
    void* y, const int* seg_row0, const int* seg_rows, const int* seg_slot,
    const int* ctx, int nseg, bool fp32, hipStream_t stream) {
#define RW(T)                                                                 \
  hipLaunchKernelGGL((retention_wide_kernel<T>), dim3(nseg * H), dim3(256),   \
                     (2 * dp + vp) * 4, stream,                               \
                     (RetentionArgs<T>{(const T*)ab, ld, H, vp, vdim, kscale, \
                                       eps, decay, table, half, state,        \
                                       (T*)y, seg_row0, seg_rows, seg_slot,   \
                                       ctx}),                                 \
                     dp)
  if (fp32) RW(float);
  else RW(unsigned short);
#undef RW
}

extern "C" void launch_retention_scan(
    const void* ab, int ld, int H, int dp, int vp, int vdim, float kscale,
    float eps, const float* decay, const float* table, int half, float* state,
    void* y, const int* seg_row0, const int* seg_rows, const int* seg_slot,
    const int* ctx, int nseg, int max_rows, bool fp32, hipStream_t stream) {
  // workgroups of 256 threads where these can hold the state: several on a
  // CU hide one another's round trips
  const int lpc = dp / 16;
  const int threads = min(1024, max(256, lpc * vp / 2));
  const int ncol = lpc * vp / threads;
#define RS(T, L, N)                                                          \
  hipLaunchKernelGGL((retention_scan_kernel<T, L, N>), dim3(nseg * H),       \
                     dim3(threads), 0, stream,                               \
                     (RetentionArgs<T>{(const T*)ab, ld, H, vp, vdim, kscale, \
                                       eps, decay, table, half, state,       \
                                       (T*)y, seg_row0, seg_rows, seg_slot,  \
                                       ctx}),                                \
                     max_rows)
#define RS_N(T, L)          \
  do {                      \
    if (ncol == 1) RS(T, L, 1); \
    else if (ncol == 2) RS(T, L, 2); \
    else RS(T, L, 4);       \
  } while (0)
#define RS_L(T)                  \
  do {                           \
    if (lpc == 4) RS_N(T, 4);    \
    else if (lpc == 8) RS_N(T, 8); \
    else RS_N(T, 16);            \
  } while (0)
  if (fp32) RS_L(float);
  else RS_L(unsigned short);
#undef RS_L
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
    typedef ChunkLds<D, N> L;                                                \
    hipLaunchKernelGGL((retention_chunk_kernel<D, N, LOC, V>),               \
                       dim3(npieces * H), dim3(N * 2),                       \
                       LOC ? L::T_B : L::BYTES, stream, a, pieces, between); \
  } while (0)
#define RC_V(D, N, LOC)                     \
  do {                                      \
    if (half % 2 == 0) RC(D, N, LOC, true); \
    else RC(D, N, LOC, false);              \
  } while (0)
#define RC_N(D, LOC)                     \
  do {                                   \
    if (vp == 64) RC_V(D, 64, LOC);      \
    else if (vp == 128) RC_V(D, 128, LOC); \
    else RC_V(D, 256, LOC);              \
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
