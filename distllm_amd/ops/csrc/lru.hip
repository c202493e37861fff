// Real-gated linear recurrent unit of a ragged step, per channel:
//   r = sigmoid(Wr u + br), i = sigmoid(Wi u + bi)   (block-diagonal W)
//   log a = decay * r;  S <- a S + sqrt(1 - a^2) i u;  out = S * gelu(y)
// u is the causal convolution of the projection's second half, y its first.
//
//   lru_conv_kernel   u
//   lru_gates_kernel  both gate products on the MFMA and everything up to
//                     the recurrence; rows of short segments: a and the
//                     drive; chunks of long ones: their recurrence from
//                     zeros and the product of the decays so far, times
//                     which a state before the chunk is added
//   lru_scan_kernel   short segments, row by row
//   lru_carry_kernel  long segments: state before every chunk
//   lru_emit_kernel   long segments: output
// Everything behind u and y is fp32. The 32-bit mode takes every segment row
// by row, with its gates from lru_gates32_kernel.
#include "short_conv.h"

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;

#define LCH 64  // rows of a chunk
#define LOG2E 1.4426950408889634f

template <typename T>
__device__ __forceinline__ float gelu_of(float x) {
  if constexpr (sizeof(T) == 2) return fast_gelu(x);
  else return gelu_exact(x);
}

// a thread: eight channels of a run of rows
template <typename T, int TAPS>
__global__ void __launch_bounds__(256)
lru_conv_kernel(ConvArgs<T> a, const float* __restrict__ bias,
                T* __restrict__ u) {
  constexpr int NT = TAPS > 0 ? TAPS : 1;
  const int vec = a.C / 8;
  const long id = (long)blockIdx.x * 256 + threadIdx.x;
  const int ch = (int)(id % vec) * 8;
  const long r0 = id / vec * a.rb;
  if (r0 >= a.M) return;
  float w[NT][8], x[NT][8], b[8];  // x[j]: the input j rows back
  load8<float>(bias + ch, b);
  if (TAPS > 0)
#pragma unroll
    for (int j = 0; j < NT; ++j)
      load8<float>(a.w + (long)(NT - 1 - j) * a.C + ch, w[j]);
  int before = -1;  // sequence of the previous row
  for (int row = (int)r0; row < min((int)r0 + a.rb, a.M); ++row) {
    const int pos = a.ctx[row] - 1;
    float z[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) z[i] = b[i];
    if (pos < 0) {  // a padding row
      before = -1;
      store8(u + (long)row * a.C + ch, z);
      continue;
    }
    const int seg = a.row_seq[row];
    const int o = row - a.seg_row0[seg];
    T* slot = a.conv + (long)a.seg_slot[seg] * (a.taps - 1) * a.C + ch;
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
    store8(u + (long)row * a.C + ch, z);
  }
}

// sqrt(1 - a^2) of a = exp2(la2) <= 1, also where la2 is tiny
__device__ __forceinline__ float drive_factor(float la2, float a) {
  const float z = la2 * 1.3862943611198906f;
  const float near = -z * (1.f + z * (0.5f + z * 0.16666667f));
  return __builtin_amdgcn_sqrtf(z > -0.03f ? near : 1.f - a * a);
}

struct LruGates {
  const float *br, *bi, *decay;
  const int *seg_row0, *seg_rows, *row_seq, *ctx;
  int M, C, blocks, bs, max_rows;
};

// Weights of both gates lie in the order in which the MFMA takes them:
// [gate, block, 32 outputs, 32 inputs, j, g, i, e], output i * 2 + j of the
// 32 and input g * 8 + e of the 32: a lane gets two neighbouring channels.
__device__ __forceinline__ long gate_at(const LruGates& a, int z, int blk,
                                        int n, int k) {
  const long tile =
      (((long)z * a.blocks + blk) * (a.bs / 32) + n / 32) * (a.bs / 32) +
      k / 32;
  return tile * 1024 + n % 2 * 512 + (k % 32 / 8 * 16 + n % 32 / 2) * 8 +
         k % 8;
}

#define PIECE 256        // inner indices that are staged in LDS at once
#define UROW (PIECE + 8)  // padded LDS row

// A wave: MT * 16 rows and 32 channels of both gates; a workgroup: four
// neighbouring groups of 32 channels. LONG: the rows are a chunk; else they
// are 16 consecutive rows, of which those of short segments count. SHARED:
// the workgroup's channels are of one block, and its u passes through LDS.
template <int MT, bool LONG, bool SHARED>
__global__ void __launch_bounds__(256, 3)
lru_gates_kernel(const unsigned short* __restrict__ u,
                 const unsigned short* __restrict__ w, const LruGates a,
                 const int* __restrict__ chunks, int groups,
                 float* __restrict__ prod, float* __restrict__ hs) {
  __shared__ __attribute__((aligned(16)))
  unsigned short ul[SHARED ? MT * 16 * UROW : 1];
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int i16 = lane & 15, g = lane >> 4;
  // an XCD keeps to neighbouring groups, whose weights stay in its L2
  int tile = blockIdx.x / groups, group = blockIdx.x % groups;
  if (groups % 8 == 0) {
    const int own = groups / 8, i = blockIdx.x / 8;
    tile = i / own;
    group = blockIdx.x % 8 * own + i % own;
  }
  const int c0 = (group * 4 + wid) * 32;
  if (!SHARED && c0 >= a.C) return;
  long row0;
  int cnt;
  if (LONG) {
    const int seg = chunks[tile * 2], c = chunks[tile * 2 + 1];
    row0 = a.seg_row0[seg] + c * LCH;
    cnt = min(LCH, a.seg_rows[seg] - c * LCH);
  } else {
    row0 = (long)tile * 16;
    cnt = min(16, a.M - tile * 16);
  }
  // rows that count, one bit each
  unsigned long long live = ~0ull;
  if (!LONG) {
    bool mine = false;
    if (i16 < cnt)
      mine = a.ctx[row0 + i16] > 0 &&
             a.seg_rows[a.row_seq[row0 + i16]] <= a.max_rows;
    live = __ballot(mine);
    if (live == 0) return;  // the same in every wave
  }

  f32x4 acc[2][2][MT];  // gate, channel i16 * 2 + j, row tile
#pragma unroll
  for (int z = 0; z < 2; ++z)
#pragma unroll
    for (int j = 0; j < 2; ++j)
#pragma unroll
      for (int m = 0; m < MT; ++m) acc[z][j][m] = (f32x4)0.f;
  const bool real = c0 < a.blocks * a.bs;  // else a column of padding
  if (SHARED || real) {
    const int blk = c0 / a.bs, n0 = c0 % a.bs;
    const unsigned short* wr[2][2];
#pragma unroll
    for (int z = 0; z < 2; ++z)
#pragma unroll
      for (int j = 0; j < 2; ++j)
        wr[z][j] = w + gate_at(a, z, blk, n0 + j, 0) + lane * 8;
    for (int p0 = 0; p0 < a.bs; p0 += PIECE) {
      const int len = SHARED ? min(PIECE, a.bs - p0) : PIECE;
      if (SHARED) {
        __syncthreads();  // the previous piece is consumed
        for (int i = threadIdx.x; i < MT * 16 * (PIECE / 8); i += 256) {
          const int row = i / (PIECE / 8), c = i % (PIECE / 8) * 8;
          if (c < len)
            *reinterpret_cast<i32x4*>(ul + row * UROW + c) =
                *reinterpret_cast<const i32x4*>(
                    u + (row0 + min(row, cnt - 1)) * a.C + blk * a.bs + p0 +
                    c);
        }
        __syncthreads();
      }
#pragma unroll 2
      for (int k = p0; k < min(p0 + PIECE, a.bs); k += 32) {
        bf16x8 uf[MT], wf[2][2];
#pragma unroll
        for (int z = 0; z < 2; ++z)
#pragma unroll
          for (int j = 0; j < 2; ++j)
            wf[z][j] =
                *reinterpret_cast<const bf16x8*>(wr[z][j] + (long)k * 32);
#pragma unroll
        for (int m = 0; m < MT; ++m) {
          const int t = m * 16 + i16;
          uf[m] = *reinterpret_cast<const bf16x8*>(
              SHARED ? ul + t * UROW + k - p0 + g * 8
                     : u + (row0 + min(t, cnt - 1)) * a.C + blk * a.bs + k +
                           g * 8);
        }
#pragma unroll
        for (int z = 0; z < 2; ++z)
#pragma unroll
          for (int j = 0; j < 2; ++j)
#pragma unroll
            for (int m = 0; m < MT; ++m)
              acc[z][j][m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                  uf[m], wf[z][j], acc[z][j][m], 0, 0, 0);
      }
    }
  }

  // Offsets from the first row, in 32 bits; a lane has rows g * 4 + r of
  // every row tile and channels c, c + 1.
  const int c = c0 + i16 * 2;
  const unsigned short* ub = u + row0 * a.C + c;
  float *pb = prod + row0 * a.C + c, *hb = hs + row0 * a.C + c;
  const bool full = real && cnt == MT * 16;
  unsigned uv[MT][4];  // two bf16
#pragma unroll
  for (int m = 0; m < MT; ++m)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const unsigned t = m * 16 + g * 4 + r;
      uv[m][r] = *reinterpret_cast<const unsigned*>(
          ub + (full ? t : min(t, (unsigned)cnt - 1)) * (unsigned)a.C);
    }
  // decays and drives; rows behind the end keep the state as it is
  f32x4 ea[2][MT], x[2][MT];
#pragma unroll
  for (int j = 0; j < 2; ++j) {
    const float br = -LOG2E * a.br[c + j], bi = -LOG2E * a.bi[c + j];
    const float decay = LOG2E * a.decay[c + j];
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float zr = fmaf(acc[0][j][m][r], -LOG2E, br);
        const float zi = fmaf(acc[1][j][m][r], -LOG2E, bi);
        const float la =
            decay * fast_rcp(1.f + __builtin_amdgcn_exp2f(zr));
        const float e = __builtin_amdgcn_exp2f(la);
        const float d =
            drive_factor(la, e) *
            bf2f((unsigned short)(j ? uv[m][r] >> 16 : uv[m][r])) *
            fast_rcp(1.f + __builtin_amdgcn_exp2f(zi));
        const bool ok = full || (real && m * 16 + g * 4 + r < cnt);
        ea[j][m][r] = ok ? e : 1.f;
        x[j][m][r] = ok ? d : 0.f;
      }
  }
  if (!LONG) {
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = g * 4 + r;
      if (live >> t & 1) {
        const f32x2 e = {ea[0][0][r], ea[1][0][r]};
        const f32x2 d = {x[0][0][r], x[1][0][r]};
        *reinterpret_cast<f32x2*>(pb + (unsigned)(t * a.C)) = e;
        *reinterpret_cast<f32x2*>(hb + (unsigned)(t * a.C)) = d;
      }
    }
    return;
  }
  // a lane's four rows, then the lanes before it in the tile
  float A[2][MT], h[2][MT], endA[2][MT], endH[2][MT];
#pragma unroll
  for (int j = 0; j < 2; ++j)
#pragma unroll
    for (int m = 0; m < MT; ++m) {
      A[j][m] = 1.f;
      h[j][m] = 0.f;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        h[j][m] = ea[j][m][r] * h[j][m] + x[j][m][r];
        A[j][m] *= ea[j][m][r];
      }
    }
#pragma unroll
  for (int off = 16; off <= 32; off <<= 1)
#pragma unroll
    for (int j = 0; j < 2; ++j)
#pragma unroll
      for (int m = 0; m < MT; ++m) {
        const float fa = __shfl_up(A[j][m], off, 64);
        const float fh = __shfl_up(h[j][m], off, 64);
        h[j][m] = lane >= off ? h[j][m] + A[j][m] * fh : h[j][m];
        A[j][m] = lane >= off ? A[j][m] * fa : A[j][m];
      }
#pragma unroll
  for (int j = 0; j < 2; ++j)
#pragma unroll
    for (int m = 0; m < MT; ++m) {
      endA[j][m] = __shfl(A[j][m], 48 + i16, 64);
      endH[j][m] = __shfl(h[j][m], 48 + i16, 64);
      const float pa = __shfl_up(A[j][m], 16, 64);
      const float ph = __shfl_up(h[j][m], 16, 64);
      A[j][m] = g == 0 ? 1.f : pa;
      h[j][m] = g == 0 ? 0.f : ph;
    }
  f32x2 A0 = {1.f, 1.f}, h0 = {0.f, 0.f};  // of the tiles before
#pragma unroll
  for (int m = 0; m < MT; ++m) {
    f32x2 s, l;
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      s[j] = A[j][m] * h0[j] + h[j][m];
      l[j] = A0[j] * A[j][m];
      h0[j] = endA[j][m] * h0[j] + endH[j][m];
      A0[j] *= endA[j][m];
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = m * 16 + g * 4 + r;
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        s[j] = ea[j][m][r] * s[j] + x[j][m][r];
        l[j] *= ea[j][m][r];
      }
      if (full || t < cnt) {
        *reinterpret_cast<f32x2*>(pb + (unsigned)(t * a.C)) = l;
        *reinterpret_cast<f32x2*>(hb + (unsigned)(t * a.C)) = s;
      }
    }
  }
}

// 32-bit mode: a thread per (row, channel)
__global__ void __launch_bounds__(256)
lru_gates32_kernel(const float* __restrict__ u, const float* __restrict__ w,
                   const LruGates a, float* __restrict__ prod,
                   float* __restrict__ hs) {
  const long id = (long)blockIdx.x * 256 + threadIdx.x;
  const long row = id / a.C;
  const int c = (int)(id % a.C);
  if (row >= a.M || a.ctx[row] <= 0) return;
  float la = 0.f, x = 0.f;
  if (c < a.blocks * a.bs) {
    const int blk = c / a.bs, n = c % a.bs;
    const float* ur = u + row * a.C + blk * a.bs;
    float zr = 0.f, zi = 0.f;
    for (int k = 0; k < a.bs; k += 4) {
      const f32x4 uv = *reinterpret_cast<const f32x4*>(ur + k);
      const f32x4 rv =
          *reinterpret_cast<const f32x4*>(w + gate_at(a, 0, blk, n, k));
      const f32x4 iv =
          *reinterpret_cast<const f32x4*>(w + gate_at(a, 1, blk, n, k));
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        zr += uv[e] * rv[e];
        zi += uv[e] * iv[e];
      }
    }
    la = a.decay[c] * sigmoid_exact(zr + a.br[c]);
    x = sqrtf(-expm1f(2.f * la)) * sigmoid_exact(zi + a.bi[c]) *
        u[row * a.C + c];
  }
  prod[id] = expf(la);
  hs[id] = x;
}

// segments of up to max_rows rows; a thread owns a channel
template <typename T>
__global__ void __launch_bounds__(256)
lru_scan_kernel(const T* __restrict__ ab, int ld,
                const float* __restrict__ a, const float* __restrict__ x,
                float* __restrict__ state, T* __restrict__ out, int C,
                const int* __restrict__ seg_row0,
                const int* __restrict__ seg_rows,
                const int* __restrict__ seg_slot,
                const int* __restrict__ ctx, int max_rows) {
  const int seg = blockIdx.y, c = blockIdx.x * 256 + threadIdx.x;
  const int n = seg_rows[seg];
  if (c >= C || n == 0 || n > max_rows) return;
  const long row0 = seg_row0[seg];
  float* st = state + (long)seg_slot[seg] * C + c;
  float s = ctx[row0] <= 1 ? 0.f : *st;
#pragma unroll 4
  for (int t = 0; t < n; ++t) {
    const long row = row0 + t;
    s = a[row * C + c] * s + x[row * C + c];
    from_f(out + row * C + c, s * gelu_of<T>(to_f(ab[row * ld + c])));
  }
  *st = s;
}

__global__ void __launch_bounds__(256)
lru_carry_kernel(const float* __restrict__ prod, const float* __restrict__ hs,
                 float* __restrict__ state, float* __restrict__ start, int C,
                 const int* __restrict__ longs,
                 const int* __restrict__ seg_row0,
                 const int* __restrict__ seg_rows,
                 const int* __restrict__ seg_slot,
                 const int* __restrict__ ctx) {
  const int c = blockIdx.x * 256 + threadIdx.x;
  if (c >= C) return;
  const int seg = longs[blockIdx.y * 2];
  const long chunk0 = longs[blockIdx.y * 2 + 1], row0 = seg_row0[seg];
  const int n = seg_rows[seg], nch = (n + LCH - 1) / LCH;
  float* st = state + (long)seg_slot[seg] * C + c;
  float s = ctx[row0] <= 1 ? 0.f : *st;
  constexpr int U = 8;
  for (int k0 = 0; k0 < nch; k0 += U) {
    float A[U], h[U];
#pragma unroll
    for (int k = 0; k < U; ++k) {  // loads first
      const long row = row0 + min((min(k0 + k, nch - 1) + 1) * LCH, n) - 1;
      A[k] = prod[row * C + c];
      h[k] = hs[row * C + c];
    }
#pragma unroll
    for (int k = 0; k < U; ++k)
      if (k0 + k < nch) {
        start[(chunk0 + k0 + k) * C + c] = s;
        s = A[k] * s + h[k];
      }
  }
  *st = s;
}

// a thread: eight channels of eight rows of a chunk
__global__ void __launch_bounds__(256)
lru_emit_kernel(const unsigned short* __restrict__ ab, int ld,
                const float* __restrict__ prod, const float* __restrict__ hs,
                const float* __restrict__ start,
                unsigned short* __restrict__ out, int C,
                const int* __restrict__ chunks, int nchunks,
                const int* __restrict__ seg_row0,
                const int* __restrict__ seg_rows) {
  const int vec = C / 8;
  const long id = (long)blockIdx.x * 256 + threadIdx.x;
  const int ch = (int)(id % vec) * 8;
  const long run = id / vec;
  const long chunk = run / (LCH / 8);
  if (chunk >= nchunks) return;
  const int seg = chunks[chunk * 2];
  const int t0 = chunks[chunk * 2 + 1] * LCH + (int)(run % (LCH / 8)) * 8;
  const int n = min(8, seg_rows[seg] - t0);
  float s[8];
  load8<float>(start + chunk * C + ch, s);
  for (int t = 0; t < n; ++t) {
    const long row = seg_row0[seg] + t0 + t;
    float A[8], h[8], y[8];
    load8<float>(prod + row * C + ch, A);
    load8<float>(hs + row * C + ch, h);
    load8<unsigned short>(ab + row * ld + ch, y);
#pragma unroll
    for (int i = 0; i < 8; ++i)
      h[i] = (h[i] + A[i] * s[i]) * fast_gelu(y[i]);
    store8(out + row * C + ch, h);
  }
}

// ab [M, y | x] of C columns each; u [M, C], prod and hs [M, C] fp32, start
// [nchunks, C] fp32: scratch. nlong 0: no long segments.
extern "C" void launch_gated_lru(
    const void* ab, int ld, int M, int C, const float* conv_w,
    const float* conv_b, int taps, const void* gates, const float* gates_b,
    int blocks, int bs, const float* decay, float* state, void* conv, void* u,
    float* prod, float* hs, float* start, void* out, const int* seg_row0,
    const int* seg_rows, const int* seg_slot, int nseg, int longest,
    const int* row_seq, const int* ctx, const int* longs, int nlong,
    const int* chunks, int nchunks, int max_rows, bool fp32,
    hipStream_t stream) {
  const bool shift = longest <= 1;
  const int rb = M >= 8192 ? 8 : M >= 2048 ? 4 : 1;
  const long conv_wgs = ((long)(M + rb - 1) / rb * (C / 8) + 255) / 256;
#define LC(T, TAPS)                                                         \
  do {                                                                      \
    const ConvArgs<T> a{(const T*)ab + C, ld, M, C, taps, rb, conv_w,       \
                        (T*)conv, seg_row0, seg_slot, row_seq, ctx, shift}; \
    hipLaunchKernelGGL((lru_conv_kernel<T, TAPS>), dim3(conv_wgs),          \
                       dim3(256), 0, stream, a, conv_b, (T*)u);             \
    if (!shift && taps > 1)                                                 \
      hipLaunchKernelGGL((conv_state_kernel<T>),                            \
                         dim3((C + 255) / 256, nseg), dim3(256), 0, stream, \
                         (const T*)ab + C, ld, C, taps, (T*)conv, seg_row0, \
                         seg_rows, seg_slot, ctx);                          \
  } while (0)
  if (fp32 && taps == 4) LC(float, 4);
  else if (fp32) LC(float, 0);
  else if (taps == 4) LC(unsigned short, 4);
  else LC(unsigned short, 0);
#undef LC
  const LruGates a{gates_b, gates_b + C, decay,  seg_row0, seg_rows, row_seq,
                   ctx,     M,           C,      blocks,   bs,       max_rows};
  const dim3 scan_grid((C + 255) / 256, nseg);
  if (fp32) {
    hipLaunchKernelGGL(lru_gates32_kernel, dim3(((long)M * C + 255) / 256),
                       dim3(256), 0, stream, (const float*)u,
                       (const float*)gates, a, prod, hs);
    hipLaunchKernelGGL(lru_scan_kernel<float>, scan_grid, dim3(256), 0,
                       stream, (const float*)ab, ld, prod, hs, state,
                       (float*)out, C, seg_row0, seg_rows, seg_slot, ctx,
                       INT_MAX);
    return;
  }
  typedef unsigned short bf;
  const int groups = (C + 127) / 128;
  const bool shared = bs % 128 == 0 && blocks * bs == C;
#define LG(MT, L, S, N)                                                      \
  hipLaunchKernelGGL((lru_gates_kernel<MT, L, S>), dim3((long)(N) * groups), \
                     dim3(256), 0, stream, (const bf*)u, (const bf*)gates,   \
                     a, chunks, groups, prod, hs)
  if (nlong < nseg) LG(1, false, false, (M + 15) / 16);
  if (nlong < nseg)
    hipLaunchKernelGGL(lru_scan_kernel<bf>, scan_grid, dim3(256), 0, stream,
                       (const bf*)ab, ld, prod, hs, state, (bf*)out, C,
                       seg_row0, seg_rows, seg_slot, ctx, max_rows);
  if (nlong == 0) return;
  if (shared) LG(LCH / 16, true, true, nchunks);
  else LG(LCH / 16, true, false, nchunks);
#undef LG
  hipLaunchKernelGGL(lru_carry_kernel, dim3((C + 255) / 256, nlong),
                     dim3(256), 0, stream, prod, hs, state, start, C, longs,
                     seg_row0, seg_rows, seg_slot, ctx);
  hipLaunchKernelGGL(lru_emit_kernel,
                     dim3(((long)nchunks * (LCH / 8) * (C / 8) + 255) / 256),
                     dim3(256), 0, stream, (const bf*)ab, ld, prod, hs, start,
                     (bf*)out, C, chunks, nchunks, seg_row0, seg_rows);
}
