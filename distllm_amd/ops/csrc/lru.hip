// Real-gated linear recurrent unit of a ragged step, per channel:
//   r = sigmoid(Wr u + br), i = sigmoid(Wi u + bi)   (block-diagonal W)
//   log a = decay * r;  S <- a S + sqrt(1 - a^2) i u;  out = S * gelu(y)
// u is the causal convolution of the projection's second half, y its first.
//
//   lru_conv_kernel   u
//   lru_gates_kernel  both gate products on the MFMA and everything up to
//                     the recurrence; rows of short segments: log a and the
//                     drive; chunks of long ones: their recurrence from
//                     zeros and the summed log a, so that a state S before
//                     the chunk adds exp(sum) S
//   lru_scan_kernel   short segments, row by row
//   lru_carry_kernel  long segments: state before every chunk
//   lru_emit_kernel   long segments: output
// Everything behind u and y is fp32. The 32-bit mode takes every segment row
// by row, with its gates from lru_gates32_kernel.
#include "short_conv.h"

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;

#define LCH 64  // rows of a chunk

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

// sqrt(1 - exp(2 la)) for la <= 0, also where la is tiny
__device__ __forceinline__ float drive_factor(float la) {
  const float z = 2.f * la;
  const float near =
      -z * (1.f +
            z * 0.5f *
                (1.f + z * 0.33333333f * (1.f + z * 0.25f * (1.f + z * 0.2f))));
  return __builtin_amdgcn_sqrtf(z > -0.1f ? near : 1.f - fast_exp(z));
}

struct LruGates {
  const float *br, *bi, *decay;
  const int *seg_row0, *seg_rows, *row_seq, *ctx;
  int M, C, blocks, bs, max_rows;
};

// A wave: MT * 16 rows and 32 channels of both gates; a workgroup: four
// neighbouring groups of 32 channels. LONG: the rows are a chunk; else they
// are 16 consecutive rows, of which those of short segments count.
template <int MT, bool LONG>
__global__ void __launch_bounds__(256)
lru_gates_kernel(const unsigned short* __restrict__ u,
                 const unsigned short* __restrict__ w, const LruGates a,
                 const int* __restrict__ chunks, int groups,
                 float* __restrict__ sum, float* __restrict__ hs) {
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int i16 = lane & 15, g = lane >> 4;
  const int tile = blockIdx.x / groups;
  const int c0 = (blockIdx.x % groups * 4 + wid) * 32;
  if (c0 >= a.C) return;
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
    if (live == 0) return;
  }

  f32x4 acc[2][2][MT];  // gate, group of 16 channels, row tile
#pragma unroll
  for (int z = 0; z < 2; ++z)
#pragma unroll
    for (int j = 0; j < 2; ++j)
#pragma unroll
      for (int m = 0; m < MT; ++m) acc[z][j][m] = (f32x4)0.f;
  const bool real = c0 < a.blocks * a.bs;  // else a column of padding
  if (real) {
    const int blk = c0 / a.bs, n0 = c0 % a.bs;
    const unsigned short* ur[MT];
#pragma unroll
    for (int m = 0; m < MT; ++m)
      ur[m] = u + (row0 + min(m * 16 + i16, cnt - 1)) * a.C + blk * a.bs +
              g * 8;
    const unsigned short* wr[2][2];
#pragma unroll
    for (int z = 0; z < 2; ++z)
#pragma unroll
      for (int j = 0; j < 2; ++j)
        wr[z][j] = w +
                   (((long)z * a.blocks + blk) * a.bs + n0 + j * 16 + i16) *
                       a.bs +
                   g * 8;
#pragma unroll 2
    for (int k = 0; k < a.bs; k += 32) {
      bf16x8 uf[MT], wf[2][2];
#pragma unroll
      for (int m = 0; m < MT; ++m)
        uf[m] = *reinterpret_cast<const bf16x8*>(ur[m] + k);
#pragma unroll
      for (int z = 0; z < 2; ++z)
#pragma unroll
        for (int j = 0; j < 2; ++j)
          wf[z][j] = *reinterpret_cast<const bf16x8*>(wr[z][j] + k);
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

#pragma unroll
  for (int j = 0; j < 2; ++j) {
    const int c = c0 + j * 16 + i16;
    const float br = a.br[c], bi = a.bi[c], decay = a.decay[c];
    float la0 = 0.f, h0 = 0.f;  // sum and state before the row tile
#pragma unroll
    for (int m = 0; m < MT; ++m) {
      // a lane holds rows g * 4 + r of the tile
      float la[4], x[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = m * 16 + g * 4 + r;
        la[r] = x[r] = 0.f;
        if (t < cnt && real) {
          const float uv = bf2f(u[(row0 + t) * a.C + c]);
          la[r] = decay * fast_rcp(1.f + fast_exp(-acc[0][j][m][r] - br));
          x[r] = drive_factor(la[r]) *
                 fast_rcp(1.f + fast_exp(-acc[1][j][m][r] - bi)) * uv;
        }
      }
      if (!LONG) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int t = g * 4 + r;
          if (live >> t & 1) {
            sum[(row0 + t) * a.C + c] = la[r];
            hs[(row0 + t) * a.C + c] = x[r];
          }
        }
        continue;
      }
      float ea[4], A = 0.f, h = 0.f;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        ea[r] = fast_exp(la[r]);
        A += la[r];
        h = ea[r] * h + x[r];
      }
      // lanes g before this one, then the tiles before
#pragma unroll
      for (int off = 16; off <= 32; off <<= 1) {
        const float pa = __shfl_up(A, off, 64), ph = __shfl_up(h, off, 64);
        if (lane >= off) {
          h += fast_exp(A) * ph;
          A += pa;
        }
      }
      const float endA = __shfl(A, 48 + i16, 64);
      const float endH = __shfl(h, 48 + i16, 64);
      float pa = __shfl_up(A, 16, 64), ph = __shfl_up(h, 16, 64);
      if (g == 0) pa = ph = 0.f;
      float s = fast_exp(pa) * h0 + ph, l = la0 + pa;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = m * 16 + g * 4 + r;
        s = ea[r] * s + x[r];
        l += la[r];
        if (t < cnt) {
          sum[(row0 + t) * a.C + c] = l;
          hs[(row0 + t) * a.C + c] = s;
        }
      }
      h0 = fast_exp(endA) * h0 + endH;
      la0 += endA;
    }
  }
}

// 32-bit mode: a thread per (row, channel)
__global__ void __launch_bounds__(256)
lru_gates32_kernel(const float* __restrict__ u, const float* __restrict__ w,
                   const LruGates a, float* __restrict__ sum,
                   float* __restrict__ hs) {
  const long id = (long)blockIdx.x * 256 + threadIdx.x;
  const long row = id / a.C;
  const int c = (int)(id % a.C);
  if (row >= a.M || a.ctx[row] <= 0) return;
  float la = 0.f, x = 0.f;
  if (c < a.blocks * a.bs) {
    const int blk = c / a.bs, n = c % a.bs;
    const float* ur = u + row * a.C + blk * a.bs;
    const float* wr = w + ((long)blk * a.bs + n) * a.bs;
    const float* wi = wr + (long)a.blocks * a.bs * a.bs;
    float zr = 0.f, zi = 0.f;
    for (int k = 0; k < a.bs; k += 4) {
      const f32x4 uv = *reinterpret_cast<const f32x4*>(ur + k);
      const f32x4 rv = *reinterpret_cast<const f32x4*>(wr + k);
      const f32x4 iv = *reinterpret_cast<const f32x4*>(wi + k);
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
  sum[id] = la;
  hs[id] = x;
}

// segments of up to max_rows rows; a thread owns a channel
template <typename T>
__global__ void __launch_bounds__(256)
lru_scan_kernel(const T* __restrict__ ab, int ld,
                const float* __restrict__ la, const float* __restrict__ x,
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
    s = expf(la[row * C + c]) * s + x[row * C + c];
    from_f(out + row * C + c, s * gelu_of<T>(to_f(ab[row * ld + c])));
  }
  *st = s;
}

__global__ void __launch_bounds__(256)
lru_carry_kernel(const float* __restrict__ sum, const float* __restrict__ hs,
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
      A[k] = sum[row * C + c];
      h[k] = hs[row * C + c];
    }
#pragma unroll
    for (int k = 0; k < U; ++k)
      if (k0 + k < nch) {
        start[(chunk0 + k0 + k) * C + c] = s;
        s = fast_exp(A[k]) * s + h[k];
      }
  }
  *st = s;
}

// a thread: eight channels of eight rows of a chunk
__global__ void __launch_bounds__(256)
lru_emit_kernel(const unsigned short* __restrict__ ab, int ld,
                const float* __restrict__ sum, const float* __restrict__ hs,
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
    load8<float>(sum + row * C + ch, A);
    load8<float>(hs + row * C + ch, h);
    load8<unsigned short>(ab + row * ld + ch, y);
#pragma unroll
    for (int i = 0; i < 8; ++i)
      h[i] = (h[i] + fast_exp(A[i]) * s[i]) * fast_gelu(y[i]);
    store8(out + row * C + ch, h);
  }
}

// ab [M, y | x] of C columns each; u [M, C], sum and hs [M, C] fp32, start
// [nchunks, C] fp32: scratch. nlong 0: no long segments.
extern "C" void launch_gated_lru(
    const void* ab, int ld, int M, int C, const float* conv_w,
    const float* conv_b, int taps, const void* gates, const float* gates_b,
    int blocks, int bs, const float* decay, float* state, void* conv, void* u,
    float* sum, float* hs, float* start, void* out, const int* seg_row0,
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
                       (const float*)gates, a, sum, hs);
    hipLaunchKernelGGL(lru_scan_kernel<float>, scan_grid, dim3(256), 0,
                       stream, (const float*)ab, ld, sum, hs, state,
                       (float*)out, C, seg_row0, seg_rows, seg_slot, ctx,
                       INT_MAX);
    return;
  }
  typedef unsigned short bf;
  const int groups = (C + 127) / 128;
  hipLaunchKernelGGL((lru_gates_kernel<1, false>),
                     dim3((long)(M + 15) / 16 * groups), dim3(256), 0, stream,
                     (const bf*)u, (const bf*)gates, a, chunks, groups, sum,
                     hs);
  hipLaunchKernelGGL(lru_scan_kernel<bf>, scan_grid, dim3(256), 0, stream,
                     (const bf*)ab, ld, sum, hs, state, (bf*)out, C, seg_row0,
                     seg_rows, seg_slot, ctx, max_rows);
  if (nlong == 0) return;
  hipLaunchKernelGGL((lru_gates_kernel<LCH / 16, true>),
                     dim3((long)nchunks * groups), dim3(256), 0, stream,
                     (const bf*)u, (const bf*)gates, a, chunks, groups, sum,
                     hs);
  hipLaunchKernelGGL(lru_carry_kernel, dim3((C + 255) / 256, nlong),
                     dim3(256), 0, stream, sum, hs, state, start, C, longs,
                     seg_row0, seg_rows, seg_slot, ctx);
  hipLaunchKernelGGL(lru_emit_kernel,
                     dim3(((long)nchunks * (LCH / 8) * (C / 8) + 255) / 256),
                     dim3(256), 0, stream, (const bf*)ab, ld, sum, hs, start,
                     (bf*)out, C, chunks, nchunks, seg_row0, seg_rows);
}
