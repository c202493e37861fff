// Attention over a paged cache of low-rank latents.
//
// A token's cache entry is one latent vector c of R numbers (rank n padded
// with zeros to R); keys and values of every head are linear in it,
// k_h = Uk_h c and v_h = Uv_h c. Folding Uk into the query (q'_h = Uk_h^T
// q_h) and Uv into the output leaves one shared "head" whose key and value
// are both c:
//     s_hj = scale * q'_h . c_j      o'_h = sum_j softmax(s)_hj c_j
// so a decode step reads R numbers per cached token for all heads. A cache
// row may go on behind the latent, with a key part that all heads share (and
// that queries have a part of their own for); RT is the length of a row.
//
// Cache layout: [num_blocks, PBLK, RT], block_table [S, max_blocks] int32.
// Every row of a batch is one token: row_seq[row] is its block-table row,
// ctx[row] its position + 1 (0: padding row, nothing is read or written).
// A row sees the last `window` positions up to its own.
#include "common.h"

#define PBLK 16  // tokens per cache block
#define LOG2E 1.4426950408889634f

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;

extern __shared__ __attribute__((aligned(16))) char smem[];

// ---- norm of the two down-projections + cache write ----------------------
// ab [M, QP (+ R)]: wave 0 of a workgroup norms the query latent (first QP
// columns, true size qn), wave 1 the cached latent (next R columns, true
// size rn) and writes it to its cache slot. cache == nullptr: the layer
// reads another layer's cache and has no latent of its own.
// Rows of up to 8192 columns stay in registers between the two passes.
template <typename T, int NC>
__global__ void __launch_bounds__(128)
latent_prep_kernel(const T* __restrict__ ab, int ld, int QP, int qn, int R,
                   int rn, const float* __restrict__ wq,
                   const float* __restrict__ wc, float eps,
                   T* __restrict__ cq, T* __restrict__ cache,
                   const int* __restrict__ block_table, int max_blocks,
                   int num_blocks, const int* __restrict__ row_seq,
                   const int* __restrict__ ctx) {
  const int row = blockIdx.x;
  const int lane = threadIdx.x & 63;
  const bool latent = threadIdx.x >= 64;
  const int n = latent ? rn : qn;
  const int np = latent ? R : QP;
  const T* src = ab + (long)row * ld + (latent ? QP : 0);
  const float* w = latent ? wc : wq;
  T* dst = cq + (long)row * QP;
  if (latent) {
    const int pos = ctx[row] - 1;
    if (pos < 0 || pos / PBLK >= max_blocks) return;
    const int blk = block_table[(long)row_seq[row] * max_blocks + pos / PBLK];
    if (blk < 0 || blk >= num_blocks) return;
    dst = cache + ((long)blk * PBLK + pos % PBLK) * R;
  }
  float v[NC][8];
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < NC; ++k) {
    const int c = (k * 64 + lane) * 8;
    if (c < np) {
      load8<T>(src + c, v[k]);
#pragma unroll
      for (int i = 0; i < 8; ++i) ss += v[k][i] * v[k][i];
    }
  }
  float wv[NC][8];  // in flight while the sum is reduced
#pragma unroll
  for (int k = 0; k < NC; ++k) {
    const int c = (k * 64 + lane) * 8;
    if (c < np) load8<float>(w + c, wv[k]);
  }
  ss = wave_reduce_sum(ss);
  const float inv = 1.f / sqrtf(ss / n + eps);
#pragma unroll
  for (int k = 0; k < NC; ++k) {
    const int c = (k * 64 + lane) * 8;
    if (c < np) {
#pragma unroll
      for (int i = 0; i < 8; ++i) v[k][i] *= inv * wv[k][i];
      store8(dst + c, v[k]);
    }
  }
}

extern "C" void launch_latent_prep(
    const void* ab, int M, int ld, int QP, int qn, int R, int rn,
    const float* wq, const float* wc, float eps, void* cq, void* cache,
    const int* block_table, int max_blocks, int num_blocks,
    const int* row_seq, const int* ctx, bool fp32, hipStream_t stream) {
  const dim3 grid(M), block(cache != nullptr ? 128 : 64);
  const int nc = ((QP > R ? QP : R) + 511) / 512;
#define LP(T, NC)                                                           \
  hipLaunchKernelGGL((latent_prep_kernel<T, NC>), grid, block, 0, stream,   \
                     (const T*)ab, ld, QP, qn, R, rn, wq, wc, eps, (T*)cq,  \
                     (T*)cache, block_table, max_blocks, num_blocks,        \
                     row_seq, ctx)
#define LP_N(T)                \
  do {                         \
    if (nc == 1) LP(T, 1);     \
    else if (nc == 2) LP(T, 2); \
    else if (nc <= 4) LP(T, 4); \
    else if (nc <= 8) LP(T, 8); \
    else LP(T, 16);            \
  } while (0)
  if (fp32) LP_N(float);
  else LP_N(unsigned short);
#undef LP_N
#undef LP
}

// ---- norm of the latent, rotation of queries and key part, cache write -------
// ab row: H heads of dp unrotated and tp rotated numbers, the latent (R, true
// size rn), the key part (tp). The first 2 * half of tp numbers rotate, those
// behind are zeros. Rotated query parts go to the end of ql's rows (first n
// rows; ql_row numbers per head) or back to ab; three waves of a workgroup do
// that, the fourth makes the cache row.

// pairs i0 .. i0 + 7 of src (number i and i + half) to dst
template <typename T>
__device__ __forceinline__ void rotate_pairs(const T* src, T* dst, int i0,
                                             int half, const float* table) {
  if ((half & 7) == 0) {
    float a[8], b[8], t[16], x[8], y[8];
    load8<T>(src + i0, a);
    load8<T>(src + half + i0, b);
    load8<float>(table + i0 * 2, t);
    load8<float>(table + i0 * 2 + 8, t + 8);
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      x[i] = a[i] * t[2 * i] - b[i] * t[2 * i + 1];
      y[i] = b[i] * t[2 * i] + a[i] * t[2 * i + 1];
    }
    store8(dst + i0, x);
    store8(dst + half + i0, y);
    return;
  }
  for (int i = i0; i < min(i0 + 8, half); ++i) {
    const float a = to_f(src[i]), b = to_f(src[half + i]);
    const float c = table[i * 2], s = table[i * 2 + 1];
    from_f(dst + i, a * c - b * s);
    from_f(dst + half + i, b * c + a * s);
  }
}

template <typename T, int NC>
__global__ void __launch_bounds__(256)
rotary_latent_prep_kernel(T* __restrict__ ab, int ld, int H, int dp, int tp,
                          int R, int rn, const float* __restrict__ wc,
                          float eps, const float* __restrict__ table,
                          int half, T* __restrict__ ql, int n, int ql_row,
                          T* __restrict__ cache,
                          const int* __restrict__ block_table,
                          int max_blocks, int num_blocks,
                          const int* __restrict__ row_seq,
                          const int* __restrict__ ctx) {
  const int row = blockIdx.x;
  T* src = ab + (long)row * ld;
  const float* cs = table + (long)row * half * 2;
  const int groups = (half + 7) / 8;
  if (threadIdx.x < 192) {
    for (int u = threadIdx.x; u < H * groups; u += 192) {
      const int head = u / groups, i0 = u % groups * 8;
      T* q = src + head * (dp + tp) + dp;
      T* dst = q;
      if (row < n) {
        dst = ql + ((long)row * H + head) * ql_row + ql_row - tp;
        if (i0 == 0)
          for (int c = 2 * half; c < tp; ++c) from_f(dst + c, 0.f);
      }
      rotate_pairs(q, dst, i0, half, cs);
    }
    return;
  }
  if (cache == nullptr) return;
  const int lane = threadIdx.x & 63;
  const int pos = ctx[row] - 1;
  if (pos < 0 || pos / PBLK >= max_blocks) return;
  const int blk = block_table[(long)row_seq[row] * max_blocks + pos / PBLK];
  if (blk < 0 || blk >= num_blocks) return;
  T* dst = cache + ((long)blk * PBLK + pos % PBLK) * (R + tp);
  src += H * (dp + tp);
  for (int g = lane; g < groups; g += 64)
    rotate_pairs(src + R, dst + R, g * 8, half, cs);
  float v[NC][8];
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < NC; ++k) {
    const int c = (k * 64 + lane) * 8;
    if (c < R) {
      load8<T>(src + c, v[k]);
#pragma unroll
      for (int i = 0; i < 8; ++i) ss += v[k][i] * v[k][i];
    }
  }
  const float inv = 1.f / sqrtf(wave_reduce_sum(ss) / rn + eps);
#pragma unroll
  for (int k = 0; k < NC; ++k) {
    const int c = (k * 64 + lane) * 8;
    if (c < R) {
      float w[8];
      load8<float>(wc + c, w);
#pragma unroll
      for (int i = 0; i < 8; ++i) v[k][i] *= inv * w[i];
      store8(dst + c, v[k]);
    }
  }
}

extern "C" void launch_rotary_latent_prep(
    void* ab, int M, int ld, int H, int dp, int tp, int R, int rn,
    const float* wc, float eps, const float* table, int half, void* ql, int n,
    int ql_row, void* cache, const int* block_table, int max_blocks,
    int num_blocks, const int* row_seq, const int* ctx, bool fp32,
    hipStream_t stream) {
  const dim3 grid(M), block(cache != nullptr ? 256 : 192);
#define RP(T, NC)                                                           \
  hipLaunchKernelGGL((rotary_latent_prep_kernel<T, NC>), grid, block, 0,    \
                     stream, (T*)ab, ld, H, dp, tp, R, rn, wc, eps, table,  \
                     half, (T*)ql, n, ql_row, (T*)cache, block_table,       \
                     max_blocks, num_blocks, row_seq, ctx)
#define RP_N(T)                   \
  do {                            \
    if (R <= 512) RP(T, 1);       \
    else if (R <= 1024) RP(T, 2); \
    else RP(T, 8);                \
  } while (0)
  if (fp32) RP_N(float);
  else RP_N(unsigned short);
#undef RP_N
#undef RP
}

// ---- latents of chosen positions, packed ----------------------------------
// Row i of out is the first vec0 pieces of the cache entry of position
// key_pos[i] of block-table row key_seq[i], row i of rest the others.
__global__ void __launch_bounds__(256)
latent_gather_kernel(const i32x4* __restrict__ cache,
                     const int* __restrict__ block_table, int max_blocks,
                     int num_blocks, const int* __restrict__ key_seq,
                     const int* __restrict__ key_pos, i32x4* __restrict__ out,
                     i32x4* __restrict__ rest, int T, int vec, int vec0) {
  const long total = (long)T * vec;
  const long stride = (long)gridDim.x * blockDim.x;
  for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x; i < total;
       i += stride) {
    const int row = (int)(i / vec), c = (int)(i % vec);
    const int pos = key_pos[row];
    i32x4 v = {0, 0, 0, 0};
    if (pos >= 0 && pos / PBLK < max_blocks) {
      const int blk =
          block_table[(long)key_seq[row] * max_blocks + pos / PBLK];
      if (blk >= 0 && blk < num_blocks)
        v = cache[((long)blk * PBLK + pos % PBLK) * vec + c];
    }
    if (c < vec0) out[(long)row * vec0 + c] = v;
    else rest[(long)row * (vec - vec0) + c - vec0] = v;
  }
}

extern "C" void launch_latent_gather(const void* cache,
                                     const int* block_table, int max_blocks,
                                     int num_blocks, const int* key_seq,
                                     const int* key_pos, void* out,
                                     void* rest, int T, int row_bytes,
                                     int out_bytes, hipStream_t stream) {
  const int vec = row_bytes / 16;
  const int blocks = (int)min(((long)T * vec + 255) / 256, (long)4096);
  hipLaunchKernelGGL(latent_gather_kernel, dim3(blocks), dim3(256), 0, stream,
                     (const i32x4*)cache, block_table, max_blocks, num_blocks,
                     key_seq, key_pos, (i32x4*)out, (i32x4*)rest, T, vec,
                     out_bytes / 16);
}

// ---- per-head products -----------------------------------------------------
// out[m, h, :] = W[h] x[m, h, :], W [H, N, K] bf16, for the few rows of a
// decode step (weight-streaming bound); rows and heads of x and out are
// strided. A wave owns 16 output columns; the
// weight fragment is read once and used for MT tiles of 16 rows.
template <int MT, int KU>
__global__ void __launch_bounds__(256)
head_gemm_kernel(const unsigned short* __restrict__ x,
                 const unsigned short* __restrict__ W,
                 unsigned short* __restrict__ out, int M, int H, int N,
                 int K, long xrow_s, int xhead_s, long orow_s,
                 int ohead_s) {
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int nb = N / 64;
  const int head = blockIdx.x / nb;
  const int n0 = (blockIdx.x % nb) * 64 + wid * 16;
  const int m0 = blockIdx.y * (16 * MT);
  const int i16 = lane & 15, g = lane >> 4;
  const unsigned short* wrow =
      W + ((long)head * N + n0 + i16) * K + g * 8;
  const unsigned short* xrow[MT];
#pragma unroll
  for (int t = 0; t < MT; ++t) {
    const int m = min(m0 + t * 16 + i16, M - 1);
    xrow[t] = x + m * xrow_s + (long)head * xhead_s + g * 8;
  }
  f32x4 acc[MT];
#pragma unroll
  for (int t = 0; t < MT; ++t) acc[t] = {0.f, 0.f, 0.f, 0.f};
  // KU steps of loads are in flight together
  for (int k0 = 0; k0 < K; k0 += 32 * KU) {
    bf16x8 wf[KU], xf[KU][MT];
#pragma unroll
    for (int s = 0; s < KU; ++s) {
      wf[s] = *reinterpret_cast<const bf16x8*>(wrow + k0 + s * 32);
#pragma unroll
      for (int t = 0; t < MT; ++t)
        xf[s][t] = *reinterpret_cast<const bf16x8*>(xrow[t] + k0 + s * 32);
    }
#pragma unroll
    for (int s = 0; s < KU; ++s)
#pragma unroll
      for (int t = 0; t < MT; ++t)
        acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[s], xf[s][t],
                                                         acc[t], 0, 0, 0);
  }
#pragma unroll
  for (int t = 0; t < MT; ++t) {
    const int m = m0 + t * 16 + i16;
    if (m < M) {
      s16x4 o;
#pragma unroll
      for (int r = 0; r < 4; ++r) o[r] = (short)f2bf(acc[t][r]);
      *reinterpret_cast<s16x4*>(out + m * orow_s + (long)head * ohead_s +
                                n0 + g * 4) = o;
    }
  }
}

extern "C" void launch_head_gemm(const void* x, const void* W, void* out,
                                 int M, int H, int N, int K, long xrow_s,
                                 int xhead_s, long orow_s, int ohead_s,
                                 hipStream_t stream) {
  // row tiles per workgroup: as many as leave two workgroups per CU
  const int tiles = (M + 15) / 16;
  const long cols = (long)H * (N / 64);
  int mt = 1;
  while (mt < 4 && mt < tiles && cols * ((tiles + 2 * mt - 1) / (2 * mt)) >= 512)
    mt *= 2;
#define HG(MT, KU)                                                        \
  hipLaunchKernelGGL((head_gemm_kernel<MT, KU>),                          \
                     dim3(cols, (M + 16 * MT - 1) / (16 * MT)),           \
                     dim3(256), 0, stream, (const unsigned short*)x,      \
                     (const unsigned short*)W, (unsigned short*)out, M, H, \
                     N, K, xrow_s, xhead_s, orow_s, ohead_s)
#define HG_K(MT)                     \
  do {                               \
    if (K % 256 == 0) HG(MT, 8);     \
    else if (K % 128 == 0) HG(MT, 4); \
    else HG(MT, 2);                  \
  } while (0)
  if (mt == 1) HG_K(1);
  else if (mt == 2) HG_K(2);
  else HG_K(4);
#undef HG_K
#undef HG
}

// ---- attention, one workgroup per (row, head), any rank and type ----------
// NV: latent columns per thread (R <= 256 * NV). sink, gate: null or the
// numbers of the heads (gate rows are ld_gate apart).
template <typename T, int NV>
__global__ void __launch_bounds__(256)
latent_attn_rows_kernel(const T* __restrict__ q, const T* __restrict__ cache,
                        const int* __restrict__ block_table,
                        const int* __restrict__ row_seq,
                        const int* __restrict__ ctx, T* __restrict__ out,
                        int H, int R, int RT, int max_blocks, int window,
                        float scale, const float* __restrict__ sink,
                        const T* __restrict__ gate, int ld_gate) {
  constexpr int V = 16 / sizeof(T);
  typedef __attribute__((ext_vector_type(V))) T vec;
  float* q_lds = reinterpret_cast<float*>(smem);  // RT
  float* p_lds = q_lds + RT;                      // 256
  int* off_lds = reinterpret_cast<int*>(p_lds + 256);  // 256 cache rows
  float* red = reinterpret_cast<float*>(off_lds + 256);  // 8
  const int row = blockIdx.x / H, head = blockIdx.x % H;
  const int tid = threadIdx.x, wid = tid >> 6, lane = tid & 63;
  const int L = min(ctx[row], max_blocks * PBLK);
  const int lo = L > window ? L - window : 0;
  const int* bt = block_table + (long)row_seq[row] * max_blocks;
  const T* qr = q + ((long)row * H + head) * RT;
  for (int c = tid; c < RT; c += 256) q_lds[c] = to_f(qr[c]) * scale;

  float m = -INFINITY, l = 0.f, acc[NV];
#pragma unroll
  for (int i = 0; i < NV; ++i) acc[i] = 0.f;
  for (int t0 = lo; t0 < L; t0 += 256) {
    const int key = t0 + tid;
    const bool live = key < L;
    __syncthreads();  // q is staged; the previous tile is consumed
    float s = -INFINITY;
    if (live) {
      const int off = bt[key / PBLK] * PBLK + key % PBLK;
      off_lds[tid] = off;
      const T* c = cache + (long)off * RT;
      float dot = 0.f;
      for (int k = 0; k < RT; k += V) {
        const vec cv = *reinterpret_cast<const vec*>(c + k);
#pragma unroll
        for (int i = 0; i < V; ++i) dot += to_f((T)cv[i]) * q_lds[k + i];
      }
      s = dot;
    }
    const float wmax = wave_reduce_max(s);
    if (lane == 0) red[wid] = wmax;
    __syncthreads();
    const float mn =
        fmaxf(m, fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])));
    const float p = live ? expf(s - mn) : 0.f;
    p_lds[tid] = p;
    const float wsum = wave_reduce_sum(p);
    if (lane == 0) red[4 + wid] = wsum;
    __syncthreads();
    const float alpha = expf(m - mn);  // 0 on the first tile
    l = l * alpha + (red[4] + red[5]) + (red[6] + red[7]);
    m = mn;
    const int nk = min(256, L - t0);
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = tid + i * 256;
      if (c < R) {
        float a = acc[i] * alpha;
        for (int j = 0; j < nk; ++j)
          a += p_lds[j] * to_f(cache[(long)off_lds[j] * RT + c]);
        acc[i] = a;
      }
    }
  }
  float inv = l > 0.f ? 1.f / l : 0.f;
  if (sink != nullptr && l > 0.f) {
    const float top = fmaxf(m, sink[head]), a = expf(m - top);
    inv = a / (l * a + expf(sink[head] - top));
  }
  if (gate != nullptr)
    inv *= sigmoid_exact(to_f(gate[(long)row * ld_gate + head]));
  T* o = out + ((long)row * H + head) * R;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = tid + i * 256;
    if (c < R) from_f(o + c, acc[i] * inv);
  }
}

extern "C" void launch_latent_attn_rows(
    const void* q, const void* cache, const int* block_table,
    const int* row_seq, const int* ctx, void* out, int M, int H, int R,
    int RT, int max_blocks, int window, float scale, const float* sink,
    const void* gate, int ld_gate, bool fp32, hipStream_t stream) {
  const int lds = (RT + 256 + 256 + 8) * 4;
#define LA(T, NV)                                                            \
  hipLaunchKernelGGL((latent_attn_rows_kernel<T, NV>), dim3(M * H),          \
                     dim3(256), lds, stream, (const T*)q, (const T*)cache,   \
                     block_table, row_seq, ctx, (T*)out, H, R, RT,           \
                     max_blocks, window, scale, sink, (const T*)gate, ld_gate)
#define LA_N(T)                    \
  do {                             \
    if (R <= 256) LA(T, 1);        \
    else if (R <= 512) LA(T, 2);   \
    else if (R <= 1024) LA(T, 4);  \
    else LA(T, 16);                \
  } while (0)
  if (fp32) LA_N(float);
  else LA_N(unsigned short);
#undef LA_N
#undef LA
}
