// Attention of single-token rows (see chunk_attention.h): a generic kernel
// for any size and type, and the MFMA kernel of bf16 decode steps.
#pragma once
#include "chunk_attention.h"

extern __shared__ __attribute__((aligned(16))) char smem[];

// ---- one workgroup per (row, head), any size and type ---------------------
// NV: value columns per thread (DV <= 256 * NV). Library functions
// throughout: this is also the kernel of the 32-bit mode.
template <typename T, int NV, typename P>
__global__ void __launch_bounds__(256)
attention_rows_kernel(const T* __restrict__ q, const T* __restrict__ kpages,
                  const T* __restrict__ vpages, const P policy,
                  const int* __restrict__ block_table,
                  const int* __restrict__ row_seq,
                  const int* __restrict__ ctx, T* __restrict__ out,
                  long ld_out, int H, int G, int DK, int DV, int max_blocks,
                  int chunk) {
  constexpr int V = 16 / sizeof(T);
  typedef __attribute__((ext_vector_type(V))) T vec;
  float* q_lds = reinterpret_cast<float*>(smem);         // DK
  float* p_lds = q_lds + DK;                             // 256
  int* page_lds = reinterpret_cast<int*>(p_lds + 256);   // 256
  float* red = reinterpret_cast<float*>(page_lds + 256);  // 8
  const int row = blockIdx.x / H, head = blockIdx.x % H;
  const int g = head / (H / G);
  const int tid = threadIdx.x, wid = tid >> 6, lane = tid & 63;
  const int L = min(ctx[row], max_blocks * PBLK);
  const int lo = L > 0 ? (L - 1) / chunk * chunk : 0;
  const int* bt = block_table + (long)row_seq[row] * max_blocks;
  const T* qr = q + ((long)row * H + head) * DK;
  for (int c = tid; c < DK; c += 256) q_lds[c] = to_f(qr[c]);
  const typename P::Head hp = policy.head(head, H);

  float m = -INFINITY, l = 0.f, acc[NV];
#pragma unroll
  for (int i = 0; i < NV; ++i) acc[i] = 0.f;
  for (int t0 = lo; t0 < L; t0 += 256) {
    const int key = t0 + tid;
    const bool live = key < L;
    __syncthreads();  // q is staged; the previous tile is consumed
    float s = -INFINITY;
    if (live) {
      const long page = (long)bt[key / PBLK] * G + g;
      page_lds[tid] = (int)page;
      const T* k = kpages + (page * PBLK + key % PBLK) * DK;
      float dot = 0.f;
      for (int c = 0; c < DK; c += V) {
        const vec kv = *reinterpret_cast<const vec*>(k + c);
#pragma unroll
        for (int i = 0; i < V; ++i) dot += to_f((T)kv[i]) * q_lds[c + i];
      }
      s = policy.exact_score(dot, hp, (float)(L - 1 - key));
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
      if (c < DV) {
        float a = acc[i] * alpha;
        for (int j = 0; j < nk; ++j)
          a += p_lds[j] * to_f(vpages[((long)page_lds[j] * DV + c) * PBLK +
                                      (t0 + j) % PBLK]);
        acc[i] = a;
      }
    }
  }
  float inv = l > 0.f ? 1.f / l : 0.f;
  if (P::SINK && l > 0.f) {
    const float s = policy.sink_of(head), top = fmaxf(m, s);
    inv = expf(m - top) / (l * expf(m - top) + expf(s - top));
  }
  T* o = out + row * ld_out + (long)head * DV;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = tid + i * 256;
    if (c < DV) {
      float v = acc[i] * inv;
      policy.template finish<T, 1>(row, head, DV, c, &v);
      from_f(o + c, v);
    }
  }
}

template <typename P>
static void launch_attention_rows(const P& policy, const void* q,
                                  const void* kpages, const void* vpages,
                                  const int* block_table, const int* row_seq,
                                  const int* ctx, void* out, long ld_out,
                                  int M, int H, int G, int DK, int DV,
                                  int max_blocks, int chunk, bool fp32,
                                  hipStream_t stream) {
  const int lds = (DK + 256 + 256 + 8) * 4;
#define CR(T, NV)                                                           \
  hipLaunchKernelGGL((attention_rows_kernel<T, NV, P>), dim3(M * H),        \
                     dim3(256), lds, stream, (const T*)q, (const T*)kpages, \
                     (const T*)vpages, policy, block_table, row_seq, ctx,   \
                     (T*)out, ld_out, H, G, DK, DV, max_blocks, chunk)
#define CR_N(T)                  \
  do {                           \
    if (DV <= 256) CR(T, 1);     \
    else if (DV <= 1024) CR(T, 4); \
    else CR(T, 16);              \
  } while (0)
  if (fp32) CR_N(float);
  else CR_N(unsigned short);
#undef CR_N
#undef CR
}

// ---- MFMA kernel of decode rows --------------------------------------------
// A workgroup serves up to 16 query heads of one key/value head of one row;
// NS workgroups share a row's keys. A wave takes every fourth tile of 32
// keys (two pages), both operands straight from the pages: for the scores
// (keys x heads) the 16 x DK key page is the A operand, for the output
// (value columns x heads) the DV x 16 value pages are. Key tile position
// t * 16 + g * 4 + r sits in lane group g of both products' operands, so the
// weights need no exchange between lanes.
template <int DK, int DV, typename P>
__global__ void __launch_bounds__(256, 2)
attention_decode_kernel(const unsigned short* __restrict__ q,
                    const unsigned short* __restrict__ kpages,
                    const unsigned short* __restrict__ vpages, const P policy,
                    const int* __restrict__ block_table,
                    const int* __restrict__ row_seq,
                    const int* __restrict__ ctx,
                    unsigned short* __restrict__ out, long ld_out,
                    float* __restrict__ pacc, float* __restrict__ pml, int H,
                    int G, int NG, int NS, int max_blocks, int chunk) {
  constexpr int OROW = DV + 4;  // padded row of the joining buffer
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int i16 = lane & 15, g = lane >> 4;
  const int split = blockIdx.x % NS;
  const int grp = blockIdx.x / NS % NG;
  const int kvh = blockIdx.x / NS / NG % G;
  const int row = blockIdx.x / NS / NG / G;
  const int GR = H / G;
  const int nlive = min(16, GR - grp * 16);
  const bool live = i16 < nlive;
  const int head = kvh * GR + grp * 16 + (live ? i16 : 0);

  const int L = min(ctx[row], max_blocks * PBLK);
  const int lo = L > 0 ? (L - 1) / chunk * chunk : 0;
  const int T0 = lo / 32, T1 = L > 0 ? (L + 31) / 32 : T0;
  const int per = (T1 - T0 + NS - 1) / NS;
  const int ts = T0 + split * per, te = min(T1, ts + per);
  const int last_page = L > 0 ? (L - 1) / PBLK : 0;
  const int* bt = block_table + (long)row_seq[row] * max_blocks;

  bf16x8 qf[DK / 32];
  {
    const unsigned short* qr = q + ((long)row * H + head) * DK + g * 8;
#pragma unroll
    for (int s = 0; s < DK / 32; ++s) {
      s16x8 v = *reinterpret_cast<const s16x8*>(qr + s * 32);
      if (!live) v = (s16x8)(short)0;
      qf[s] = __builtin_bit_cast(bf16x8, v);
    }
  }
  const typename P::Head hp = policy.head(head, H);

  float m = -1e30f, l = 0.f;
  f32x4 acc[DV / 16];
#pragma unroll
  for (int i = 0; i < DV / 16; ++i) acc[i] = {0.f, 0.f, 0.f, 0.f};

  for (int t = ts + wid; t < te; t += 4) {
    long page[2];
#pragma unroll
    for (int h = 0; h < 2; ++h)
      page[h] = (long)bt[min(t * 2 + h, last_page)] * G + kvh;
    bf16x8 kf[2][DK / 32];
    i32x2 vf[2][DV / 16];
#pragma unroll
    for (int h = 0; h < 2; ++h)
#pragma unroll
      for (int s = 0; s < DK / 32; ++s)
        kf[h][s] = *reinterpret_cast<const bf16x8*>(
            kpages + (page[h] * PBLK + i16) * DK + s * 32 + g * 8);
#pragma unroll
    for (int h = 0; h < 2; ++h)
#pragma unroll
      for (int b = 0; b < DV / 16; ++b)
        vf[h][b] = *reinterpret_cast<const i32x2*>(
            vpages + (page[h] * DV + b * 16 + i16) * PBLK + g * 4);
    float p[2][4];
    float pmax = -INFINITY;
#pragma unroll
    for (int h = 0; h < 2; ++h) {
      f32x4 s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int k = 0; k < DK / 32; ++k)
        s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[h][k], qf[k], s, 0, 0,
                                                    0);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int key = t * 32 + h * 16 + g * 4 + r;
        const float v = policy.score(s[r], hp, (float)(L - 1 - key));
        p[h][r] = key >= lo && key < L ? v : -INFINITY;
        pmax = fmaxf(pmax, p[h][r]);
      }
    }
    pmax = fmaxf(pmax, __shfl_xor(pmax, 16, 64));
    pmax = fmaxf(pmax, __shfl_xor(pmax, 32, 64));
    if (!__all(pmax <= m)) {
      const float mn = fmaxf(m, pmax);
      const float alpha = __builtin_amdgcn_exp2f(m - mn);
      m = mn;
      l *= alpha;
#pragma unroll
      for (int i = 0; i < DV / 16; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) acc[i][r] *= alpha;
    }
    s16x8 pb;
#pragma unroll
    for (int h = 0; h < 2; ++h)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float e = __builtin_amdgcn_exp2f(p[h][r] - m);
        l += e;  // this lane's keys only; lanes are joined at the end
        pb[h * 4 + r] = (short)f2bf(e);
      }
    const bf16x8 pf = __builtin_bit_cast(bf16x8, pb);
#pragma unroll
    for (int b = 0; b < DV / 16; ++b) {
      i32x4 v;
      v[0] = vf[0][b][0];
      v[1] = vf[0][b][1];
      v[2] = vf[1][b][0];
      v[3] = vf[1][b][1];
      acc[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
          __builtin_bit_cast(bf16x8, v), pf, acc[b], 0, 0, 0);
    }
  }
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);

  // join the four waves
  float* wm = reinterpret_cast<float*>(smem);  // [4][16]
  float* wl = wm + 64;                         // [4][16]
  float* wo = wl + 64;                         // [4][16][OROW]
  if (g == 0) {
    wm[wid * 16 + i16] = m;
    wl[wid * 16 + i16] = l;
  }
#pragma unroll
  for (int b = 0; b < DV / 16; ++b)
    *reinterpret_cast<f32x4*>(wo + (wid * 16 + i16) * OROW + b * 16 + g * 4) =
        acc[b];
  __syncthreads();
  for (int i = threadIdx.x; i < nlive * (DV / 4); i += 256) {
    const int hl = i / (DV / 4), c = i % (DV / 4) * 4;
    float M = -1e30f, lsum = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) M = fmaxf(M, wm[w * 16 + hl]);
    f32x4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int w = 0; w < 4; ++w) {
      const float a = __builtin_amdgcn_exp2f(wm[w * 16 + hl] - M);
      lsum += a * wl[w * 16 + hl];
      const f32x4 v =
          *reinterpret_cast<const f32x4*>(wo + (w * 16 + hl) * OROW + c);
#pragma unroll
      for (int r = 0; r < 4; ++r) o[r] += a * v[r];
    }
    const int hd = kvh * GR + grp * 16 + hl;
    const long rh = (long)row * H + hd;
    if (NS == 1) {
      const float inv = softmax_factor(policy, hd, M, lsum);
      float v[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) v[r] = o[r] * inv;
      policy.template finish<unsigned short, 4>(row, hd, DV, c, v);
      s16x4 ov;
#pragma unroll
      for (int r = 0; r < 4; ++r) ov[r] = (short)f2bf(v[r]);
      *reinterpret_cast<s16x4*>(out + row * ld_out + (long)hd * DV + c) = ov;
    } else {
      *reinterpret_cast<f32x4*>(pacc + (rh * NS + split) * DV + c) = o;
      if (c == 0) {
        pml[(rh * NS + split) * 2] = M;
        pml[(rh * NS + split) * 2 + 1] = lsum;
      }
    }
  }
}

// one wave per (row, head): join NS partial results
template <typename P>
__global__ void __launch_bounds__(256)
attention_combine_kernel(const float* __restrict__ pacc,
                         const float* __restrict__ pml, const P policy,
                         unsigned short* __restrict__ out, long ld_out,
                         int RH, int H, int DV, int NS) {
  const int lane = threadIdx.x & 63;
  const long rh = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (rh >= RH) return;
  float M = -1e30f;
  for (int s = 0; s < NS; ++s) M = fmaxf(M, pml[(rh * NS + s) * 2]);
  float l = 0.f;
  for (int s = 0; s < NS; ++s)
    l += pml[(rh * NS + s) * 2 + 1] *
         __builtin_amdgcn_exp2f(pml[(rh * NS + s) * 2] - M);
  const int row = (int)(rh / H), hd = (int)(rh % H);
  const float inv = softmax_factor(policy, hd, M, l);
  for (int c = lane * 4; c < DV; c += 256) {
    f32x4 o = {0.f, 0.f, 0.f, 0.f};
    for (int s = 0; s < NS; ++s) {
      const float a =
          __builtin_amdgcn_exp2f(pml[(rh * NS + s) * 2] - M) * inv;
      const f32x4 v =
          *reinterpret_cast<const f32x4*>(pacc + (rh * NS + s) * DV + c);
#pragma unroll
      for (int i = 0; i < 4; ++i) o[i] += a * v[i];
    }
    float v[4] = {o[0], o[1], o[2], o[3]};
    policy.template finish<unsigned short, 4>(row, hd, DV, c, v);
    s16x4 ov;
#pragma unroll
    for (int i = 0; i < 4; ++i) ov[i] = (short)f2bf(v[i]);
    *reinterpret_cast<s16x4*>(out + row * ld_out + (long)hd * DV + c) = ov;
  }
}

template <typename P>
static void launch_attention_decode(
    const P& policy, const void* q, const void* kpages, const void* vpages,
    const int* block_table, const int* row_seq, const int* ctx, void* out,
    long ld_out, void* pacc, void* pml, int M, int H, int G, int DK, int DV,
    int NS, int max_blocks, int chunk, hipStream_t stream) {
  const int ng = (H / G + 15) / 16;
#define CD(KK, VV)                                                          \
  hipLaunchKernelGGL((attention_decode_kernel<KK, VV, P>),                  \
                     dim3((long)M * G * ng * NS), dim3(256),                \
                     (128 + 64 * (VV + 4)) * 4, stream,                     \
                     (const unsigned short*)q, (const unsigned short*)kpages, \
                     (const unsigned short*)vpages, policy, block_table,    \
                     row_seq, ctx, (unsigned short*)out, ld_out,            \
                     (float*)pacc, (float*)pml, H, G, ng, NS, max_blocks,   \
                     chunk)
#define CD_V(KK)               \
  do {                         \
    if (DV == 64) CD(KK, 64);  \
    else if (DV == 128) CD(KK, 128); \
    else CD(KK, 256);          \
  } while (0)
  if (DK == 64) CD_V(64);
  else if (DK == 128) CD_V(128);
  else CD_V(256);
#undef CD_V
#undef CD
  if (NS > 1)
    hipLaunchKernelGGL(attention_combine_kernel<P>, dim3((M * H + 3) / 4),
                       dim3(256), 0, stream, (const float*)pacc,
                       (const float*)pml, policy, (unsigned short*)out,
                       ld_out, M * H, H, DV, NS);
}
