// MFMA attention of single-token rows over paged bf16 latents (see
// latent_attention.hip for the mechanism, the cache layout and the row
// arguments; that file's one-head kernel covers the other types and ranks).
//
// A workgroup serves HG groups of 16 heads of one row, so a latent is read
// from HBM once for all of them; the visible keys of a row are split over NS
// workgroups whose partial results a second kernel joins.
//
// Tiles of 32 keys go global -> registers -> LDS, where each tile is kept
// twice: row-major (key operand of the score product) and transposed (the
// same numbers as value operand). The next tile's loads are in flight while
// the current one is used.
//
// KS waves work on each head group. For the scores they split the keys of
// the tile (and, when KS is 4, the latent columns, whose partial sums meet
// in LDS); for the output each owns R / KS latent columns, which keeps the
// accumulators of a wave small. Both products use
// mfma_f32_16x16x32_bf16 with keys (then latent columns) as rows and heads
// as columns, so softmax state and rescaling are lane-local.
//
// Cache rows and queries have RR = R + ROT numbers, of which all take part in
// the scores and the first R are the value. The others need no transposed
// copy: they go to LDS directly, while the tile before is weighted.
#include "common.h"

#define PBLK 16
#define KT 32
#define LOG2E 1.4426950408889634f

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;

extern __shared__ __attribute__((aligned(16))) char smem[];

#define SROW 36  // padded row of 32 scores

// byte address of the 16-byte slot (4 per row: 32 keys) of latent column r;
// 64 bytes of padding per 8 rows and the slot swizzle spread the banks
__device__ __forceinline__ int ct_slot(int r, int slot) {
  return r * 64 + (r >> 3) * 64 + ((slot ^ ((r >> 2) & 3)) * 16);
}

// Weight of a row's sum: 1 / l with the softmax's state m (log2 units), l and
// the sink of the head, times its gate.
__device__ __forceinline__ float row_weight(float m, float l, long row,
                                            int head, const float* sink,
                                            const unsigned short* gate,
                                            int ld_gate) {
  float inv = l > 0.f ? 1.f / l : 0.f;
  if (sink != nullptr && l > 0.f) {
    const float s = sink[head] * LOG2E, top = fmaxf(m, s);
    const float a = __builtin_amdgcn_exp2f(m - top);
    inv = a / (l * a + __builtin_amdgcn_exp2f(s - top));
  }
  if (gate != nullptr) inv *= sigmoid_exact(bf2f(gate[row * ld_gate + head]));
  return inv;
}

template <int R, int ROT, int HG, int KS>
__global__ void __launch_bounds__(64 * HG * KS, 2)
latent_decode_kernel(const unsigned short* __restrict__ q,
                     const unsigned short* __restrict__ cache,
                     const int* __restrict__ block_table,
                     const int* __restrict__ row_seq,
                     const int* __restrict__ ctx,
                     unsigned short* __restrict__ out,
                     float* __restrict__ pacc, float* __restrict__ pml,
                     int H, int NG, int NS, int max_blocks, int window,
                     float scale, const float* __restrict__ sink,
                     const unsigned short* __restrict__ gate, int ld_gate) {
  constexpr int NT = 64 * HG * KS;
  constexpr int RR = R + ROT;
  constexpr int UNITS = R;  // a unit: 4 keys x 8 latent columns
  constexpr int UPT = (UNITS + NT - 1) / NT;
  constexpr int SW = R % 128 == 0 ? 15 : 7;
  constexpr int CT = KT * R * 2;        // LDS offset of the transposed copy
  constexpr int SC = CT + R * 72;       // LDS offset of the scores
  constexpr int RSPLIT = KS / 2;       // column parts, besides key halves
  constexpr int RO = SC + HG * RSPLIT * 16 * SROW * 4;  // of the key parts
  constexpr int QS = R / 32 / RSPLIT;  // score steps of a wave
  constexpr int TS = ROT / 32 / RSPLIT;  // and those behind the latent
  constexpr int OB = R / 16 / KS;      // output blocks of a wave
  static_assert(KS == 2 || KS == 4, "two key halves");

  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int i16 = lane & 15, g = lane >> 4;
  const int hgrp = wid / KS, ks = wid % KS;
  const int khalf = ks % 2, rhalf = ks / 2;
  const int split = blockIdx.x % NS;
  const int grp = blockIdx.x / NS % NG;
  const int row = blockIdx.x / NS / NG;
  const int head = (grp * HG + hgrp) * 16 + i16;
  const bool live = head < H;

  const int L = min(ctx[row], max_blocks * PBLK);
  const int lo = L > window ? L - window : 0;
  const int T0 = lo / KT, T1 = L > 0 ? (L + KT - 1) / KT : T0;
  const int per = (T1 - T0 + NS - 1) / NS;
  const int ts = T0 + split * per, te = min(T1, ts + per);
  const int last_page = L > 0 ? (L - 1) / PBLK : 0;
  const int* bt = block_table + (long)row_seq[row] * max_blocks;

  const int kg = (threadIdx.x >> 3) & 7;  // key group of all my units
  auto page_of = [&](int t) {
    return bt[min(t * (KT / PBLK) + (kg >> 2), last_page)];
  };
  i32x4 kv[UPT][4];
  auto issue = [&](int page) {
    const unsigned short* base =
        cache + ((long)page * PBLK + (kg & 3) * 4) * RR;
#pragma unroll
    for (int i = 0; i < UPT; ++i) {
      const int u = threadIdx.x + i * NT;
      if (UNITS % NT == 0 || u < UNITS) {
        const int c = (u >> 6) * 8 + (u & 7);
#pragma unroll
        for (int j = 0; j < 4; ++j)
          kv[i][j] =
              *reinterpret_cast<const i32x4*>(base + (long)j * RR + c * 8);
      }
    }
  };
  auto stage = [&]() {
#pragma unroll
    for (int i = 0; i < UPT; ++i) {
      const int u = threadIdx.x + i * NT;
      if (UNITS % NT == 0 || u < UNITS) {
        const int c = (u >> 6) * 8 + (u & 7);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const int key = kg * 4 + j;
          *reinterpret_cast<i32x4*>(smem + key * (R * 2) +
                                    ((c ^ (key & SW)) * 16)) = kv[i][j];
        }
#pragma unroll
        for (int w = 0; w < 4; ++w) {
          i32x2 even, odd;
          even[0] = __builtin_amdgcn_perm(kv[i][1][w], kv[i][0][w],
                                          0x05040100);
          even[1] = __builtin_amdgcn_perm(kv[i][3][w], kv[i][2][w],
                                          0x05040100);
          odd[0] = __builtin_amdgcn_perm(kv[i][1][w], kv[i][0][w],
                                         0x07060302);
          odd[1] = __builtin_amdgcn_perm(kv[i][3][w], kv[i][2][w],
                                         0x07060302);
          const int r = c * 8 + w * 2;
          char* dst = smem + CT + (kg & 1) * 8;
          *reinterpret_cast<i32x2*>(dst + ct_slot(r, kg >> 1)) = even;
          *reinterpret_cast<i32x2*>(dst + ct_slot(r + 1, kg >> 1)) = odd;
        }
      }
    }
  };

  // key parts: four waves copy eight keys each
  auto part_page = [&](int t) {
    return bt[min(t * (KT / PBLK) + (wid >> 1), last_page)];
  };
  auto stage_part = [&](int page) {
    static_assert(ROT == 0 || ROT == 64, "eight 16-byte pieces per key");
    if (wid >= 4) return;
    const int key = wid * 8 + (lane >> 3);
    const unsigned short* src = cache +
                                ((long)page * PBLK + (key & 15)) * RR + R +
                                ((lane & 7) ^ (key & 7)) * 8;
    auto dst = (__attribute__((address_space(3))) unsigned int*)(
        smem + RO + wid * 1024 + lane * 16);
    __builtin_amdgcn_global_load_lds(
        (const __attribute__((address_space(1))) unsigned int*)src, dst, 16,
        0, 0);
  };

  int page = 0, ppage = 0;
  if (ts < te) {
    issue(page_of(ts));
    page = page_of(min(ts + 1, te - 1));
    if (ROT > 0) {
      stage_part(part_page(ts));
      ppage = part_page(min(ts + 1, te - 1));
    }
  }
  bf16x8 qf[QS + TS];
  {
    const unsigned short* qr =
        q + ((long)row * H + (live ? head : 0)) * RR + g * 8;
#pragma unroll
    for (int s = 0; s < QS + TS; ++s) {
      s16x8 v = *reinterpret_cast<const s16x8*>(
          qr + (s < QS ? (rhalf * QS + s) * 32
                       : R + (rhalf * TS + s - QS) * 32));
      if (!live) v = (s16x8)(short)0;
      qf[s] = __builtin_bit_cast(bf16x8, v);
    }
  }

  float m = -1e30f, l = 0.f;
  f32x4 acc[OB];
#pragma unroll
  for (int i = 0; i < OB; ++i) acc[i] = {0.f, 0.f, 0.f, 0.f};
  const float scale2 = scale * LOG2E;
  float* scores = reinterpret_cast<float*>(smem + SC) +
                  hgrp * (RSPLIT * 16 * SROW) + i16 * SROW;

  for (int t = ts; t < te; ++t) {
    __syncthreads();  // every wave is done with the previous tile
    if (ROT > 0) asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    stage();
    if (t + 1 < te) {
      issue(page);
      page = page_of(min(t + 2, te - 1));
    }
    __syncthreads();

    // scores of my keys over my columns, in two chains
    f32x4 sa[2];
    sa[0] = {0.f, 0.f, 0.f, 0.f};
    sa[1] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int s = 0; s < QS; ++s) {
      const int chunk = (rhalf * QS + s) * 4 + g;
      const char* a = smem + (khalf * 16 + i16) * (R * 2) +
                      ((chunk ^ (i16 & SW)) * 16);
      const bf16x8 k0 = *reinterpret_cast<const bf16x8*>(a);
      sa[s & 1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
          k0, qf[s], sa[s & 1], 0, 0, 0);
    }
#pragma unroll
    for (int s = 0; s < TS; ++s) {
      const int chunk = (rhalf * TS + s) * 4 + g;
      const bf16x8 k0 = *reinterpret_cast<const bf16x8*>(
          smem + RO + (khalf * 16 + i16) * 128 + ((chunk ^ (i16 & 7)) * 16));
      sa[s & 1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
          k0, qf[QS + s], sa[s & 1], 0, 0, 0);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) sa[0][r] += sa[1][r];
    *reinterpret_cast<f32x4*>(scores + rhalf * (16 * SROW) + khalf * 16 +
                              g * 4) = sa[0];
    __syncthreads();
    if (ROT > 0 && t + 1 < te) {
      stage_part(ppage);
      ppage = part_page(min(t + 2, te - 1));
    }

    // weights of all 32 keys for my head: lane group g has keys g*8 .. + 7
    float p[8];
    float pmax = -INFINITY;
#pragma unroll
    for (int h = 0; h < 2; ++h) {
      f32x4 v = *reinterpret_cast<const f32x4*>(scores + g * 8 + h * 4);
      if (RSPLIT == 2) {
        const f32x4 v2 = *reinterpret_cast<const f32x4*>(
            scores + 16 * SROW + g * 8 + h * 4);
#pragma unroll
        for (int r = 0; r < 4; ++r) v[r] += v2[r];
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int key = t * KT + g * 8 + h * 4 + r;
        p[h * 4 + r] = key >= lo && key < L ? v[r] * scale2 : -INFINITY;
        pmax = fmaxf(pmax, p[h * 4 + r]);
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
      for (int i = 0; i < OB; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) acc[i][r] *= alpha;
    }
    s16x8 pb;
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const float e = __builtin_amdgcn_exp2f(p[i] - m);
      l += e;  // this lane's keys only; lanes are joined at the end
      pb[i] = (short)f2bf(e);
    }
    const bf16x8 pf = __builtin_bit_cast(bf16x8, pb);
#pragma unroll
    for (int i = 0; i < OB; ++i) {
      const bf16x8 v = *reinterpret_cast<const bf16x8*>(
          smem + CT + ct_slot((ks * OB + i) * 16 + i16, g));
      acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, pf, acc[i], 0, 0,
                                                       0);
    }
  }
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  if (!live) return;
  const long rh = (long)row * H + head;
  const int col = ks * (OB * 16) + g * 4;
  if (NS == 1) {
    const float inv = row_weight(m, l, row, head, sink, gate, ld_gate);
#pragma unroll
    for (int i = 0; i < OB; ++i) {
      s16x4 o;
#pragma unroll
      for (int r = 0; r < 4; ++r) o[r] = (short)f2bf(acc[i][r] * inv);
      *reinterpret_cast<s16x4*>(out + rh * R + col + i * 16) = o;
    }
  } else {
    const long part = rh * NS + split;
#pragma unroll
    for (int i = 0; i < OB; ++i)
      *reinterpret_cast<f32x4*>(pacc + part * R + col + i * 16) = acc[i];
    if (g == 0 && ks == 0) {
      pml[part * 2] = m;
      pml[part * 2 + 1] = l;
    }
  }
}

// one wave per (row, head): join NS partial results
__global__ void __launch_bounds__(256)
latent_combine_kernel(const float* __restrict__ pacc,
                      const float* __restrict__ pml,
                      unsigned short* __restrict__ out, int RH, int R,
                      int NS, int H, const float* __restrict__ sink,
                      const unsigned short* __restrict__ gate, int ld_gate) {
  const int lane = threadIdx.x & 63;
  const long rh = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (rh >= RH) return;
  float M = -1e30f;
  for (int s = 0; s < NS; ++s) M = fmaxf(M, pml[(rh * NS + s) * 2]);
  float l = 0.f;
  for (int s = 0; s < NS; ++s)
    l += pml[(rh * NS + s) * 2 + 1] *
         __builtin_amdgcn_exp2f(pml[(rh * NS + s) * 2] - M);
  const float inv =
      row_weight(M, l, rh / H, (int)(rh % H), sink, gate, ld_gate);
  for (int c = lane * 4; c < R; c += 256) {
    f32x4 o = {0.f, 0.f, 0.f, 0.f};
    for (int s = 0; s < NS; ++s) {
      const float a =
          __builtin_amdgcn_exp2f(pml[(rh * NS + s) * 2] - M) * inv;
      const f32x4 v =
          *reinterpret_cast<const f32x4*>(pacc + (rh * NS + s) * R + c);
#pragma unroll
      for (int i = 0; i < 4; ++i) o[i] += a * v[i];
    }
    s16x4 ov;
#pragma unroll
    for (int i = 0; i < 4; ++i) ov[i] = (short)f2bf(o[i]);
    *reinterpret_cast<s16x4*>(out + rh * R + c) = ov;
  }
}

// heads that one workgroup serves
extern "C" int latent_decode_heads(int H) {
  return H <= 16 ? 16 : H <= 32 ? 32 : 64;
}

extern "C" bool latent_decode_covers(int R, int rot) {
  if (rot != 0 && rot != 64) return false;
  return R == 64 || R == 128 || R == 192 || R == 256 || R == 384 || R == 512;
}

extern "C" void launch_latent_decode(
    const void* q, const void* cache, const int* block_table,
    const int* row_seq, const int* ctx, void* out, void* pacc, void* pml,
    int M, int H, int R, int rot, int NS, int max_blocks, int window,
    float scale, const float* sink, const void* gate, int ld_gate,
    hipStream_t stream) {
  const int heads = latent_decode_heads(H);
  const int ng = (H + heads - 1) / heads;
#define LD(RR, RO, HG, KS)                                                    \
  hipLaunchKernelGGL((latent_decode_kernel<RR, RO, HG, KS>),                  \
                     dim3(M * ng * NS), dim3(64 * HG * KS),                   \
                     KT * (RR + RO) * 2 + RR * 72 +                           \
                         HG * (KS == 4 ? 2 : 1) * 16 * SROW * 4,              \
                     stream, (const unsigned short*)q,                        \
                     (const unsigned short*)cache, block_table, row_seq, ctx, \
                     (unsigned short*)out, (float*)pacc, (float*)pml, H, ng,  \
                     NS, max_blocks, window, scale, sink,                     \
                     (const unsigned short*)gate, ld_gate)
#define LD_H(RR, RO)                      \
  do {                                    \
    if (heads == 16) LD(RR, RO, 1, 4);    \
    else if (heads == 32) LD(RR, RO, 2, 2); \
    else LD(RR, RO, 4, 2);                \
  } while (0)
#define LD_R(RR)              \
  do {                        \
    if (rot == 0) LD_H(RR, 0); \
    else LD_H(RR, 64);        \
  } while (0)
  switch (R) {
    case 64: LD_R(64); break;
    case 128: LD_R(128); break;
    case 192: LD_R(192); break;
    case 256: LD_R(256); break;
    case 384: LD_R(384); break;
    default: LD_R(512); break;
  }
#undef LD_R
#undef LD_H
#undef LD
  if (NS > 1)
    hipLaunchKernelGGL(latent_combine_kernel, dim3((M * H + 3) / 4),
                       dim3(256), 0, stream, (const float*)pacc,
                       (const float*)pml, (unsigned short*)out, M * H, R, NS,
                       H, sink, (const unsigned short*)gate, ld_gate);
}
