// Flash attention of prompt portions over paged keys and values (see
// chunk_attention.h), bf16.
//
// A workgroup of four waves serves 128 consecutive queries of one portion
// and head, 32 per wave; key tiles of 64 (four pages) pass through LDS in
// two buffers. Keys and transposed values come from their pages by
// global_load_lds alone: value pages are already the A operand of the
// output product. The scores are computed transposed (keys x queries), so
// a lane holds 32 scores of one query and the softmax state is lane-local
// up to one exchange between the halves of the wave.
#pragma once
#include "chunk_attention.h"

#define KVBLK 64
#define QWAVE 32

extern __shared__ __attribute__((aligned(16))) char smem[];

union frag_u {
  bf16x8 v;
  unsigned int d[4];
};

__device__ __forceinline__ void load_lds16(const unsigned short* src,
                                           char* dst) {
  __builtin_amdgcn_global_load_lds(
      (const __attribute__((address_space(1))) unsigned int*)src,
      (__attribute__((address_space(3))) unsigned int*)dst, 16, 0, 0);
}

template <int DK, int DV, typename P>
__global__ void __launch_bounds__(256, DK + DV <= 256 ? 2 : 1)
attention_flash_kernel(const unsigned short* __restrict__ Q,
                   const unsigned short* __restrict__ kpages,
                   const unsigned short* __restrict__ vpages, const P policy,
                   unsigned short* __restrict__ O, long ld_out,
                   const int* __restrict__ block_table, int max_blocks,
                   const int* __restrict__ portions,
                   const int* __restrict__ blocks, int nblocks, int H, int G,
                   int chunk) {
  constexpr int NCH = DK / 8;              // 16-byte units per key
  constexpr int DBLK = DV / 32;
  constexpr int KTILE = KVBLK * DK * 2;    // bytes
  constexpr int VTILE = KVBLK * DV * 2;
  constexpr int KPIECES = KTILE / 1024, VPIECES = VTILE / 1024;
  constexpr int KROWS = 1024 / (2 * DK);   // keys per piece
  constexpr int VPP = DV / 32;             // pieces per value page

  const int lane = threadIdx.x & 63;
  const int wid = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int h = lane >> 5, qcol = lane & 31;

  // neighbouring query blocks of a head share most of their keys: give
  // each XCD a contiguous run of them
  const int bid = xcd_run(blockIdx.x, gridDim.x);
  const int head = bid / nblocks;
  const int* pm = portions + blocks[(bid % nblocks) * 2] * 4;
  const int qb = blocks[(bid % nblocks) * 2 + 1];
  const int seq = pm[0], row0 = pm[1], start = pm[2], n = pm[3];
  const int kvh = head / (H / G);
  const int* bt = block_table + (long)seq * max_blocks;

  const int q0w = qb * (4 * QWAVE) + wid * QWAVE;  // first query of the wave
  const int qpos = start + q0w + qcol;
  const int qlo = qpos / chunk * chunk;
  const int wlo = (start + q0w) / chunk * chunk;
  const int last = start + min(qb * 4 * QWAVE + 4 * QWAVE, n) - 1;
  const int tile0 = (start + qb * 4 * QWAVE) / chunk * chunk / KVBLK;
  const int ntile = last / KVBLK + 1;
  const int last_page = min(last / PBLK, max_blocks - 1);

  const int offK[2] = {0, KTILE};
  const int offV[2] = {2 * KTILE, 2 * KTILE + VTILE};

  bf16x8 qf[DK / 16];
  {
    const int qr = row0 + min(q0w + qcol, n - 1);
    const unsigned short* src = Q + ((long)qr * H + head) * DK + h * 8;
#pragma unroll
    for (int s = 0; s < DK / 16; ++s)
      qf[s] = *reinterpret_cast<const bf16x8*>(src + s * 16);
  }
  const typename P::Head hp = policy.head(head, H);

  float m = -1e30f, l = 0.f;
  f32x16 accO[DBLK];
#pragma unroll
  for (int d = 0; d < DBLK; ++d)
#pragma unroll
    for (int i = 0; i < 16; ++i) accO[d][i] = 0.f;

  // lane (i & 3) holds the i-th page of a tile
  auto pages_of = [&](int t) {
    return bt[min(t * (KVBLK / PBLK) + (lane & 3), last_page)];
  };
  auto stage = [&](int pages, int buf) {
#pragma unroll
    for (int i = 0; i < KPIECES / 4; ++i) {
      const int p = wid + i * 4;
      const int row = p * KROWS + lane / NCH;
      const int c = (lane % NCH) ^ (row & (NCH - 1));
      const long page =
          __builtin_amdgcn_readlane(pages, p * KROWS / PBLK);
      load_lds16(kpages + ((page * G + kvh) * PBLK + row % PBLK) * DK + c * 8,
                 smem + offK[buf] + p * 1024 + lane * 16);
    }
#pragma unroll
    for (int i = 0; i < VPIECES / 4; ++i) {
      const int p = wid + i * 4;
      const int row = p % VPP * 32 + lane / 2;
      const int half = (lane & 1) ^ ((row >> 3) & 1);
      const long page = __builtin_amdgcn_readlane(pages, p / VPP);
      load_lds16(vpages + ((page * G + kvh) * DV + row) * PBLK + half * 8,
                 smem + offV[buf] + p * 1024 + lane * 16);
    }
  };

  int pages = pages_of(tile0);
  stage(pages, 0);
  pages = pages_of(tile0 + 1);
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  __syncthreads();

  int cur = 0;
  for (int t = tile0; t < ntile; ++t) {
    const int k0 = t * KVBLK;
    if (t + 1 < ntile) {
      stage(pages, cur ^ 1);
      pages = pages_of(t + 2);
    }
    const bool wave_active = q0w < n && k0 <= start + q0w + QWAVE - 1 &&
                             k0 + KVBLK > wlo;
    if (wave_active) {
      // key k is visible when 0 <= k - qlo <= qpos - qlo: one unsigned
      // compare, free of branches
      const unsigned int span = qpos - qlo;
      const int koff = k0 + 4 * h - qlo;
      const float qdist = (float)(qpos - k0 - 4 * h);
      float p[32];
      float pmax = -1e30f;
#pragma unroll
      for (int kb = 0; kb < 2; ++kb) {
        f32x16 accP;
#pragma unroll
        for (int i = 0; i < 16; ++i) accP[i] = 0.f;
        __builtin_amdgcn_s_setprio(1);
#pragma unroll
        for (int s = 0; s < DK / 16; ++s) {
          const int key = kb * 32 + qcol;
          const int c = (s * 2 + h) ^ (key & (NCH - 1));
          const bf16x8 kf = *reinterpret_cast<const bf16x8*>(
              smem + offK[cur] + key * (2 * DK) + c * 16);
          accP = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf, qf[s], accP, 0,
                                                         0, 0);
        }
        __builtin_amdgcn_s_setprio(0);
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const int key = kb * 32 + (r & 3) + 8 * (r >> 2);
          const float s = policy.score(accP[r], hp, qdist - (float)key);
          p[kb * 16 + r] =
              (unsigned int)(koff + key) <= span ? s : -INFINITY;
          pmax = fmaxf(pmax, p[kb * 16 + r]);
        }
      }
      pmax = fmaxf(pmax, __shfl_xor(pmax, 32, 64));
      // the accumulators are rescaled only when the running maximum has
      // grown by more than 2^8, which fp32 sums absorb
      float mn = m, alpha = 1.f;
      if (!__all(pmax - m <= 8.f)) {
        mn = fmaxf(m, pmax);
        alpha = __builtin_amdgcn_exp2f(m - mn);
#pragma unroll
        for (int d = 0; d < DBLK; ++d)
#pragma unroll
          for (int i = 0; i < 16; ++i) accO[d][i] *= alpha;
      }
      float rs = 0.f;
#pragma unroll
      for (int r = 0; r < 32; ++r) {
        p[r] = __builtin_amdgcn_exp2f(p[r] - mn);
        rs += p[r];
      }
      rs += __shfl_xor(rs, 32, 64);
      l = l * alpha + rs;
      m = mn;
      // weights of 16 keys (a page) -> B operand, then their product
#pragma unroll
      for (int kh = 0; kh < 4; ++kh) {
        const float* pp = p + kh * 8;
        unsigned int w[4];
#pragma unroll
        for (int i = 0; i < 4; ++i)
          w[i] = ((unsigned int)f2bf(pp[2 * i])) |
                 ((unsigned int)f2bf(pp[2 * i + 1]) << 16);
        const i32x2 s0 = __builtin_amdgcn_permlane32_swap((int)w[0],
                                                          (int)w[2], false,
                                                          false);
        const i32x2 s1 = __builtin_amdgcn_permlane32_swap((int)w[1],
                                                          (int)w[3], false,
                                                          false);
        frag_u pa;
        pa.d[0] = (unsigned int)s0[0];
        pa.d[1] = (unsigned int)s1[0];
        pa.d[2] = (unsigned int)s0[1];
        pa.d[3] = (unsigned int)s1[1];
        __builtin_amdgcn_s_setprio(1);
#pragma unroll
        for (int d = 0; d < DBLK; ++d) {
          const int row = d * 32 + qcol;
          const bf16x8 vf = *reinterpret_cast<const bf16x8*>(
              smem + offV[cur] + kh * (DV * 32) + row * 32 +
              ((h ^ ((row >> 3) & 1)) * 16));
          accO[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, pa.v,
                                                            accO[d], 0, 0, 0);
        }
        __builtin_amdgcn_s_setprio(0);
      }
    }
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();  // one barrier per tile
    cur ^= 1;
  }

  // ---- O^T in registers -> padded LDS -> coalesced stores -----------------
  const float inv_l = softmax_factor(policy, head, m, l);
  float* oimg = reinterpret_cast<float*>(smem) + wid * QWAVE * (DV + 1);
#pragma unroll
  for (int d = 0; d < DBLK; ++d)
#pragma unroll
    for (int r = 0; r < 16; ++r)
      oimg[qcol * (DV + 1) + d * 32 + (r & 3) + 8 * (r >> 2) + 4 * h] =
          accO[d][r] * inv_l;
  __syncthreads();
  constexpr int LPR = DV / 4 < 64 ? DV / 4 : 64;  // lanes per query
  const int c = lane % LPR * 4;
  for (int q = lane / LPR; q < QWAVE; q += 64 / LPR) {
    if (q0w + q >= n) break;
    const long row = row0 + q0w + q;
    float v[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = oimg[q * (DV + 1) + c + i];
    policy.template finish<unsigned short, 4>(row, head, DV, c, v);
    s16x4 ov;
#pragma unroll
    for (int i = 0; i < 4; ++i) ov[i] = (short)f2bf(v[i]);
    *reinterpret_cast<s16x4*>(O + row * ld_out + (long)head * DV + c) = ov;
  }
}

template <typename P>
static void launch_attention_flash(
    const P& policy, const void* Q, const void* kpages, const void* vpages,
    void* O, long ld_out, const int* block_table, int max_blocks,
    const int* portions, const int* blocks, int nblocks, int H, int G, int DK,
    int DV, int chunk, hipStream_t stream) {
  const int stage_b = 2 * KVBLK * 2 * (DK + DV);
  const int epi_b = 4 * QWAVE * (DV + 1) * 4;
  const int lds = stage_b > epi_b ? stage_b : epi_b;
#define CF(KK, VV)                                                          \
  hipLaunchKernelGGL((attention_flash_kernel<KK, VV, P>), dim3(nblocks * H), \
                     dim3(256), lds, stream, (const unsigned short*)Q,      \
                     (const unsigned short*)kpages,                         \
                     (const unsigned short*)vpages, policy,                 \
                     (unsigned short*)O, ld_out, block_table, max_blocks,   \
                     portions, blocks, nblocks, H, G, chunk)
#define CF_V(KK)               \
  do {                         \
    if (DV == 64) CF(KK, 64);  \
    else if (DV == 128) CF(KK, 128); \
    else CF(KK, 256);          \
  } while (0)
  if (DK == 64) CF_V(64);
  else if (DK == 128) CF_V(128);
  else CF_V(256);
#undef CF_V
#undef CF
}
