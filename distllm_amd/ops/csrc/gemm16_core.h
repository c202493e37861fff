// Main loop of the 256 x 256 x 64 deep-pipelined MFMA product (see
// gemm16.hip for the schedule), for kernels that differ in where the rows
// of A come from and in their epilogues.
#pragma once
#include "common.h"

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;

#define G16_BM 256
#define G16_BN 256
#define G16_BK 64
#define G16_HTILE_B (128 * G16_BK * 2)  // one half image: 16 KiB
#define G16_LDS (8 * G16_HTILE_B)       // 2 buf x {A,B} x 2 half = 128 KiB

extern __shared__ __attribute__((aligned(16))) char smem16[];

__device__ __forceinline__ int g16_img_off(int row, int c16) {
  return row * 128 + ((c16 ^ (row & 7)) * 16);
}

// stage_a(k0, buf, half), stage_b(k0, buf, half): start the copies of one
// half image (128 rows x 64 columns from column k0 on) by g16_stage. On
// return the LDS is free for the epilogue. acc[mi][ni]: rows mw * 128 +
// mi * 16, columns nw * 64 + ni * 16 of the tile.
__device__ __forceinline__ char* g16_img(int op, int buf, int half) {
  return smem16 + ((op * 2 + buf) * 2 + half) * G16_HTILE_B;
}

// piece pp (0, 1) of a wave's share of a half image; src: this lane's row
// and, XOR-swizzled by it, 16-byte column
__device__ __forceinline__ void g16_stage(const unsigned short* src, int op,
                                          int buf, int half, int pp, int wid,
                                          int lane) {
  auto dst = (__attribute__((address_space(3))) unsigned int*)(
      g16_img(op, buf, half) + (wid * 2 + pp) * 1024 + lane * 16);
  __builtin_amdgcn_global_load_lds(
      (const __attribute__((address_space(1))) unsigned int*)src, dst, 16, 0,
      0);
}

template <typename StageA, typename StageB>
__device__ __forceinline__ void g16_mainloop(const StageA& stage_a,
                                             const StageB& stage_b, int K,
                                             int lane, int mw, int nw,
                                             f32x4 (&acc)[8][4]) {
  const int fr_row = lane & 15;
  const int fr_c = lane >> 4;  // kk sub-chunk 0..3 (8 bf16 each)
  auto read_frag = [&](const char* image, int row16, int kk) {
    return *reinterpret_cast<const bf16x8*>(
        image + g16_img_off(row16 * 16 + fr_row, kk * 4 + fr_c));
  };

#pragma unroll
  for (int i = 0; i < 8; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = {0.f, 0.f, 0.f, 0.f};

  const int bh = nw >> 1;         // wave's B half image
  const int br16 = (nw & 1) * 4;  // local row16 base within it
  const int nt = K / G16_BK;      // even (host guarantees K%128==0)

  // ---- prologue: tile 0 complete + B0(1); steady state stages the
  // rest of tile 1 at ph0/ph1 of the first iteration ----------------
  stage_a(0, 0, 0);
  stage_a(0, 0, 1);
  stage_b(0, 0, 0);
  stage_b(0, 0, 1);
  stage_b(G16_BK, 1, 0);
  asm volatile("s_waitcnt vmcnt(2)" ::: "memory");  // tile 0 landed
  __builtin_amdgcn_s_barrier();
  asm volatile("" ::: "memory");

  bf16x8 af[8];   // current A subtile: 4 mi x 2 kk
  bf16x8 b01[4];  // ni 0..1 x kk 0..1 (live the whole tile)
  bf16x8 b23[4];  // ni 2..3 x kk 0..1

  auto mfma_quad = [&](int mi0, int ni0, const bf16x8* a,
                       const bf16x8* b) {
    __builtin_amdgcn_s_setprio(1);
#pragma unroll
    for (int mi = 0; mi < 4; ++mi)
#pragma unroll
      for (int ni = 0; ni < 2; ++ni)
#pragma unroll
        for (int kk = 0; kk < 2; ++kk)
          acc[mi0 + mi][ni0 + ni] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              a[mi * 2 + kk], b[ni * 2 + kk], acc[mi0 + mi][ni0 + ni],
              0, 0, 0);
    __builtin_amdgcn_s_setprio(0);
  };
  auto rd_a = [&](const char* Ai, int mih) {
#pragma unroll
    for (int mi = 0; mi < 4; ++mi)
#pragma unroll
      for (int kk = 0; kk < 2; ++kk)
        af[mi * 2 + kk] = read_frag(Ai, mih * 4 + mi, kk);
  };
  auto rd_b = [&](const char* Bi, int nih, bf16x8* dst) {
#pragma unroll
    for (int ni = 0; ni < 2; ++ni)
#pragma unroll
      for (int kk = 0; kk < 2; ++kk)
        dst[ni * 2 + kk] = read_frag(Bi, br16 + nih * 2 + ni, kk);
  };

// one barrier per phase, placed between {reads+stage} and {MFMA}
#define G16_BAR()                                        \
  __builtin_amdgcn_s_barrier();                          \
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory")

  const char* A0c = (const char*)g16_img(0, 0, mw);  // wave's A half, buf0
  const char* B0c = (const char*)g16_img(1, 0, bh);
  const char* A1c = (const char*)g16_img(0, 1, mw);  // buf1
  const char* B1c = (const char*)g16_img(1, 1, bh);

  const int niters = nt / 2;
  for (int it = 0; it < niters; ++it) {
    const int t = 2 * it;  // first K-tile of the pair (buf 0)
    const long kT1 = (long)(t + 1) * G16_BK;
    const long kT2 = (long)(t + 2) * G16_BK;
    const long kT3 = (long)(t + 3) * G16_BK;
    const bool hT2 = t + 2 < nt, hT3 = t + 3 < nt;

    // ======== K-tile t (buf 0); zigzag q00->q01->q11->q10 ========
    // ph0: read A(mi0-3)+B(ni0-1); stage B1(t+1)+A0(t+1) -> buf1
    rd_a(A0c, 0);
    rd_b(B0c, 0, b01);
    stage_b(kT1, 1, 1);
    stage_a(kT1, 1, 0);
    G16_BAR();
    mfma_quad(0, 0, af, b01);

    // ph1: read B(ni2-3); stage A1(t+1) -> buf1
    rd_b(B0c, 1, b23);
    stage_a(kT1, 1, 1);
    G16_BAR();
    mfma_quad(0, 2, af, b23);

    // ph2: read A(mi4-7)
    rd_a(A0c, 1);
    G16_BAR();
    mfma_quad(4, 2, af, b23);

    // ph3: stage B0(t+2) -> buf0 (B(buf0) last read ph1: 2 bars ago);
    //      counted wait ensures tile t+1 fully landed for ph4
    if (hT2) stage_b(kT2, 0, 0);
    __builtin_amdgcn_s_barrier();
    mfma_quad(4, 0, af, b01);
    if (hT2)
      asm volatile("s_waitcnt vmcnt(2)" ::: "memory");
    else
      asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    asm volatile("" ::: "memory");
    __builtin_amdgcn_s_barrier();  // tile boundary (keeps ph4 reads
    asm volatile("" ::: "memory"); // behind every wave's ph3 MFMA srcs)

    // ======== K-tile t+1 (buf 1) ========
    // ph4: read A(mi0-3)+B(ni0-1); stage B1(t+2)+A0(t+2) -> buf0
    rd_a(A1c, 0);
    rd_b(B1c, 0, b01);
    if (hT2) {
      stage_b(kT2, 0, 1);
      stage_a(kT2, 0, 0);
    }
    G16_BAR();
    mfma_quad(0, 0, af, b01);

    // ph5: read B(ni2-3); stage A1(t+2) -> buf0
    rd_b(B1c, 1, b23);
    if (hT2) stage_a(kT2, 0, 1);
    G16_BAR();
    mfma_quad(0, 2, af, b23);

    // ph6: read A(mi4-7)
    rd_a(A1c, 1);
    G16_BAR();
    mfma_quad(4, 2, af, b23);

    // ph7: stage B0(t+3) -> buf1; counted wait for tile t+2
    if (hT3) stage_b(kT3, 1, 0);
    __builtin_amdgcn_s_barrier();
    mfma_quad(4, 0, af, b01);
    if (hT3)
      asm volatile("s_waitcnt vmcnt(2)" ::: "memory");
    else if (hT2)
      asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    asm volatile("" ::: "memory");
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
  }
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  __syncthreads();  // staging quiet before LDS becomes the slab
#undef G16_BAR
}
