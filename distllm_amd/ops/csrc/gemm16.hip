// 8-phase deep-pipelined CDNA4 MFMA GEMM: C[M,N] = A[M,K] @ B[N,K]^T
// (+fused bias/activation). The gemm8.hip successor targeting the
// K-shallow flagship encoder shapes (M=262144, N in {768,2304,3072},
// K in {768,3072}) where hipBLASLt previously owned ~52% of the
// flagship step (reference anchor: the delegated projection GEMMs of
// distllm/embed/encoders/auto.py:116-138).
//
// Structure per the guide's 256^2 8-phase template
// (cdna_hip_programming.md §5 "The 256² 8-phase template"), own
// implementation and schedule:
//   - 256x256x64 tile, 512 threads = 8 waves as 2(M) x 4(N); per-wave
//     output 128x64 (8 mi x 4 ni fragments of mfma_f32_16x16x32_bf16).
//   - one iteration consumes TWO K-tiles (8 phases); ZIGZAG quadrant
//     order {q(mi0-3,ni01), q(mi0-3,ni23), q(mi4-7,ni23),
//     q(mi4-7,ni01)}: at most one A-subtile (32 VGPR) plus both
//     B-subtiles (32) live at once -> no spills at 2 waves/SIMD.
//   - ONE barrier per phase: {ds_read subtile; glds stage;
//     s_barrier; lgkmcnt(0); s_setprio(1); 16 MFMA; s_setprio(0)}.
//     PMC on the two-barrier variant showed 37% of wave cycles parked
//     (SQ_WAIT_ANY); the post-MFMA barrier is dropped by DEFERRING
//     every stage slot to >= 2 barriers after its target image's last
//     read: any wave issuing the stage has passed BAR(p-1), and every
//     wave's reads from 2+ phases ago completed before its own
//     lgkmcnt(0)+MFMA which precede BAR(p-1) — placement-independent.
//   - stage slots (tile pair t,t+1 consuming bufs 0,1):
//       ph0: B1(t+1)+A0(t+1) -> buf1   ph1: A1(t+1) -> buf1
//       ph3: B0(t+2) -> buf0           ph4: B1(t+2)+A0(t+2) -> buf0
//       ph5: A1(t+2) -> buf0           ph7: B0(t+3) -> buf1
//     counted s_waitcnt vmcnt(2) ONCE per K-tile (end of ph3 and ph7)
//     leaves exactly the newest half-tile in flight (T3+T4).
//   - XOR swizzle (chunk ^ (row&7)) on the glds SOURCE address and the
//     ds_read offset (guide rule 21 / T2).
//   - T1 bijective XCD swizzle, tm-major so the N-tiles sharing an
//     A-panel land on one XCD's L2.
//   - epilogue: per-wave padded-LDS transpose rounds (wave-local
//     lgkmcnt ordering, no workgroup barriers); each lane packs 8 f32
//     into ONE 16-byte dwordx4 store per row pass (T21), bias +
//     branch-free GELU/SiLU fused.
// Requires M%256==0, N%256==0, K%128==0 (host falls back otherwise).
#include "gemm16_core.h"

enum G16Act { G16_NONE = 0, G16_GELU_TANH = 1, G16_GELU_ERF = 2,
              G16_SILU = 3 };

template <int ACT, bool HAS_BIAS>
__global__ void __launch_bounds__(512, 2)
gemm16_kernel(const unsigned short* __restrict__ A,
              const unsigned short* __restrict__ B,
              const unsigned short* __restrict__ bias,
              unsigned short* __restrict__ C, int M, int N, int K) {
  const int lane = threadIdx.x & 63;
  const int wid = threadIdx.x >> 6;  // 0..7
  const int mw = wid >> 2;           // M half (0/1): rows mw*128..+127
  const int nw = wid & 3;            // N quarter: cols nw*64..+63

  // T1 bijective XCD swizzle (tm-major tile order underneath)
  const int ntm = M / G16_BM, ntn = N / G16_BN;
  const int nwg = ntm * ntn;
  int bid = blockIdx.x;
  {
    const int q = nwg / 8, r = nwg % 8;
    const int xcd = bid % 8, j = bid / 8;
    bid = (xcd < r ? xcd * (q + 1) : r * (q + 1) + (xcd - r) * q) + j;
  }
  const int tm = bid / ntn, tn = bid % ntn;

  const unsigned short* Atile = A + (long)tm * G16_BM * K;
  const unsigned short* Btile = B + (long)tn * G16_BN * K;

  const int r_in = lane >> 3;   // 0..7 within the 8-row piece
  const int c_dst = lane & 7;   // 16B chunk within the row
  auto stage = [&](const unsigned short* G, long k0, int op, int buf,
                   int half) {
#pragma unroll
    for (int pp = 0; pp < 2; ++pp) {
      const int row = (wid * 2 + pp) * 8 + r_in;
      const int c_src = c_dst ^ (row & 7);
      g16_stage(G + (long)(half * 128 + row) * K + k0 + c_src * 8, op, buf,
                half, pp, wid, lane);
    }
  };
  f32x4 acc[8][4];
  g16_mainloop(
      [&](long k0, int buf, int half) { stage(Atile, k0, 0, buf, half); },
      [&](long k0, int buf, int half) { stage(Btile, k0, 1, buf, half); }, K,
      lane, mw, nw, acc);

  // ---- epilogue: per-wave transpose slab, one 16-row round per mi
  // fragment; wave-local lgkmcnt ordering only; each lane emits one
  // dwordx4 store per row pass (T21) -------------------------------
  {
    constexpr int SLAB_W = 68;  // 64 + 4 f32 pad
    float* slab = reinterpret_cast<float*>(smem16) + wid * 16 * SLAB_W;
    const int grow0 = tm * G16_BM + mw * 128;
    const int gcol0 = tn * G16_BN + nw * 64;
    const int c8 = lane & 7;
    const int pr = lane >> 3;

    float bv[8];
    if (HAS_BIAS) {
      const s16x8 raw =
          *reinterpret_cast<const s16x8*>(bias + gcol0 + c8 * 8);
      bf8_to_f32(raw, bv);
    }

#pragma unroll
    for (int rd = 0; rd < 8; ++rd) {  // one 16-row mi fragment each
#pragma unroll
      for (int ni = 0; ni < 4; ++ni) {
        const f32x4 v = acc[rd][ni];
        const int col = ni * 16 + (lane & 15);
        const int row0 = (lane >> 4) * 4;
#pragma unroll
        for (int r = 0; r < 4; ++r)
          slab[(row0 + r) * SLAB_W + col] = v[r];
      }
      asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
#pragma unroll
      for (int p = 0; p < 2; ++p) {
        const int r = p * 8 + pr;
        unsigned short o[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          float x = slab[r * SLAB_W + c8 * 8 + e];
          if (HAS_BIAS) x += bv[e];
          if (ACT == G16_GELU_TANH) x = fast_gelu(x);
          else if (ACT == G16_GELU_ERF) x = gelu_erf(x);
          else if (ACT == G16_SILU) x = silu(x);
          o[e] = f2bf(x);
        }
        *reinterpret_cast<i32x4*>(
            C + (long)(grow0 + rd * 16 + r) * N + gcol0 + c8 * 8) =
            *reinterpret_cast<const i32x4*>(o);
      }
      asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    }
  }
}

extern "C" void launch_gemm16_bf16(const void* A, const void* B,
                                   const void* bias, void* C, int M, int N,
                                   int K, int act, hipStream_t stream) {
  const int nwg = (M / G16_BM) * (N / G16_BN);
#define G16D(ACT, HB)                                                         \
  hipLaunchKernelGGL((gemm16_kernel<ACT, HB>), dim3(nwg), dim3(512),          \
                     G16_LDS, stream, (const unsigned short*)A,               \
                     (const unsigned short*)B, (const unsigned short*)bias,   \
                     (unsigned short*)C, M, N, K)
  const bool hb = bias != nullptr;
  switch (act) {
    case G16_GELU_TANH: if (hb) G16D(1, true); else G16D(1, false); break;
    case G16_GELU_ERF: if (hb) G16D(2, true); else G16D(2, false); break;
    case G16_SILU: if (hb) G16D(3, true); else G16D(3, false); break;
    default: if (hb) G16D(0, true); else G16D(0, false); break;
  }
#undef G16D
}
