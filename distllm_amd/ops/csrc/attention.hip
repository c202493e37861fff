// Launchers of the flash-attention forward kernel for the padded and the
// packed bidirectional / causal geometries; attention_kernel.h has the
// kernel and its design notes.
#include "attention_kernel.h"

extern "C" void launch_attn_fwd(const void* Q, const void* K, const void* V,
                                const float* mask, void* O, int B, int SQ,
                                int SKV, int H, int HKV, int D, bool causal,
                                float scale, long bstr_q, long tstr_q,
                                long bstr_k, long tstr_k,
                                hipStream_t stream) {
  const int nwave = 4;
  const int qblk = nwave * 32;
  const int nqb = (SQ + qblk - 1) / qblk;
  const int grid = B * H * nqb;
  const int ktile = KVBLK * D * 2, vtile = D * VROW * 2;
  const int stage_b = 2 * ktile + 2 * vtile + 2 * KVBLK * 4;
  const int epi_b = nwave * 32 * (D + 1) * 4;
  const int lds = stage_b > epi_b ? stage_b : epi_b;

  // measured on MI355X: LDS-staged V wins at D=64 (330 vs 302 TF),
  // direct-global V wins at D=128 (176 vs 105 TF — drops the VGPR
  // pressure that pinned the kernel at 1 wave/SIMD). Env-overridable.
  static int vdirect = -1;
  if (vdirect < 0) {
    const char* e = getenv("DISTLLM_ATTN_VDIRECT");
    vdirect = e ? (e[0] == '1' ? 1 : 0) : -1;
  }
  const int vd = (vdirect >= 0) ? vdirect : (D == 128 ? 1 : 0);
#define ATTN_DISPATCH(DD, CC, MM)                                              \
  do {                                                                         \
    if (vd)                                                               \
      hipLaunchKernelGGL((attn_fwd_kernel<DD, CC, MM, true>), dim3(grid),      \
                         dim3(nwave * 64), lds, stream,                        \
                         (const unsigned short*)Q, (const unsigned short*)K,   \
                         (const unsigned short*)V, mask, (unsigned short*)O,   \
                         B, SQ, SKV, H, HKV, scale, bstr_q, tstr_q, bstr_k,    \
                         tstr_k);                                              \
    else                                                                       \
      hipLaunchKernelGGL((attn_fwd_kernel<DD, CC, MM, false>), dim3(grid),     \
                         dim3(nwave * 64), lds, stream,                        \
                         (const unsigned short*)Q, (const unsigned short*)K,   \
                         (const unsigned short*)V, mask, (unsigned short*)O,   \
                         B, SQ, SKV, H, HKV, scale, bstr_q, tstr_q, bstr_k,    \
                         tstr_k);                                              \
  } while (0)
  const bool hm = mask != nullptr;
  if (D == 64) {
    if (causal && hm) ATTN_DISPATCH(64, true, true);
    else if (causal) ATTN_DISPATCH(64, true, false);
    else if (hm) ATTN_DISPATCH(64, false, true);
    else ATTN_DISPATCH(64, false, false);
  } else if (D == 128) {
    if (causal && hm) ATTN_DISPATCH(128, true, true);
    else if (causal) ATTN_DISPATCH(128, true, false);
    else if (hm) ATTN_DISPATCH(128, false, true);
    else ATTN_DISPATCH(128, false, false);
  }
#undef ATTN_DISPATCH
}

extern "C" void launch_attn_varlen(const void* Q, const void* K,
                                   const void* V, void* O, const int* cu,
                                   const int* blk_seq, const int* blk_qb,
                                   int nblocks, int B, int H, int HKV,
                                   int D, float scale,
                                   hipStream_t stream) {
  const int nwave = 4;
  const int grid = nblocks * H;
  const int ktile = KVBLK * D * 2, vtile = D * VROW * 2;
  const int stage_b = 2 * ktile + 2 * vtile + 2 * KVBLK * 4;
  const int epi_b = nwave * 32 * (D + 1) * 4;
  const int lds = stage_b > epi_b ? stage_b : epi_b;
  const long tq = (long)H * D, tk = (long)HKV * D;
  static int vdirect = -1;
  if (vdirect < 0) {
    const char* e = getenv("DISTLLM_ATTN_VDIRECT");
    vdirect = e ? (e[0] == '1' ? 1 : 0) : -1;
  }
  const int vd = (vdirect >= 0) ? vdirect : (D == 128 ? 1 : 0);
#define AVL(DD, VD)                                                           \
  hipLaunchKernelGGL((attn_fwd_kernel<DD, false, false, VD, true>),           \
                     dim3(grid), dim3(nwave * 64), lds, stream,               \
                     (const unsigned short*)Q, (const unsigned short*)K,      \
                     (const unsigned short*)V, (const float*)nullptr,         \
                     (unsigned short*)O, B, 0, 0, H, HKV, scale, 0L, tq,      \
                     0L, tk, cu, blk_seq, blk_qb)
  if (D == 64) { if (vd) AVL(64, true); else AVL(64, false); }
  else if (D == 128) { if (vd) AVL(128, true); else AVL(128, false); }
#undef AVL
}
