// Launcher of the flash-attention forward kernel for packed continuations
// of cached prompts: causal, sliding window, separate key and value head
// sizes, one key/value pair per query head, optionally with key numbers that
// all heads share, sinks and gates.
#include "attention_kernel.h"

extern "C" void launch_attn_window(
    const void* Q, const void* K, const void* V, const void* Kr, void* O,
    const int* cu_q, const int* cu_k, const int* blk_seq, const int* blk_qb,
    int nblocks, int B, int H, int DK, int DV, long tstr_q, long tstr_kv,
    int window, float scale, const float* sink, const void* gate, int ld_gate,
    hipStream_t stream) {
  const int nwave = 4;
  const int rot = Kr != nullptr ? 64 : 0;
  const int ktile = KVBLK * (DK + rot) * 2, vtile = DV * KVBLK * 2;
  const int stage_b = 2 * ktile + 2 * vtile;
  const int epi_b = nwave * QWAVE * (DV + 1) * 4;
  const int lds = stage_b > epi_b ? stage_b : epi_b;
#define AWN(KK, VV, RO)                                                       \
  hipLaunchKernelGGL(                                                         \
      (attn_fwd_kernel<KK, true, false, false, true, VV, true, RO>),          \
      dim3(nblocks * H), dim3(nwave * 64), lds, stream,                       \
      (const unsigned short*)Q, (const unsigned short*)K,                     \
      (const unsigned short*)V, (const float*)nullptr, (unsigned short*)O, B, \
      0, 0, H, H, scale, 0L, tstr_q, 0L, tstr_kv, cu_q, blk_seq, blk_qb,      \
      cu_k, window, (const unsigned short*)Kr, sink,                          \
      (const unsigned short*)gate, ld_gate)
#define AWN_R(KK, VV)           \
  do {                          \
    if (rot) AWN(KK, VV, 64);   \
    else AWN(KK, VV, 0);        \
  } while (0)
#define AWN_V(KK)                 \
  do {                            \
    if (DV == 64) AWN_R(KK, 64);  \
    else if (DV == 128) AWN_R(KK, 128); \
    else AWN_R(KK, 256);          \
  } while (0)
  if (DK == 64) AWN_V(64);
  else if (DK == 128) AWN_V(128);
  else AWN_V(256);
#undef AWN_V
#undef AWN_R
#undef AWN
}
