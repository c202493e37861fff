// Single-token rows with capped scores and a distance bias.
#include "attention_rows.h"

static CappedScore capped(float scale, float softcap, const float* dist,
                          const void* gate, int ld_gate) {
  return {scale, softcap, 2.f * scale / softcap * LOG2E, softcap * LOG2E,
          dist, gate, ld_gate};
}

extern "C" void launch_chunk_rows(const void* q, const void* kpages,
                                  const void* vpages, const void* gate,
                                  int ld_gate, const int* block_table,
                                  const int* row_seq, const int* ctx,
                                  void* out, int M, int H, int G, int DK,
                                  int DV, int max_blocks, int chunk,
                                  float scale, float softcap,
                                  const float* dist, bool fp32,
                                  hipStream_t stream) {
  launch_attention_rows(capped(scale, softcap, dist, gate, ld_gate), q,
                        kpages, vpages, block_table, row_seq, ctx, out,
                        (long)H * DV, M, H, G, DK, DV, max_blocks, chunk,
                        fp32, stream);
}

extern "C" void launch_chunk_decode(
    const void* q, const void* kpages, const void* vpages, const void* gate,
    int ld_gate, const int* block_table, const int* row_seq, const int* ctx,
    void* out, void* pacc, void* pml, int M, int H, int G, int DK, int DV,
    int NS, int max_blocks, int chunk, float scale, float softcap,
    const float* dist, hipStream_t stream) {
  launch_attention_decode(capped(scale, softcap, dist, gate, ld_gate), q,
                          kpages, vpages, block_table, row_seq, ctx, out,
                          (long)H * DV, pacc, pml, M, H, G, DK, DV, NS,
                          max_blocks, chunk, stream);
}
