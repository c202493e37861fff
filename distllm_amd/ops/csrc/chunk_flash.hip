// Prompt portions with capped scores and a distance bias.
#include "attention_flash.h"

extern "C" void launch_chunk_flash(
    const void* Q, const void* kpages, const void* vpages, const void* gate,
    int ld_gate, void* O, const int* block_table, int max_blocks,
    const int* portions, const int* blocks, int nblocks, int H, int G, int DK,
    int DV, int chunk, float scale, float softcap, const float* dist,
    hipStream_t stream) {
  const CappedScore p{scale, softcap, 2.f * scale / softcap * LOG2E,
                      softcap * LOG2E, dist, gate, ld_gate};
  launch_attention_flash(p, Q, kpages, vpages, O, (long)H * DV, block_table,
                         max_blocks, portions, blocks, nblocks, H, G, DK, DV,
                         chunk, stream);
}
