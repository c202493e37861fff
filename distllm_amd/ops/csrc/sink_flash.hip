// Prompt portions of plain causal attention with a sink per head.
#include "attention_flash.h"

extern "C" void launch_sink_flash(
    const void* Q, const void* kpages, const void* vpages, void* O,
    long ld_out, const int* block_table, int max_blocks, const int* portions,
    const int* blocks, int nblocks, int H, int G, int DK, int DV, float scale,
    const float* sink, float out_scale, hipStream_t stream) {
  launch_attention_flash(SinkScore{scale, scale * LOG2E, sink, out_scale}, Q,
                         kpages, vpages, O, ld_out, block_table, max_blocks,
                         portions, blocks, nblocks, H, G, DK, DV, 1 << 30,
                         stream);
}
