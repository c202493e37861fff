// Single-token rows of plain causal attention with a sink per head.
#include "attention_rows.h"

extern "C" void launch_sink_rows(const void* q, const void* kpages,
                                 const void* vpages, const int* block_table,
                                 const int* row_seq, const int* ctx,
                                 void* out, long ld_out, int M, int H, int G,
                                 int DK, int DV, int max_blocks, float scale,
                                 const float* sink, float out_scale,
                                 bool fp32, hipStream_t stream) {
  launch_attention_rows(SinkScore{scale, scale * LOG2E, sink, out_scale}, q,
                        kpages, vpages, block_table, row_seq, ctx, out,
                        ld_out, M, H, G, DK, DV, max_blocks, 1 << 30, fp32,
                        stream);
}

extern "C" void launch_sink_decode(
    const void* q, const void* kpages, const void* vpages,
    const int* block_table, const int* row_seq, const int* ctx, void* out,
    long ld_out, void* pacc, void* pml, int M, int H, int G, int DK, int DV,
    int NS, int max_blocks, float scale, const float* sink, float out_scale,
    hipStream_t stream) {
  launch_attention_decode(SinkScore{scale, scale * LOG2E, sink, out_scale},
                          q, kpages, vpages, block_table, row_seq, ctx, out,
                          ld_out, pacc, pml, M, H, G, DK, DV, NS, max_blocks,
                          1 << 30, stream);
}
