// Shared by the bindings of attention over paged keys and values: checks of
// pages and rows, launch shapes.
#pragma once

#include "ext_common.h"

struct Pages {
  int nblk, G, DK, DV;
};

static inline Pages check_pages(const torch::Tensor& k, const torch::Tensor& v) {
  CHECK_DEV(k); CHECK_CONT(k); CHECK_T(k);
  CHECK_DEV(v); CHECK_CONT(v); CHECK_SAME(k, v);
  TORCH_CHECK(k.dim() == 4 && v.dim() == 4 && k.size(2) == 16 &&
                  v.size(3) == 16 && k.size(0) == v.size(0) &&
                  k.size(1) == v.size(1),
              "pages must be [blocks, heads, 16, dim], [blocks, heads, "
              "vdim, 16]");
  TORCH_CHECK(k.size(3) % 64 == 0 && v.size(2) % 64 == 0,
              "head sizes % 64");
  return {(int)k.size(0), (int)k.size(1), (int)k.size(3), (int)v.size(2)};
}

static inline void check_rows(const torch::Tensor& bt, const torch::Tensor& row_seq,
                       const torch::Tensor& ctx, long M) {
  CHECK_INTS(bt); CHECK_INTS(row_seq); CHECK_INTS(ctx);
  TORCH_CHECK(bt.dim() == 2 && row_seq.numel() == M && ctx.numel() == M,
              "one row_seq and ctx entry per row");
}

// Split each row's keys until the CUs are full (four workgroups each), as
// long as a wave keeps two tiles. All sizes are known on the host, so a
// captured graph stays valid as contexts grow.
static inline long key_splits(long nsplit, long M, long H, long G, long chunk,
                       long max_blocks) {
  if (nsplit <= 0) {
    const long wgs = M * G * ((H / G + 15) / 16);
    const long tiles = std::min<long>(chunk, max_blocks * 16L) / 32 + 1;
    nsplit = std::min<long>({(1024 + wgs - 1) / wgs, tiles / 8, 64L});
  }
  return std::max<long>(nsplit, 1);
}

static inline bool mfma_size(int d) { return d == 64 || d == 128 || d == 256; }
