"""Softmax attention on paged keys and values, visible chunk by chunk."""

from __future__ import annotations

import torch
from torch import nn

from .. import ops
from .blocks import (Part, head_pad, norm_weight, pad64, padded,
                     padded_heads, weight)
from .config import AttentionDims


class PagedAttention(Part):
    """Normed queries and keys, capped scores with a distance bias, gated
    heads (AttentionDims). One product yields queries, keys, values and
    gates; one launch norms them and writes the cache; short portions and
    decoded tokens are attended row by row, longer portions by the flash
    kernel, both straight from the pages.

    Key pages are [blocks, heads, BLK, dim]; value pages are transposed,
    [blocks, heads, vdim, BLK], which is the operand order of the
    weights-times-values product.
    """

    def __init__(self, d: AttentionDims, width: int, eps: float, dtype):
        super().__init__()
        self.d, self.width, self.eps = d, width, eps
        self.wp = pad64(width)
        self.dp, self.vp = head_pad(d.dim), head_pad(d.vdim)
        self.own = d.kv_from is None
        # columns of the projection: queries, keys, values, gates
        kv = d.kv_heads * (self.dp + self.vp) if self.own else 0
        self.gate_at = d.heads * self.dp + kv
        n = pad64(self.gate_at + d.heads * self.vp)
        self.wqkvg = weight(n, self.wp, dtype)
        self.bias = nn.Parameter(torch.empty(n, dtype=dtype))
        self.q_norm = norm_weight(self.dp)
        self.k_norm = norm_weight(self.dp) if self.own else None
        # distance bias: r1, then r2, per head
        self.dist = nn.Parameter(torch.empty(2, d.heads,
                                             dtype=torch.float32))
        self.wo = weight(self.wp, d.heads * self.vp, dtype)

    @property
    def kv_from(self):
        return self.d.kv_from

    def tensors(self):
        d, W = self.d, self.width
        t = {"q": (d.heads * d.dim, W), "q.b": (d.heads * d.dim,),
             "q.norm": (d.dim,)}
        if self.own:
            t |= {"k": (d.kv_heads * d.dim, W),
                  "k.b": (d.kv_heads * d.dim,), "k.norm": (d.dim,),
                  "v": (d.kv_heads * d.vdim, W),
                  "v.b": (d.kv_heads * d.vdim,)}
        return t | {"r1": (d.heads,), "r2": (d.heads,),
                    "g": (d.heads * d.vdim, W), "o": (W, d.heads * d.vdim)}

    def checkpoint(self, src, pre):
        d = self.d
        t = self.checked(src, pre)
        parts = [("q", d.heads, d.dim, self.dp)]
        if self.own:
            parts += [("k", d.kv_heads, d.dim, self.dp),
                      ("v", d.kv_heads, d.vdim, self.vp)]
        parts.append(("g", d.heads, d.vdim, self.vp))
        w = torch.cat([padded_heads(t[n], h, a, b, self.wp)
                       for n, h, a, b in parts])
        bias = torch.cat([padded_heads(t[n + ".b"][:, None], h, a, b, 1)[:, 0]
                          if n != "g" else w.new_zeros(h * b)
                          for n, h, a, b in parts])
        out = {"wqkvg": padded(w, *self.wqkvg.shape),
               "bias": padded(bias, *self.bias.shape),
               "q_norm": padded(t["q.norm"], self.dp),
               "dist": torch.stack([t["r1"], t["r2"]]),
               "wo": padded_heads(t["o"].t(), d.heads, d.vdim, self.vp,
                                  self.wp).t()}
        if self.own:
            out["k_norm"] = padded(t["k.norm"], self.dp)
        return out

    def cache_numel(self):
        return self.d.kv_heads * (self.dp + self.vp) if self.own else 0

    def make_cache(self, num_blocks, blk, num_slots, dtype, device):
        G = self.d.kv_heads
        return (torch.zeros(num_blocks, G, blk, self.dp, dtype=dtype,
                            device=device),
                torch.zeros(num_blocks, G, self.vp, blk, dtype=dtype,
                            device=device))

    def expands(self) -> bool:
        """Whether the flash kernel covers this layer's dtype and sizes."""
        w = self.wo
        return (max(self.dp, self.vp) <= 256
                and (w.dtype == torch.bfloat16 or not w.is_cuda))

    def forward(self, h, batch, pages):
        d, M = self.d, h.shape[0]
        kpages, vpages = pages
        ab = ops.linear(h, self.wqkvg, self.bias)
        q = ops.attn_prep(ab, d.heads, d.kv_heads, self.dp, self.vp, d.dim,
                          self.q_norm, self.k_norm, self.eps,
                          pages if self.own else None, batch.block_table,
                          batch.row_seq, batch.ctx)
        n = batch.n_folded if self.expands() else M
        o = h.new_empty(M, d.heads, self.vp)
        if n > 0:
            ops.paged_attn_rows(
                q[:n], kpages, vpages, ab[:n], self.gate_at, o[:n],
                batch.block_table, batch.row_seq[:n], batch.ctx[:n],
                d.chunk, d.scale, d.softcap, self.dist)
        if n < M:
            ops.paged_attn_prompts(
                q, kpages, vpages, ab, self.gate_at, o, batch.block_table,
                batch.prompt_blocks(d.chunk), d.chunk, d.scale, d.softcap,
                self.dist)
        return ops.linear(o.view(M, d.heads * self.vp), self.wo)
