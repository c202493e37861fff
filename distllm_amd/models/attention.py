"""Softmax attention on paged keys and values."""

from __future__ import annotations

import torch
from torch import nn

from .. import ops
from .blocks import (Branch, Part, head_pad, norm_weight, pad64, padded,
                     padded_heads, weight)
from .config import AttentionDims, RotaryAttentionDims


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


class RotaryAttention(Branch):
    """Causal attention with normed and rotated queries and keys, keys as
    projected for values and a sink per head (RotaryAttentionDims), on the
    pages of PagedAttention. One launch norms, rotates and writes the
    cache."""

    EVERYTHING = 1 << 30  # chunk size of plain causal attention

    def __init__(self, d: RotaryAttentionDims, width: int, eps: float,
                 dtype):
        super().__init__()
        self.d, self.width, self.eps = d, width, eps
        self.wp, self.dp = pad64(width), head_pad(d.dim)
        self.in_rows = (d.heads + d.kv_heads) * self.dp
        self.out_cols = d.heads * self.dp
        self.q_norm = norm_weight(self.dp)
        self.k_norm = norm_weight(self.dp)
        self.sink = norm_weight(d.heads)
        freq, self.rot_mult = d.rot.frequencies()
        self.rot_key = d.rot.model_dump_json()
        self.register_buffer("freq", torch.tensor(freq, dtype=torch.float64),
                             persistent=False)
        self.bf16 = dtype == torch.bfloat16

    def tensors(self):
        d, W = self.d, self.width
        q, k = d.heads * d.dim, d.kv_heads * d.dim
        return {"q": (q, W), "q.b": (q,), "q.norm": (d.dim,),
                "k": (k, W), "k.b": (k,), "k.norm": (d.dim,),
                "sink": (d.heads,), "o": (W, q), "o.b": (W,)}

    def _heads(self):
        return (("q", self.d.heads), ("k", self.d.kv_heads))

    def in_weight(self, t):
        return torch.cat([padded_heads(t[n], h, self.d.dim, self.dp, self.wp)
                          for n, h in self._heads()])

    def in_bias(self, t):
        return torch.cat([padded_heads(t[n + ".b"][:, None], h, self.d.dim,
                                       self.dp, 1)[:, 0]
                          for n, h in self._heads()])

    def out_weight(self, t):
        return padded_heads(t["o"].t(), self.d.heads, self.d.dim, self.dp,
                            self.wp).t()

    def out_bias(self, t):
        return t["o.b"]

    def extra(self, t):
        return {"q_norm": padded(t["q.norm"], self.dp),
                "k_norm": padded(t["k.norm"], self.dp), "sink": t["sink"]}

    def cache_numel(self):
        return 2 * self.d.kv_heads * self.dp

    def make_cache(self, num_blocks, blk, num_slots, dtype, device):
        G = self.d.kv_heads
        return (torch.zeros(num_blocks, G, blk, self.dp, dtype=dtype,
                            device=device),
                torch.zeros(num_blocks, G, self.dp, blk, dtype=dtype,
                            device=device))

    def run(self, ab, batch, pages, out, scale):
        d, M = self.d, ab.shape[0]
        kpages, vpages = pages
        table = batch.rotation(self.rot_key, self.freq, self.rot_mult)
        q = ops.rotary_prep(ab, d.heads, d.kv_heads, self.dp, d.dim,
                            self.q_norm, self.k_norm, self.eps, table, pages,
                            batch.block_table, batch.row_seq, batch.ctx)
        flash = self.dp <= 256 and (self.bf16 or not ab.is_cuda)
        n = batch.n_folded if flash else M
        if n > 0:
            ops.sink_attn_rows(q[:n], kpages, vpages, out[:n],
                               batch.block_table, batch.row_seq[:n],
                               batch.ctx[:n], d.scale, self.sink, scale)
        if n < M:
            ops.sink_attn_prompts(
                q, kpages, vpages, out, batch.block_table,
                batch.prompt_blocks(self.EVERYTHING), d.scale, self.sink,
                scale)
