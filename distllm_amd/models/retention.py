"""Retention: linear attention with a fixed decay per head."""

from __future__ import annotations

import torch

from .. import ops
from .blocks import Part, head_pad, pad64, padded_heads, weight
from .config import RetentionDims


class Retention(Part):
    """S <- decay S + k v^T; o = S^T q per head, with rotated queries and
    keys, outputs normed per head and gated by silu (RetentionDims). One
    product yields queries, keys, values and gates; the rest up to the
    output product is one launch for short segments of a step and one or
    three for long ones.

    A slot of the state is kept transposed, [heads, vdim, dim], so that
    what one value column needs is contiguous."""

    def __init__(self, d: RetentionDims, width: int, eps: float, dtype):
        super().__init__()
        self.d, self.width, self.eps = d, width, eps
        self.wp = pad64(width)
        self.dp, self.vp = head_pad(d.dim), head_pad(d.vdim)
        H = d.heads
        self.win = weight(2 * H * (self.dp + self.vp), self.wp, dtype)
        self.wo = weight(self.wp, H * self.vp, dtype)
        freq, self.rot_mult = d.rot.frequencies()
        self.rot_key = d.rot.model_dump_json()
        self.register_buffer("freq", torch.tensor(freq, dtype=torch.float64),
                             persistent=False)
        # decays, and their base-2 logarithms, per head
        g = torch.tensor(d.decay, dtype=torch.float64)
        self.register_buffer("decay", torch.stack([g, g.log2()]).float(),
                             persistent=False)

    def tensors(self):
        d, W = self.d, self.width
        qk, v = d.heads * d.dim, d.heads * d.vdim
        return {"q": (qk, W), "k": (qk, W), "v": (v, W), "g": (v, W),
                "o": (W, v)}

    def checkpoint(self, src, pre):
        d = self.d
        t = self.checked(src, pre)
        sizes = {"q": (d.dim, self.dp), "k": (d.dim, self.dp),
                 "v": (d.vdim, self.vp), "g": (d.vdim, self.vp)}
        return {"win": torch.cat([padded_heads(t[n], d.heads, a, b, self.wp)
                                  for n, (a, b) in sizes.items()]),
                "wo": padded_heads(t["o"].t(), d.heads, d.vdim, self.vp,
                                   self.wp).t()}

    def state_numel(self):
        return self.d.heads * self.vp * self.dp, 0

    def make_cache(self, num_blocks, blk, num_slots, dtype, device):
        return torch.zeros(num_slots, self.d.heads, self.vp, self.dp,
                           dtype=torch.float32, device=device)

    def forward(self, h, batch, state):
        d = self.d
        ab = ops.linear(h, self.win)
        table = batch.rotation(self.rot_key, self.freq, self.rot_mult)
        y = ops.retention(ab, d.heads, self.dp, self.vp, d.dim, d.vdim,
                          self.decay, table, self.eps, state, batch.segments,
                          batch.ctx)
        return ops.linear(y, self.wo)
