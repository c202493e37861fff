"""Latent attention with rotated key parts, sinks and head gates."""

from __future__ import annotations

import torch

from .. import ops
from .blocks import (LatentAttention, Part, head_pad, norm_weight, pad64,
                     padded, padded_heads, rank_pad, weight)
from .config import RotaryLatentDims


class RotaryLatentAttention(LatentAttention):
    """Causal latent attention whose scores also have a rotated part, with
    keys that all heads share, a sink per head in the softmax and a gate per
    head on the output (RotaryLatentDims). A token's cache row is its latent
    followed by its rotated key part; the two forms are those of
    LatentAttention.

    One product yields everything that reads the mixer's input: queries
    (per head its unrotated numbers, then the rotated ones), latent, key
    part, gates. One launch norms, rotates and writes the cache.
    """

    EVERYTHING = 1 << 30  # window of plain causal attention

    def __init__(self, d: RotaryLatentDims, width: int, eps: float, dtype):
        Part.__init__(self)
        self.d, self.width, self.eps = d, width, eps
        self.wp = pad64(width)
        self.dp, self.vp = head_pad(d.dim), head_pad(d.vdim)
        self.rp, self.tp = rank_pad(d.kv_rank), pad64(d.rot_dim)
        self.own = d.kv_from is None
        H = d.heads
        self.q_cols = H * (self.dp + self.tp)
        self.gate_at = self.q_cols + (self.rp + self.tp if self.own else 0)
        self.win = weight(self.gate_at + pad64(H), self.wp, dtype)
        self.kv_norm = norm_weight(self.rp) if self.own else None
        # all heads' key rows, then all heads' value rows
        self.wukv = weight(H * (self.dp + self.vp), self.rp, dtype)
        self.wo = weight(self.wp, H * self.vp, dtype)
        self.sink = norm_weight(H)
        freq, self.rot_mult = d.rot.frequencies()
        self.rot_key = d.rot.model_dump_json()
        self.register_buffer("freq", torch.tensor(freq, dtype=torch.float64),
                             persistent=False)
        self._fold: tuple | None = None

    def tensors(self):
        d, H, W = self.d, self.d.heads, self.width
        t = {"q": (H * (d.dim + d.rot_dim), W)}
        if self.own:
            t |= {"dkv": (d.kv_rank + d.rot_dim, W),
                  "dkv.norm": (d.kv_rank,)}
        return t | {"uk": (H * d.dim, d.kv_rank),
                    "uv": (H * d.vdim, d.kv_rank), "sink": (H,),
                    "g": (H, W), "o": (W, H * d.vdim)}

    def checkpoint(self, src, pre):
        d, H = self.d, self.d.heads
        t = self.checked(src, pre)
        q = t["q"].view(H, d.dim + d.rot_dim, self.width)
        rows = [torch.cat([
            padded(q[:, : d.dim], H, self.dp, self.wp),
            padded(q[:, d.dim:], H, self.tp, self.wp)], 1).flatten(0, 1)]
        out = {}
        if self.own:
            rows += [padded(t["dkv"][: d.kv_rank], self.rp, self.wp),
                     padded(t["dkv"][d.kv_rank:], self.tp, self.wp)]
            out["kv_norm"] = padded(t["dkv.norm"], self.rp)
        rows.append(padded(t["g"], pad64(H), self.wp))
        return out | {
            "win": torch.cat(rows), "sink": t["sink"],
            "wukv": torch.cat([
                padded_heads(t["uk"], H, d.dim, self.dp, self.rp),
                padded_heads(t["uv"], H, d.vdim, self.vp, self.rp)]),
            "wo": padded_heads(t["o"].t(), H, d.vdim, self.vp, self.wp).t()}

    def cache_numel(self):
        return self.rp + self.tp if self.own else 0

    def make_cache(self, num_blocks, blk, num_slots, dtype, device):
        """Paged rows [blocks, BLK, latent | rotated key part]."""
        return torch.zeros(num_blocks, blk, self.rp + self.tp, dtype=dtype,
                           device=device)

    def expands(self) -> bool:
        """Whether the flash kernel covers this layer's dtype and sizes."""
        w = self.wo
        return (max(self.dp, self.vp) <= 256 and self.tp == 64
                and (w.dtype == torch.bfloat16 or not w.is_cuda))

    def forward(self, h, batch, rows):
        """h [M, width]; rows: the paged cache of the layer that owns it."""
        d, H = self.d, self.d.heads
        M = h.shape[0]
        bt, ctx = batch.block_table, batch.ctx
        ab = ops.linear(h, self.win)
        # leading rows folded, then the rows of expanded portions
        n = batch.n_folded if self.expands() else M
        ql = h.new_empty(n, H, self.rp + self.tp)
        table = batch.rotation(self.rot_key, self.freq, self.rot_mult)
        ops.rotary_latent_prep(ab, H, self.dp, self.tp, d.kv_rank,
                               self.kv_norm, self.eps, table,
                               rows if self.own else None, bt, batch.row_seq,
                               ctx, ql)
        q = ab[:, : self.q_cols].view(M, H, self.dp + self.tp)
        gate = ab[:, self.gate_at: self.gate_at + H]
        o = (h.new_empty if n == M else h.new_zeros)(M, H, self.vp)
        if n > 0:
            uk_t, uv = self._folded()
            ops.head_gemm(q[:n, :, : self.dp], uk_t, out=ql[..., : self.rp])
            ol = ops.latent_attn(ql, rows, bt, batch.row_seq[:n], ctx[:n],
                                 self.EVERYTHING, d.scale, rank=self.rp,
                                 sink=self.sink, gate=gate[:n])
            ops.head_gemm(ol, uv, out=o[:n])
        if n < M:
            e = batch.expansion(self.EVERYTHING)
            c, kr = ops.latent_gather(rows, bt, e.key_seq, e.key_pos,
                                      self.rp)
            kv = ops.linear(c, self.wukv)
            ops.attn_window(q[n:], kv, o[n:], e.cu_q, e.cu_k, e.block_map,
                            self.EVERYTHING, d.scale, kr=kr, sink=self.sink,
                            gate=gate[n:])
        return ops.linear(o.view(M, H * self.vp), self.wo)
