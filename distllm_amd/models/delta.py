"""Gated delta rules with short convolutions."""

from __future__ import annotations

import torch
from torch import nn

from .. import ops
from .blocks import (Branch, Part, norm_weight, pad64, padded, padded_heads,
                     weight)
from .config import ChannelDeltaDims, DeltaDims


def state_pad(n: int) -> int:
    """Head sizes of the state kernels: 64, 128, 256."""
    for p in (64, 128, 256):
        if n <= p:
            return p
    raise ValueError(f"delta-rule heads of {n} numbers; at most 256")


class DeltaState:
    """Slots of one layer: the fp32 state, transposed to [slots, heads,
    vdim, dim] so that what one value column needs is contiguous, and the
    convolutions' last inputs [slots, taps - 1, channels]."""

    def __init__(self, m: "GatedDelta | ChannelDelta", num_slots: int, dtype, device):
        self.s = torch.zeros(num_slots, m.d.heads, m.vp, m.dp,
                             dtype=torch.float32, device=device)
        self.conv = torch.zeros(num_slots, m.d.conv - 1, m.channels,
                                dtype=dtype, device=device)


class GatedDelta(Part):
    """S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q per head
    (DeltaDims). One product yields queries, keys, values, gates and the
    numbers behind decays and step sizes."""

    def __init__(self, d: DeltaDims, width: int, eps: float, dtype):
        super().__init__()
        self.d, self.width, self.eps = d, width, eps
        self.wp = pad64(width)
        self.dp, self.vp = state_pad(d.dim), state_pad(d.vdim)
        H, G = d.heads, d.kv_heads
        # columns: queries, keys, values (these pass the convolutions),
        # gates, then b and a of every head
        self.channels = 2 * G * self.dp + H * self.vp
        self.ba_at = self.channels + H * self.vp
        self.win = weight(pad64(self.ba_at + 2 * H), self.wp, dtype)
        # [taps, channels]: the last row is the current token's
        self.conv = nn.Parameter(torch.empty(d.conv, self.channels,
                                             dtype=torch.float32))
        # A_log, then dt_bias, per head
        self.decay = nn.Parameter(torch.empty(2, H, dtype=torch.float32))
        self.o_norm = norm_weight(self.vp)
        self.wo = weight(self.wp, H * self.vp, dtype)

    def tensors(self):
        d, W = self.d, self.width
        qk, v = d.kv_heads * d.dim, d.heads * d.vdim
        return {"q": (qk, W), "q.conv": (qk, d.conv), "k": (qk, W),
                "k.conv": (qk, d.conv), "v": (v, W), "v.conv": (v, d.conv),
                "b": (d.heads, W), "A_log": (d.heads,), "norm": (d.vdim,),
                "a": (d.heads, W), "dt_bias": (d.heads,), "g": (v, W),
                "o": (W, v)}

    def checkpoint(self, src, pre):
        d = self.d
        t = self.checked(src, pre)
        heads = {"q": (d.kv_heads, d.dim, self.dp),
                 "k": (d.kv_heads, d.dim, self.dp),
                 "v": (d.heads, d.vdim, self.vp),
                 "g": (d.heads, d.vdim, self.vp)}
        w = [padded_heads(t[n], *heads[n], self.wp) for n in "qkvg"]
        w += [padded(t[n], d.heads, self.wp) for n in "ba"]
        conv = [padded_heads(t[n + ".conv"], *heads[n], d.conv)
                for n in "qkv"]
        return {"win": padded(torch.cat(w), *self.win.shape),
                "conv": torch.cat(conv).t(),
                "decay": torch.stack([t["A_log"], t["dt_bias"]]),
                "o_norm": padded(t["norm"], self.vp),
                "wo": padded_heads(t["o"].t(), d.heads, d.vdim, self.vp,
                                   self.wp).t()}

    def state_numel(self):
        return (self.d.heads * self.vp * self.dp,
                (self.d.conv - 1) * self.channels)

    def make_cache(self, num_blocks, blk, num_slots, dtype, device):
        return DeltaState(self, num_slots, dtype, device)

    def forward(self, h, batch, state):
        d = self.d
        ab = ops.linear(h, self.win)
        y = ops.gated_delta(
            ab, d.heads, d.kv_heads, self.dp, self.vp, d.dim, d.vdim,
            self.conv, self.decay, self.o_norm, d.unit_eps, self.eps,
            state.s, state.conv, batch.segments, batch.row_seq, batch.ctx)
        return ops.linear(y, self.wo)


class ChannelDelta(Branch):
    """The delta rule with a decay per head and key channel
    (ChannelDeltaDims). The inner numbers of decays and output gates are
    columns of the input product; one second product, block-diagonal, turns
    them into both."""

    def __init__(self, d: ChannelDeltaDims, width: int, eps: float, dtype):
        super().__init__()
        self.d, self.width, self.eps = d, width, eps
        self.wp = pad64(width)
        self.dp, self.vp = state_pad(d.dim), state_pad(d.vdim)
        H, G = d.heads, d.kv_heads
        # columns: queries, keys, values (these pass the convolutions),
        # the numbers behind step sizes, then the inner numbers
        self.channels = 2 * G * self.dp + H * self.vp
        self.inner_at = self.channels + pad64(H)
        self.inner = pad64(d.decay_rank + d.gate_rank)
        self.in_rows = self.inner_at + self.inner
        self.out_cols = H * self.vp
        # decays of all heads, then gates of all heads
        self.w2 = weight(H * (self.dp + self.vp), self.inner, dtype)
        self.conv = nn.Parameter(torch.empty(d.conv, self.channels,
                                             dtype=torch.float32))
        self.a_log = norm_weight(H)
        self.dt_bias = norm_weight(H * self.dp)
        self.o_norm = norm_weight(self.vp)

    def tensors(self):
        d, W = self.d, self.width
        qk, k, v = d.kv_heads * d.dim, d.heads * d.dim, d.heads * d.vdim
        return {"q": (qk, W), "q.conv": (qk, d.conv), "k": (qk, W),
                "k.conv": (qk, d.conv), "v": (v, W), "v.conv": (v, d.conv),
                "b": (d.heads, W), "A_log": (d.heads,), "norm": (d.vdim,),
                "a1": (d.decay_rank, W), "a2": (k, d.decay_rank),
                "dt_bias": (k,), "g1": (d.gate_rank, W),
                "g2": (v, d.gate_rank), "o": (W, v)}

    def _heads(self):
        d = self.d
        return (("q", d.kv_heads, d.dim, self.dp),
                ("k", d.kv_heads, d.dim, self.dp),
                ("v", d.heads, d.vdim, self.vp))

    def in_weight(self, t):
        w = [padded_heads(t[n], h, a, b, self.wp)
             for n, h, a, b in self._heads()]
        w.append(padded(t["b"], pad64(self.d.heads), self.wp))
        w.append(padded(torch.cat([t["a1"], t["g1"]]), self.inner, self.wp))
        return torch.cat(w)

    def out_weight(self, t):
        d = self.d
        return padded_heads(t["o"].t(), d.heads, d.vdim, self.vp,
                            self.wp).t()

    def extra(self, t):
        d, r = self.d, self.d.decay_rank
        a2 = padded_heads(t["a2"], d.heads, d.dim, self.dp, self.inner)
        g2 = padded_heads(t["g2"], d.heads, d.vdim, self.vp, d.gate_rank)
        low = a2.new_zeros(d.heads * self.vp, self.inner)
        low[:, r: r + d.gate_rank] = g2
        return {"w2": torch.cat([a2, low]),
                "conv": torch.cat([padded_heads(t[n + ".conv"], h, a, b,
                                                d.conv)
                                   for n, h, a, b in self._heads()]).t(),
                "a_log": t["A_log"],
                "dt_bias": padded_heads(t["dt_bias"][:, None], d.heads,
                                        d.dim, self.dp, 1)[:, 0],
                "o_norm": padded(t["norm"], self.vp)}

    def state_numel(self):
        return (self.d.heads * self.vp * self.dp,
                (self.d.conv - 1) * self.channels)

    def make_cache(self, num_blocks, blk, num_slots, dtype, device):
        return DeltaState(self, num_slots, dtype, device)

    def run(self, ab, batch, state, out, scale):
        d = self.d
        ag = ops.linear(ab[:, self.inner_at:], self.w2)
        ops.channel_delta(
            ab, ag, d.heads, d.kv_heads, self.dp, self.vp, d.dim, d.vdim,
            self.conv, self.a_log, self.dt_bias, self.o_norm, d.unit_eps,
            self.eps, scale, state.s, state.conv, batch.segments,
            batch.row_seq, batch.ctx, out)
