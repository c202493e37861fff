"""Mixers made of branches that share one input and one output product."""

from __future__ import annotations

import torch
from torch import nn

from .. import ops
from .attention import RotaryAttention
from .blocks import Branch, Part, norm_weight, pad64, padded, weight
from .config import ParallelDims
from .delta import ChannelDelta


class BranchMixer(Part):
    """Sum of branches, each times its scale. One product yields what all
    branches want of the mixer's input, one product maps all their outputs;
    the scales are applied to the fp32 outputs of the branches, and output
    biases are left to the launch that adds the mixer's result to the
    residual stream (`out_bias`, fp32)."""

    def __init__(self, branches: dict[str, tuple[Branch, float]], width: int,
                 dtype):
        super().__init__()
        self.width, self.wp = width, pad64(width)
        self.prefixes = list(branches)
        self.scales = [s for _, s in branches.values()]
        self.branches = nn.ModuleList(b for b, _ in branches.values())
        n = sum(b.in_rows for b in self.branches)
        self.win = weight(n, self.wp, dtype)
        self.bias = nn.Parameter(torch.empty(n, dtype=dtype))
        self.wo = weight(self.wp, sum(b.out_cols for b in self.branches),
                         dtype)
        self.out_bias = norm_weight(self.wp)

    def tensors(self):
        return {p + n: s for p, b in zip(self.prefixes, self.branches)
                for n, s in b.tensors().items()}

    def checkpoint(self, src, pre):
        ts = [b.checked(src, pre + p)
              for p, b in zip(self.prefixes, self.branches)]
        each = list(zip(self.branches, ts, self.scales))
        biases = [b.in_bias(t) for b, t, _ in each]
        out = {"win": torch.cat([b.in_weight(t) for b, t, _ in each]),
               "bias": torch.cat([
                   x if x is not None else next(iter(t.values())).new_zeros(
                       b.in_rows)
                   for x, (b, t, _) in zip(biases, each)]),
               "wo": torch.cat([b.out_weight(t) for b, t, _ in each], 1)}
        total = [scale * padded(b.out_bias(t).float(), self.wp)
                 for b, t, scale in each if b.out_bias(t) is not None]
        out["out_bias"] = sum(total, out["win"].new_zeros(
            self.wp, dtype=torch.float32))
        for i, (b, t, _) in enumerate(each):
            out |= {f"branches.{i}.{k}": v for k, v in b.extra(t).items()}
        return out

    def cache_numel(self):
        return sum(b.cache_numel() for b in self.branches)

    def state_numel(self):
        each = [b.state_numel() for b in self.branches]
        return sum(f for f, _ in each), sum(o for _, o in each)

    def make_cache(self, *args):
        return [b.make_cache(*args) for b in self.branches]

    def forward(self, h, batch, caches):
        ab = ops.linear(h, self.win, self.bias)
        o = h.new_empty(h.shape[0], self.wo.shape[1])
        at = col = 0
        for b, cache, scale in zip(self.branches, caches, self.scales):
            b.run(ab[:, at: at + b.in_rows], batch, cache,
                  o[:, col: col + b.out_cols], scale)
            at += b.in_rows
            col += b.out_cols
        return ops.linear(o, self.wo)


def parallel_mixer(d: ParallelDims, width: int, eps: float,
                   dtype) -> BranchMixer:
    return BranchMixer(
        {"left.": (RotaryAttention(d.left, width, eps, dtype), d.left_scale),
         "right.": (ChannelDelta(d.right, width, eps, dtype),
                    d.right_scale)}, width, dtype)
