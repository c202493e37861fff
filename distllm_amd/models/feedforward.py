"""Feed-forwards: SwiGLU, xIELU, routed gated-unit and squared-ReLU
experts."""

from __future__ import annotations

import torch
from torch import nn

from .. import ops
from .blocks import Part, norm_weight, pad64, padded, weight
from .config import ExpertsDims, GatedExpertsDims, SwigluDims, XieluDims


class SwigluMlp(Part):
    """down(silu(gate h) * (up h)): the clamped unit without a limit."""

    def __init__(self, d: SwigluDims, width: int, dtype):
        super().__init__()
        self.d, self.width = d, width
        self.wp, self.fp = pad64(width), pad64(d.ff)
        self.wgup = weight(2 * self.fp, self.wp, dtype)
        self.wdown = weight(self.wp, self.fp, dtype)

    def tensors(self):
        ff, W = self.d.ff, self.width
        return {"gate": (ff, W), "up": (ff, W), "down": (W, ff)}

    def checkpoint(self, src, pre):
        t = self.checked(src, pre)
        return {"wgup": torch.cat([padded(t[n], self.fp, self.wp)
                                   for n in ("gate", "up")]),
                "wdown": padded(t["down"], self.wp, self.fp)}

    def forward(self, h):
        y = ops.gateup_clamped_glu(h, self.wgup, float("inf"), 1.0, 0.0)
        return ops.linear(y, self.wdown)


class XieluMlp(Part):
    """down(xielu(up h)); the activation's two numbers stay on the device,
    where the kernels read them."""

    def __init__(self, d: XieluDims, width: int, dtype):
        super().__init__()
        self.d, self.width = d, width
        self.wp, self.fp = pad64(width), pad64(d.ff)
        self.wup = weight(self.fp, self.wp, dtype)
        self.wdown = weight(self.wp, self.fp, dtype)
        self.act = nn.Parameter(torch.empty(2, dtype=torch.float32))

    def tensors(self):
        ff, W = self.d.ff, self.width
        return {"up": (ff, W), "down": (W, ff), "act": (2,)}

    def checkpoint(self, src, pre):
        t = self.checked(src, pre)
        return {"wup": padded(t["up"], self.fp, self.wp),
                "wdown": padded(t["down"], self.wp, self.fp),
                "act": t["act"]}

    def forward(self, h):
        return ops.linear(ops.up_xielu(h, self.wup, self.act), self.wdown)


class RoutedExperts(Part):
    """Routed experts (ExpertsDims): rows are sorted by expert and every
    expert's products run on its rows only. Gate and up rows of an expert
    alternate in groups of 16, so that one tile of the product holds both
    halves of the unit."""

    UNIT = 16

    def __init__(self, d: ExpertsDims, width: int, dtype):
        super().__init__()
        self.d, self.width = d, width
        self.wp, self.fp = pad64(width), pad64(d.ff)
        self.router = weight(d.experts, self.wp, dtype)
        self.wgup = nn.Parameter(torch.empty(d.experts, 2 * self.fp, self.wp,
                                             dtype=dtype))
        self.wdown = nn.Parameter(torch.empty(d.experts, self.wp, self.fp,
                                              dtype=dtype))

    def tensors(self):
        ff, W = self.d.ff, self.width
        t = {}
        for e in range(self.d.experts):
            t |= {f"e{e}.gate": (ff, W), f"e{e}.up": (ff, W),
                  f"e{e}.down": (W, ff)}
        return t | {"router": (self.d.experts, W)}

    def checkpoint(self, src, pre):
        t = self.checked(src, pre)
        U = self.UNIT

        def gup(e):
            halves = [padded(t[f"e{e}.{n}"], self.fp, self.wp)
                      .view(-1, U, self.wp) for n in ("gate", "up")]
            return torch.stack(halves, 1).view(2 * self.fp, self.wp)

        return {"router": padded(t["router"], self.d.experts, self.wp),
                "wgup": torch.stack([gup(e) for e in range(self.d.experts)]),
                "wdown": torch.stack([padded(t[f"e{e}.down"], self.wp,
                                             self.fp)
                                      for e in range(self.d.experts)])}

    def forward(self, h, ctx):
        """-> outputs [rows * top, width] of the chosen experts, row by
        row, and their weights [rows, top]; rows with ctx 0 have none."""
        d = self.d
        ids, weights = ops.route(h, self.router, ctx, d.top, d.groups,
                                 d.keep)
        return ops.experts(h, ids, self.wgup, self.wdown), weights


class GatedExperts(Part):
    """Squared-ReLU experts chosen by corrected sigmoid scores, beside a
    shared one with a gate per token (GatedExpertsDims). The shared
    expert's gate is a row behind the router's.

    Its columns are cut into shards of the size of an expert: a sum over
    columns, it is the sum of experts that serve every token. With few rows
    the shards are stored behind the experts and run with them, which saves
    the launches of two more products; with many rows they are the two
    products, the second on a copy of the weights in its order."""

    FEW = 256  # rows

    def __init__(self, d: GatedExpertsDims, width: int, dtype):
        super().__init__()
        self.d, self.width = d, width
        self.wp, self.fp = pad64(width), pad64(d.ff)
        n = d.experts
        self.shards = -(-(d.shared or 0) // self.fp)
        self.router = weight(n + (d.shared is not None), self.wp, dtype)
        self.correction = norm_weight(n)
        self.wup = nn.Parameter(torch.empty(n + self.shards, self.fp,
                                            self.wp, dtype=dtype))
        self.wdown = nn.Parameter(torch.empty(n + self.shards, self.wp,
                                              self.fp, dtype=dtype))
        if d.shared is not None:
            self.sp = pad64(d.shared)
            self.shared_down = weight(self.wp, self.sp, dtype)

    def tensors(self):
        d, W = self.d, self.width
        t = {}
        for e in range(d.experts):
            t |= {f"e{e}.up": (d.ff, W), f"e{e}.down": (W, d.ff)}
        t |= {"router": (d.experts, W), "correction": (d.experts,)}
        if d.shared is not None:
            t |= {"shared.up": (d.shared, W), "shared.down": (W, d.shared),
                  "shared.sg": (1, W)}
        return t

    def checkpoint(self, src, pre):
        t, n = self.checked(src, pre), self.d.experts
        up = [padded(t[f"e{e}.up"], self.fp, self.wp) for e in range(n)]
        down = [padded(t[f"e{e}.down"], self.wp, self.fp) for e in range(n)]
        router, out = t["router"], {}
        if self.d.shared is not None:
            router = torch.cat([router, t["shared.sg"]])
            out = {"shared_down": padded(t["shared.down"], self.wp, self.sp)}
            m = self.shards * self.fp
            up += padded(t["shared.up"], m, self.wp).split(self.fp)
            down += padded(t["shared.down"], self.wp, m).split(self.fp, 1)
        return out | {"router": padded(router, *self.router.shape),
                      "correction": t["correction"],
                      "wup": torch.stack(up), "wdown": torch.stack(down)}

    def forward(self, h, ctx):
        """-> outputs of the chosen experts, row by row [rows * choices,
        width], the shared expert's [rows, width] where it is not among
        them, and the weights of both; rows with ctx 0 have none."""
        d = self.d
        few = h.shape[0] <= self.FEW
        ids, weights = ops.route_sigmoid(
            h, self.router, self.correction, ctx, d.top, d.scale,
            self.shards if few else 0)
        y = ops.experts(h, ids, self.wup, self.wdown, gated=False)
        shared = None
        if d.shared is not None and not few:
            up = self.wup[d.experts:].flatten(0, 1)[: self.sp]
            shared = ops.linear(ops.up_relu2(h, up), self.shared_down)
        return y, shared, weights
