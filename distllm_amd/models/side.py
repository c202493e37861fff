"""Per-layer token inputs."""

from __future__ import annotations

from .. import ops
from .blocks import Part, norm_weight, pad64, padded, weight


class SideInput(Part):
    """What a layer adds to the residual stream for its token: a gated part
    of a second embedding table, proj(gelu(gate x) * e), RMS-normed by the
    launch that adds it."""

    def __init__(self, dim: int, width: int, dtype):
        super().__init__()
        self.dim, self.width = dim, width
        self.wp, self.sp = pad64(width), pad64(dim)
        self.gate = weight(self.sp, self.wp, dtype)
        self.proj = weight(self.wp, self.sp, dtype)
        self.norm = norm_weight(self.wp)

    def tensors(self):
        return {"gate": (self.dim, self.width),
                "proj": (self.width, self.dim), "norm": (self.width,)}

    def checkpoint(self, src, pre):
        t = self.checked(src, pre)
        return {"gate": padded(t["gate"], self.sp, self.wp),
                "proj": padded(t["proj"], self.wp, self.sp),
                "norm": padded(t["norm"], self.wp)}

    def forward(self, x, tokens, table, part: int):
        """x: the stream in the model's dtype; part: which `dim` columns
        of the table are this layer's."""
        g = ops.gated_rows(x, self.gate, tokens, table, part * self.dim,
                           self.dim)
        return ops.linear(g, self.proj)
