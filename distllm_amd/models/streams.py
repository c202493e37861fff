"""Several copies of the residual stream, mixed around every sublayer."""

from __future__ import annotations

import torch
from torch import nn

from .blocks import Part


class StreamMix(Part):
    """How a sublayer sits between the streams: it reads sum_s in[s] x_s,
    and x_t becomes sum_s mix[s, t] x_s + out[t] y for its output y. The
    numbers stay on the device, where the launch that joins sublayers reads
    them: in, out, then mix from-major, in fp32."""

    def __init__(self, streams: int):
        super().__init__()
        self.streams = streams
        self.coef = nn.Parameter(torch.empty(streams * (streams + 2),
                                             dtype=torch.float32))

    @property
    def reads(self) -> torch.Tensor:
        return self.coef[: self.streams]

    @property
    def writes(self) -> torch.Tensor:
        return self.coef[self.streams:]

    def tensors(self):
        s = self.streams
        return {"in": (s,), "out": (s,), "mix": (s, s)}

    def initial(self):
        s = self.streams
        return {"in": torch.full((s,), 1.0 / s), "out": torch.ones(s),
                "mix": torch.eye(s)}

    def checkpoint(self, src, pre):
        t = self.checked(src, pre)
        return {"coef": torch.cat([t[n].flatten()
                                   for n in ("in", "out", "mix")])}
