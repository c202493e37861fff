"""Real-gated linear recurrent unit."""

from __future__ import annotations

import torch
from torch import nn

from .. import ops
from .blocks import Part, norm_weight, pad64, padded, weight
from .config import LruDims


class LruState:
    """Slots of one layer: the fp32 state [slots, width] and the
    convolution's last inputs [slots, taps - 1, width]."""

    def __init__(self, m: "GatedLru", num_slots: int, dtype, device):
        self.s = torch.zeros(num_slots, m.cols, dtype=torch.float32,
                             device=device)
        self.conv = torch.zeros(num_slots, m.d.conv - 1, m.cols, dtype=dtype,
                                device=device)


class GatedLru(Part):
    """S <- a S + sqrt(1 - a^2) i u per channel (LruDims), the output times
    the GELU of a second branch. Blocks are padded to multiples of 32
    channels. One product yields both branches."""

    CHUNK = 64  # rows of a prompt whose recurrence starts from zeros

    def __init__(self, d: LruDims, width: int, eps: float, dtype):
        super().__init__()
        self.d, self.width, self.wp = d, width, pad64(width)
        self.size = d.width // d.blocks
        self.bs = (self.size + 31) // 32 * 32
        self.cols = pad64(d.blocks * self.bs)
        # the GELU branch, then the recurrent one
        self.win = weight(2 * self.cols, self.wp, dtype)
        self.bias = nn.Parameter(torch.empty(2 * self.cols, dtype=dtype))
        self.conv = nn.Parameter(torch.empty(d.conv, self.cols,
                                             dtype=torch.float32))
        self.conv_b = norm_weight(self.cols)
        # decay and input gates: [gate, block, out, in], stored in the order
        # of ops.lru_gate_order
        self.gates = nn.Parameter(torch.empty(2, d.blocks, self.bs, self.bs,
                                              dtype=dtype))
        self.gates_b = nn.Parameter(torch.empty(2, self.cols,
                                                dtype=torch.float32))
        self.decay = norm_weight(self.cols)  # -decay_scale * softplus(lam)
        self.wo = weight(self.wp, self.cols, dtype)

    def tensors(self):
        d, n, s = self.d, self.d.width, self.size
        return {"y": (n, self.width), "y.b": (n,), "x": (n, self.width),
                "x.b": (n,), "conv": (n, d.conv), "conv.b": (n,),
                "ra": (d.blocks, s, s), "ra.b": (d.blocks, s),
                "ri": (d.blocks, s, s), "ri.b": (d.blocks, s),
                "lam": (n,), "o": (self.width, n)}

    def _blocks(self, w: torch.Tensor) -> torch.Tensor:
        """[width, ...] -> [cols, ...]"""
        w = w.reshape(self.d.blocks, self.size, *w.shape[1:])
        rest = w.shape[2:]
        w = padded(w, self.d.blocks, self.bs, *rest)
        return padded(w.reshape(-1, *rest), self.cols, *rest)

    def checkpoint(self, src, pre):
        t = self.checked(src, pre)
        B = self.d.blocks

        def gate(n):
            return padded(t[n], B, self.bs, self.bs)

        soft = torch.nn.functional.softplus(t["lam"].double())
        return {"win": torch.cat([padded(self._blocks(t[n]), self.cols,
                                         self.wp) for n in "yx"]),
                "bias": torch.cat([self._blocks(t[n + ".b"]) for n in "yx"]),
                "conv": self._blocks(t["conv"]).t(),
                "conv_b": self._blocks(t["conv.b"]),
                "gates": ops.lru_gate_order(
                    torch.stack([gate("ra"), gate("ri")])),
                "gates_b": torch.stack([self._blocks(t[n].reshape(-1))
                                        for n in ("ra.b", "ri.b")]),
                "decay": self._blocks(-self.d.decay_scale * soft),
                "wo": padded(self._blocks(t["o"].t()), self.cols,
                             self.wp).t()}

    def state_numel(self):
        return self.cols, (self.d.conv - 1) * self.cols

    def make_cache(self, num_blocks, blk, num_slots, dtype, device):
        return LruState(self, num_slots, dtype, device)

    def forward(self, h, batch, state):
        ab = ops.linear(h, self.win, self.bias)
        y = ops.gated_lru(ab, self.conv, self.conv_b, self.gates,
                          self.gates_b, self.decay, state.s, state.conv,
                          batch.segments, batch.row_seq, batch.ctx,
                          self.CHUNK)
        return ops.linear(y, self.wo)
