"""Kedelorn: a decoder-only LM of retention and latent-attention layers
with routed squared-ReLU experts, on several residual streams.

Every sublayer reads an RMS-normed mix of the streams; its output goes to
all of them while they are mixed with one another. One launch per sublayer
boundary sums the experts' outputs, mixes the fp32 streams and norms the
next input; until the first sublayer's output the streams are the embedding
itself and are not stored, and after the last one only their sum is formed.
"""

from __future__ import annotations

import torch

from .. import ops
from .layered import LayeredCache, LayeredModel


class KedelornModel(LayeredModel):
    layer_norms = ("norm1",)
    mlp_norms = ("norm2",)
    norm_offset = 1.0  # norm weights are stored around zero

    @torch.no_grad()
    def forward_step(self, batch, cache: LayeredCache,
                     trace: list | None = None) -> torch.Tensor:
        d = self.dims
        W, eps = d.hidden_size, d.norm_eps
        x = torch.empty(batch.tokens.shape[0], d.streams,
                        self.tok_emb.shape[1], dtype=torch.float32,
                        device=self.device)
        first = self.layers[0]
        embed = (batch.tokens, self.tok_emb)
        h = ops.stream_step(x, embed=embed, read=first.hc1.reads,
                            norm=(first.norm1, W, eps), dtype=self.dtype)
        for i, layer in enumerate(self.layers):
            last = i + 1 == len(self.layers)
            after = ({"norm": (self.final_norm, W, eps),
                      "store": trace is not None} if last else
                     {"norm": (self.layers[i + 1].norm1, W, eps),
                      "read": self.layers[i + 1].hc1.reads})
            y, hc = layer.mixer(h, batch, cache.layers[i]), layer.hc1
            mix = shared = None
            if layer.mlp is not None:
                h = ops.stream_step(x, y, hc.writes, embed=embed,
                                    read=layer.hc2.reads,
                                    norm=(layer.norm2, W, eps))
                # the experts' outputs are summed by the next launch
                y, shared, mix = layer.mlp(h, batch.ctx)
                hc, embed = layer.hc2, None
            h = ops.stream_step(x, y, hc.writes, mix=mix, shared=shared,
                                embed=embed, **after)
            embed = None
            if trace is not None:
                trace.append(x[..., :W].sum(1))
        return h
