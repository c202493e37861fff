"""Bufulorn: a decoder-only LM of chunked-attention and delta-rule layers
with xIELU feed-forwards or routed experts.

The sublayers read the residual stream itself and only their outputs are
normed (x += layer_norm(f(x))); the stream is fp32 and starts as token
plus position vector. A step is a chain of products and mixer kernels
joined by one launch per sublayer that norms, adds and casts.
"""

from __future__ import annotations

import torch

from .. import ops
from .feedforward import RoutedExperts
from .layered import LayeredCache, LayeredModel


class BufulornModel(LayeredModel):
    layer_norms = ("norm1", "norm1.b")
    mlp_norms = ("norm2", "norm2.b")
    final_norms = ("final.norm", "final.norm.b")
    has_positions = True

    @torch.no_grad()
    def forward_step(self, batch, cache: LayeredCache,
                     trace: list | None = None) -> torch.Tensor:
        W, eps = self.dims.hidden_size, self.dims.norm_eps
        h, x = ops.embed_positions(batch.tokens, batch.ctx, self.tok_emb,
                                   self.pos_emb)
        for i, layer in enumerate(self.layers):
            final = (None if i + 1 < len(self.layers)
                     else (self.final_norm, self.final_norm_b))
            y = layer.mixer(h, batch, cache.layers[i])
            h = ops.layer_norm_add(
                y, x, layer.norm1, layer.norm1_b, W, eps,
                final if layer.mlp is None else None)
            if layer.mlp is not None:
                mix = None
                if isinstance(layer.mlp, RoutedExperts):
                    # the experts' outputs are summed by the next launch
                    y, mix = layer.mlp(h, batch.ctx)
                else:
                    y = layer.mlp(h)
                h = ops.layer_norm_add(y, x, layer.norm2, layer.norm2_b, W,
                                       eps, final, mix)
            if trace is not None:
                trace.append(x[:, :W].clone())
        return h
