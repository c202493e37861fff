"""Kanotar: a decoder-only LM of latent-attention layers.

Every layer has its own sizes, sliding window and feed-forward; a layer
may read an earlier layer's cached latents instead of having its own.
There are no positions in the attention. Each sublayer is normed on both
sides (x += norm(f(norm(x)))) and the residual stream is fp32, so the
step is a chain of products joined by one fused norm-add-norm launch per
sublayer.
"""

from __future__ import annotations

import torch

from .. import ops
from .layered import LayeredCache, LayeredModel


class KanotarModel(LayeredModel):
    layer_norms = ("norm1", "norm1b")
    mlp_norms = ("norm2", "norm2b")

    @torch.no_grad()
    def forward_step(self, batch, cache: LayeredCache,
                     trace: list | None = None) -> torch.Tensor:
        W, eps = self.dims.hidden_size, self.dims.norm_eps
        h, x = ops.embed_norm(batch.tokens, self.tok_emb,
                              self.layers[0].norm1, W, eps)
        for i, layer in enumerate(self.layers):
            after = (self.layers[i + 1].norm1 if i + 1 < len(self.layers)
                     else self.final_norm)
            y = layer.mixer(h, batch, cache.layers[i])
            if layer.mlp is None:
                h = ops.post_norm_add(y, x, layer.norm1b, after, W, eps)
            else:
                h = ops.post_norm_add(y, x, layer.norm1b, layer.norm2, W,
                                      eps)
                h = ops.post_norm_add(layer.mlp(h), x, layer.norm2b, after,
                                      W, eps)
            if trace is not None:
                trace.append(x[:, :W].clone())
        return h
