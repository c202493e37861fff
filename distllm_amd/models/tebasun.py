"""Tebasun: a decoder-only LM of two kinds of layers, attention beside a
delta rule and linear recurrent units, some of which run in a loop.

Sublayers read tanh(alpha x) w + b of the fp32 residual stream and their
outputs are added as they are; every layer ends with a gated input of its
own for its token. Before a pass of the loop, the pass's vector and, from
the second pass on, the embedding output are added. One launch per sublayer
boundary adds, activates and casts.
"""

from __future__ import annotations

import torch

from .. import ops
from .layered import LayeredCache, LayeredModel


class TebasunModel(LayeredModel):
    layer_norms = ("norm1", "norm1.b", "norm1.alpha")
    mlp_norms = ("norm2", "norm2.b", "norm2.alpha")
    final_norms = ("final.norm", "final.norm.b", "final.norm.alpha")
    tied_head = True

    def _before(self, run: int, tokens):
        """What a layer run is preceded by: arguments of residual_step
        that add to the stream, and the activation of its input (of the
        head's input, after the last run)."""
        if run == len(self.runs):
            return {}, (self.final_norm, self.final_norm_b,
                        self.final_norm_alpha)
        i, start = self.runs[run]
        layer, add = self.layers[i], {}
        if start is not None:
            add["vec"] = self.loop_step[start]
            if start > 0:
                add["embed"] = (tokens, self.tok_emb, self.dims.embed_scale)
        return add, (layer.norm1, layer.norm1_b, layer.norm1_alpha)

    @torch.no_grad()
    def forward_step(self, batch, cache: LayeredCache,
                     trace: list | None = None) -> torch.Tensor:
        W, eps = self.dims.hidden_size, self.dims.norm_eps
        tokens = batch.tokens
        x = torch.empty(tokens.shape[0], self.tok_emb.shape[1],
                        dtype=torch.float32, device=self.device)
        add, act = self._before(0, tokens)
        h = ops.residual_step(x, act=act, fresh=True, **{
            "embed": (tokens, self.tok_emb, self.dims.embed_scale), **add})
        for r, (i, _) in enumerate(self.runs):
            layer = self.layers[i]
            y = layer.mixer(h, batch, cache.layers[r])
            bias = getattr(layer.mixer, "out_bias", None)
            if layer.mlp is not None:
                h = ops.residual_step(x, y, bias=bias, act=(
                    layer.norm2, layer.norm2_b, layer.norm2_alpha))
                y, bias = layer.mlp(h), None
            add, act = self._before(r + 1, tokens)
            last = {}
            if layer.side is not None:
                h = ops.residual_step(x, y, bias=bias)
                y = layer.side(h, tokens, self.side_emb, i)
                bias, last = None, {"rms": (layer.side.norm, W, eps)}
            if trace is not None:
                ops.residual_step(x, y, bias=bias, **last)
                trace.append(x[:, :W].clone())
                y, bias, last = None, None, {}
            h = ops.residual_step(x, y, bias=bias, act=act,
                                  dtype=self.dtype, **last, **add)
        return h
