"""Kanotar: a decoder-only LM of latent-attention layers.

Every layer has its own sizes, sliding window and feed-forward; a layer
may read an earlier layer's cached latents instead of having its own.
There are no positions in the attention. Each sublayer is normed on both
sides (x += norm(f(norm(x)))) and the residual stream is fp32, so the
step is a chain of products joined by one fused norm-add-norm launch per
sublayer.

The model works on ragged step batches only (engine/step.py): rows of
any mix of prompt portions and single decoded tokens, against one paged
latent cache per layer that owns latents.
"""

from __future__ import annotations

import torch
from torch import nn

from .. import ops
from .blocks import MIXERS, MLPS, expect, norm_weight, pad64, padded
from .config import LayeredDims


class LatentCache:
    """Paged latents: one [blocks, BLK, rank] tensor per layer that has a
    latent of its own; layers that share one hold the same tensor."""

    def __init__(self, model: "KanotarModel", num_blocks: int, blk: int):
        self.layers: list[torch.Tensor] = []
        for layer in model.layers:
            m = layer.mixer
            if m.own:
                self.layers.append(torch.zeros(
                    num_blocks, blk, m.rp, dtype=model.dtype,
                    device=model.device))
            else:
                self.layers.append(self.layers[m.d.kv_from])


class KanotarLayer(nn.Module):
    def __init__(self, d, width: int, eps: float, dtype):
        super().__init__()
        wp = pad64(width)
        self.mixer = MIXERS[d.mixer.type](d.mixer, width, eps, dtype)
        self.norm1, self.norm1b = norm_weight(wp), norm_weight(wp)
        self.mlp = self.norm2 = self.norm2b = None
        if d.mlp is not None:
            self.mlp = MLPS[d.mlp.kind](d.mlp, width, dtype)
            self.norm2, self.norm2b = norm_weight(wp), norm_weight(wp)


class KanotarModel(nn.Module):
    # the engine feeds ragged step batches and grows sequences as they go
    ragged = True
    # portions of at least this many tokens take the expanded attention
    expand_min = 32

    def __init__(self, dims: LayeredDims, dtype=torch.bfloat16,
                 tp_group=None):
        super().__init__()
        if tp_group is not None:
            raise ValueError("kanotar models run on one GPU per engine "
                             "(tensor_parallel_size 1)")
        self.dims = dims
        W, wp = dims.hidden_size, pad64(dims.hidden_size)
        self.vp = pad64(dims.vocab_size)
        self.tok_emb = nn.Parameter(
            torch.empty(dims.vocab_size, wp, dtype=dtype))
        self.layers = nn.ModuleList(
            KanotarLayer(d, W, dims.norm_eps, dtype) for d in dims.layers)
        self.final_norm = norm_weight(wp)
        self.lm_head = nn.Parameter(torch.empty(self.vp, wp, dtype=dtype))
        self.reset_parameters()

    @torch.no_grad()
    def reset_parameters(self):
        """Random weights, through the loader so that padding stays 0."""
        dims = self.dims
        src = {}
        dev = self.device

        def lin(name, rows, cols):
            src[name] = torch.randn(rows, cols, device=dev,
                                    dtype=self.dtype) * 0.02

        def ones(name, n):
            src[name] = torch.ones(n, device=dev)

        W = dims.hidden_size
        lin("embed", dims.vocab_size, W)
        for i, layer in enumerate(dims.layers):
            p, m = f"l{i}.", layer.mixer
            ones(p + "norm1", W), ones(p + "norm1b", W)
            lin(p + "mix.dq", m.q_rank, W)
            ones(p + "mix.dq.norm", m.q_rank)
            lin(p + "mix.uq", m.heads * m.dim, m.q_rank)
            if m.kv_from is None:
                lin(p + "mix.dkv", m.kv_rank, W)
                ones(p + "mix.dkv.norm", m.kv_rank)
            lin(p + "mix.uk", m.heads * m.dim, m.kv_rank)
            lin(p + "mix.uv", m.heads * m.vdim, m.kv_rank)
            lin(p + "mix.o", W, m.heads * m.vdim)
            if layer.mlp is not None:
                ones(p + "norm2", W), ones(p + "norm2b", W)
                lin(p + "mlp.gate", layer.mlp.ff, W)
                lin(p + "mlp.up", layer.mlp.ff, W)
                lin(p + "mlp.down", W, layer.mlp.ff)
            # layer by layer: a large model is not held twice
            self._copy_layer(src, i)
            for k in [k for k in src if k.startswith(p)]:
                del src[k]
        ones("final.norm", W)
        lin("head", dims.vocab_size, W)
        self._copy_ends(src)

    def _layer_tensors(self, src: dict, i: int) -> dict[str, torch.Tensor]:
        layer, p = self.layers[i], f"l{i}."
        W = self.dims.hidden_size
        out = {}
        for n in ("norm1", "norm1b", "norm2", "norm2b"):
            if getattr(layer, n) is not None:
                out[n] = padded(expect(p + n, src[p + n], W), pad64(W))
        for k, v in layer.mixer.checkpoint(src, p + "mix.").items():
            out["mixer." + k] = v
        if layer.mlp is not None:
            for k, v in layer.mlp.checkpoint(src, p + "mlp.").items():
                out["mlp." + k] = v
        return {f"layers.{i}.{k}": v for k, v in out.items()}

    def _end_tensors(self, src: dict) -> dict[str, torch.Tensor]:
        W, V = self.dims.hidden_size, self.dims.vocab_size
        wp = pad64(W)
        return {
            "tok_emb": padded(expect("embed", src["embed"], V, W), V, wp),
            "final_norm": padded(
                expect("final.norm", src["final.norm"], W), wp),
            "lm_head": padded(expect("head", src["head"], V, W),
                              self.vp, wp),
        }

    def checkpoint(self, src: dict) -> dict[str, torch.Tensor]:
        """Parameter name -> tensor, from a checkpoint's raw tensors."""
        out = self._end_tensors(src)
        for i in range(len(self.layers)):
            out.update(self._layer_tensors(src, i))
        return out

    def checkpoint_names(self) -> set[str]:
        """Every tensor name that a checkpoint of these dims holds."""
        names = {"embed", "final.norm", "head"}
        for i, layer in enumerate(self.dims.layers):
            p = f"l{i}."
            mix = ["dq", "dq.norm", "uq", "uk", "uv", "o"]
            if layer.mixer.kv_from is None:
                mix += ["dkv", "dkv.norm"]
            names |= {p + "norm1", p + "norm1b"}
            names |= {p + "mix." + n for n in mix}
            if layer.mlp is not None:
                names |= {p + "norm2", p + "norm2b", p + "mlp.gate",
                          p + "mlp.up", p + "mlp.down"}
        return names

    def _copy(self, tensors: dict):
        own = dict(self.named_parameters())
        for k, v in tensors.items():
            own[k].copy_(v.to(own[k].dtype))

    def _copy_layer(self, src, i):
        self._copy(self._layer_tensors(src, i))

    def _copy_ends(self, src):
        self._copy(self._end_tensors(src))

    @property
    def device(self):
        return self.tok_emb.device

    @property
    def dtype(self):
        return self.tok_emb.dtype

    @property
    def embedding_size(self) -> int:
        return self.dims.hidden_size

    # ---- cache ----------------------------------------------------------
    def cache_bytes_per_block(self, blk: int, kv_cache_dtype: str) -> int:
        el = self.tok_emb.element_size()
        return sum(m.rp * blk * el for m in
                   (layer.mixer for layer in self.layers) if m.own)

    def make_cache(self, num_blocks: int, blk: int,
                   kv_cache_dtype: str) -> LatentCache:
        if kv_cache_dtype != "bf16":
            raise ValueError("the latent cache is kept in the model's "
                             f"dtype, not {kv_cache_dtype}")
        return LatentCache(self, num_blocks, blk)

    # ---- step -----------------------------------------------------------
    @torch.no_grad()
    def forward_step(self, batch, cache: LatentCache,
                     trace: list | None = None) -> torch.Tensor:
        """Final normed hidden state [M, padded width] of every row.
        trace, when given, collects the residual after every layer."""
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

    @torch.no_grad()
    def logits(self, hidden: torch.Tensor) -> torch.Tensor:
        """hidden [..., width or padded width] -> [..., vocab] f32."""
        wp = self.lm_head.shape[1]
        if hidden.shape[-1] != wp:
            hidden = nn.functional.pad(hidden, (0, wp - hidden.shape[-1]))
        out = ops.linear(hidden.contiguous(), self.lm_head)
        return (out[..., : self.dims.vocab_size].float()
                * self.dims.logit_scale)

    @torch.no_grad()
    def decode_step(self, tokens, cache: LatentCache, block_tables,
                    ctx_lens) -> torch.Tensor:
        """One token for each of B sequences (ctx_lens counts it)."""
        from ..engine.step import StepBatch

        batch = StepBatch.decode(tokens, block_tables, ctx_lens)
        return self.logits(self.forward_step(batch, cache))

    @torch.no_grad()
    def forward(self, input_ids: torch.Tensor,
                attention_mask: torch.Tensor) -> torch.Tensor:
        """Whole padded sequences without an engine: [B, S] ->
        hidden [B, S, width], zeros at padding."""
        from ..engine.step import StepBatch

        blk = 16
        mask = attention_mask.bool()
        rows = [input_ids[b][mask[b]].tolist()
                for b in range(input_ids.shape[0])]
        need = [(len(r) + blk - 1) // blk for r in rows]
        cache = LatentCache(self, sum(need) + 1, blk)
        entries, at = [], 1
        for b, r in enumerate(rows):
            if r:
                entries.append((r, 0, list(range(at, at + need[b]))))
            at += need[b]
        out = torch.zeros(*input_ids.shape, self.dims.hidden_size,
                          dtype=self.dtype, device=self.device)
        if entries:
            batch = StepBatch.build(entries, blk, self.device)
            h = self.forward_step(batch, cache)
            order = torch.cat([torch.as_tensor(r) for r in batch.rows])
            out[mask] = h[order.to(self.device),
                          : self.dims.hidden_size]
        return out
