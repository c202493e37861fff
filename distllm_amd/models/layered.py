"""Decoders that are described layer by layer (LayeredDims).

A layer is a mixer and, mostly, a feed-forward, each with sizes of its
own; how they are joined to the fp32 residual stream is the design's and
left to a subclass (`forward_step`). The model runs on ragged step
batches only (engine/step.py): rows of any mix of prompt portions and
single decoded tokens, against one cache entry per layer that owns one
and, where there are recurrent layers, one state slot per sequence. Layers
of a loop run several times; every run has a cache entry of its own.
"""

from __future__ import annotations

import torch
from torch import nn

from .. import ops
from .attention import PagedAttention
from .blocks import (ClampedGlu, LatentAttention, expect, norm_weight, pad64,
                     padded, weight)
from .branches import parallel_mixer
from .config import (AttentionDims, ClampedGluDims, DeltaDims, ExpertsDims,
                     GatedExpertsDims, LatentAttentionDims, LayeredDims,
                     LruDims, ParallelDims, RetentionDims, RotaryLatentDims,
                     SwigluDims, XieluDims)
from .delta import GatedDelta
from .feedforward import GatedExperts, RoutedExperts, SwigluMlp, XieluMlp
from .latent import RotaryLatentAttention
from .recurrent import GatedLru
from .retention import Retention
from .side import SideInput
from .streams import StreamMix

MIXERS = {LatentAttentionDims: LatentAttention,
          AttentionDims: PagedAttention, DeltaDims: GatedDelta,
          ParallelDims: parallel_mixer, LruDims: GatedLru,
          RotaryLatentDims: RotaryLatentAttention, RetentionDims: Retention}
MLPS = {ClampedGluDims: ClampedGlu, SwigluDims: SwigluMlp,
        XieluDims: XieluMlp, ExpertsDims: RoutedExperts,
        GatedExpertsDims: GatedExperts}


class LayeredCache:
    """What every layer run keeps between steps. A layer that shares
    another layer's cache holds the same object."""

    def __init__(self, model: "LayeredModel", num_blocks: int, blk: int,
                 num_slots: int = 0):
        self.layers: list = []
        latest: dict[int, object] = {}  # of the layer's runs so far
        for i, _ in model.runs:
            m = model.layers[i].mixer
            latest[i] = (m.make_cache(num_blocks, blk, num_slots,
                                      model.dtype, model.device)
                         if m.own else latest[m.kv_from])
            self.layers.append(latest[i])


class Layer(nn.Module):
    def __init__(self, d, width: int, eps: float, dtype,
                 norms: tuple[str, ...], mlp_norms: tuple[str, ...],
                 side: int | None = None, streams: int | None = None):
        super().__init__()
        wp = pad64(width)
        self.mixer = MIXERS[type(d.mixer)](d.mixer, width, eps, dtype)
        self.mlp = None
        if d.mlp is not None:
            self.mlp = MLPS[type(d.mlp)](d.mlp, width, dtype)
        self.side = (SideInput(side, width, dtype) if side is not None
                     else None)
        # how either sublayer sits between several residual streams
        self.hc1 = self.hc2 = None
        if streams is not None:
            self.hc1 = StreamMix(streams)
            self.hc2 = StreamMix(streams) if self.mlp is not None else None
        self.norm_names = norms + (mlp_norms if self.mlp is not None else ())
        for n in norms + mlp_norms:
            present = n in self.norm_names
            setattr(self, n.replace(".", "_"),
                    norm_weight(norm_size(n, wp)) if present else None)

    def parts(self) -> list[tuple[str, str, nn.Module]]:
        """(parameter prefix, checkpoint prefix, part)"""
        return [(a, b, m) for a, b, m in
                (("mixer.", "mix.", self.mixer), ("mlp.", "mlp.", self.mlp),
                 ("side.", "side.", self.side), ("hc1.", "hc1.", self.hc1),
                 ("hc2.", "hc2.", self.hc2)) if m is not None]


def norm_size(name: str, wp: int) -> int:
    """Numbers of a norm's tensor: one scale before the activation, or a
    vector."""
    return 1 if name.endswith(".alpha") else wp


class LayeredModel(nn.Module):
    # the engine feeds ragged step batches and grows sequences as they go
    ragged = True
    # portions of at least this many tokens take the attention form that
    # is made for prompts
    expand_min = 32
    # norm tensors of a layer, of a layer with a feed-forward, of the model
    layer_norms: tuple[str, ...] = ()
    mlp_norms: tuple[str, ...] = ()
    final_norms: tuple[str, ...] = ("final.norm",)
    has_positions = False  # a table of position vectors
    tied_head = False      # the output product uses the embedding table
    norm_offset = 0.0      # what is added to stored norm weights

    def __init__(self, dims: LayeredDims, dtype=torch.bfloat16,
                 tp_group=None):
        super().__init__()
        if tp_group is not None:
            raise ValueError(f"{dims.arch} models run on one GPU per engine "
                             "(tensor_parallel_size 1)")
        self.dims = dims
        W, wp = dims.hidden_size, pad64(dims.hidden_size)
        self.vp = pad64(dims.vocab_size)
        # layer runs in order: (layer, loop pass that begins with it)
        self.runs = dims.layer_runs()
        self.tok_emb = weight(self.vp if self.tied_head else dims.vocab_size,
                              wp, dtype)
        self.pos_emb = (weight(dims.max_position_embeddings, wp, dtype)
                        if self.has_positions else None)
        self.layers = nn.ModuleList(
            Layer(d, W, dims.norm_eps, dtype, self.layer_norms,
                  self.mlp_norms, dims.side_dim, dims.streams)
            for d in dims.layers)
        for n in self.final_norms:
            setattr(self, n.replace(".", "_"),
                    norm_weight(norm_size(n, wp)))
        self.side_emb = self.loop_step = None
        if dims.side_dim is not None:
            self.side_emb = weight(dims.vocab_size,
                                   len(dims.layers) * dims.side_dim, dtype)
        if dims.loop is not None:
            self.loop_step = nn.Parameter(torch.empty(
                dims.loop.times, wp, dtype=torch.float32))
        if not self.tied_head:
            self.lm_head = weight(self.vp, wp, dtype)
        self.reset_parameters()

    # ---- weights --------------------------------------------------------
    def _end_shapes(self) -> dict[str, tuple[int, ...]]:
        d = self.dims
        t = {"embed": (d.vocab_size, d.hidden_size)}
        if not self.tied_head:
            t["head"] = (d.vocab_size, d.hidden_size)
        if self.has_positions:
            t["pos"] = (d.max_position_embeddings, d.hidden_size)
        if d.side_dim is not None:
            t["side.embed"] = (d.vocab_size, len(d.layers) * d.side_dim)
        if d.loop is not None:
            t["loop.step"] = (d.loop.times, d.hidden_size)
        return t | {n: self._norm_shape(n) for n in self.final_norms}

    def _norm_shape(self, name: str) -> tuple[int, ...]:
        return () if name.endswith(".alpha") else (self.dims.hidden_size,)

    def _layer_shapes(self, i: int) -> dict[str, tuple[int, ...]]:
        layer, p = self.layers[i], f"l{i}."
        t = {p + n: self._norm_shape(n) for n in layer.norm_names}
        for _, pre, part in layer.parts():
            t |= {p + pre + n: s for n, s in part.tensors().items()}
        return t

    def checkpoint_names(self) -> set[str]:
        """Every tensor name that a checkpoint of these dims holds."""
        names = set(self._end_shapes())
        for i in range(len(self.layers)):
            names |= set(self._layer_shapes(i))
        return names

    def _end_tensors(self, src: dict) -> dict[str, torch.Tensor]:
        wp = self.tok_emb.shape[1]
        t = {n: expect(n, src[n], *s) for n, s in self._end_shapes().items()}
        out = {"tok_emb": padded(t["embed"], *self.tok_emb.shape)}
        if not self.tied_head:
            out["lm_head"] = padded(t["head"], self.vp, wp)
        if self.has_positions:
            out["pos_emb"] = padded(t["pos"], t["pos"].shape[0], wp)
        if self.side_emb is not None:
            out["side_emb"] = t["side.embed"]
        if self.loop_step is not None:
            out["loop_step"] = padded(t["loop.step"], *self.loop_step.shape)
        for n in self.final_norms:
            out[n.replace(".", "_")] = self._norm_tensor(n, t[n])
        return out

    def _norm_tensor(self, name: str, w: torch.Tensor) -> torch.Tensor:
        w = expect(name, w, *self._norm_shape(name))
        if w.dim() == 0:
            return w.reshape(1)
        if self.norm_offset:
            w = w.float() + self.norm_offset
        return padded(w, self.tok_emb.shape[1])

    def _layer_tensors(self, src: dict, i: int) -> dict[str, torch.Tensor]:
        layer, p = self.layers[i], f"l{i}."
        out = {n.replace(".", "_"): self._norm_tensor(p + n, src[p + n])
               for n in layer.norm_names}
        for name, pre, part in layer.parts():
            for k, v in part.checkpoint(src, p + pre).items():
                out[name + k] = v
        return {f"layers.{i}.{k}": v for k, v in out.items()}

    def checkpoint(self, src: dict) -> dict[str, torch.Tensor]:
        """Parameter name -> tensor, from a checkpoint's raw tensors."""
        out = self._end_tensors(src)
        for i in range(len(self.layers)):
            out.update(self._layer_tensors(src, i))
        return out

    @torch.no_grad()
    def reset_parameters(self):
        """Random weights, through the loader so that padding stays 0;
        layer by layer, so that a large model is not held twice."""
        own = dict(self.named_parameters())

        def fill(shapes, to_own, initial={}):
            src = {}
            for n, s in shapes.items():
                if n in initial:
                    src[n] = initial[n].to(self.device)
                elif n.endswith(".b") and len(s) == 1:
                    src[n] = torch.zeros(s, device=self.device)
                elif len(s) <= 1:
                    src[n] = torch.ones(s, device=self.device)
                else:
                    src[n] = torch.randn(s, device=self.device,
                                         dtype=self.dtype) * 0.02
            for k, v in to_own(src).items():
                own[k].copy_(v.to(own[k].dtype))

        def unit_norms(pre, names):
            if not self.norm_offset:
                return {}
            return {pre + n: torch.full(self._norm_shape(n),
                                        1.0 - self.norm_offset)
                    for n in names}

        for i in range(len(self.layers)):
            initial = {f"l{i}.{pre}{n}": v
                       for _, pre, part in self.layers[i].parts()
                       for n, v in part.initial().items()}
            initial |= unit_norms(f"l{i}.", self.layers[i].norm_names)
            fill(self._layer_shapes(i), lambda src: self._layer_tensors(
                src, i), initial)
        fill(self._end_shapes(), self._end_tensors,
             unit_norms("", self.final_norms))

    # ---- cache ----------------------------------------------------------
    def cache_bytes_per_block(self, blk: int, kv_cache_dtype: str) -> int:
        el = self.tok_emb.element_size()
        mixers = [self.layers[i].mixer for i, _ in self.runs]
        return sum(m.cache_numel() * blk * el for m in mixers if m.own)

    def state_bytes_per_slot(self) -> int:
        el = self.tok_emb.element_size()
        return sum(f32 * 4 + own * el for f32, own in
                   (self.layers[i].mixer.state_numel()
                    for i, _ in self.runs))

    def make_cache(self, num_blocks: int, blk: int, kv_cache_dtype: str,
                   num_slots: int = 0) -> LayeredCache:
        if kv_cache_dtype != "bf16":
            raise ValueError(f"the cache of {self.dims.arch} models is kept "
                             f"in the model's dtype, not {kv_cache_dtype}")
        return LayeredCache(self, num_blocks, blk, num_slots)

    # ---- step -----------------------------------------------------------
    def forward_step(self, batch, cache: LayeredCache,
                     trace: list | None = None) -> torch.Tensor:
        """Final normed hidden state [M, padded width] of every row.
        trace, when given, collects the residual after every layer run."""
        raise NotImplementedError

    @torch.no_grad()
    def logits(self, hidden: torch.Tensor) -> torch.Tensor:
        """hidden [..., width or padded width] -> [..., vocab] f32."""
        head = self.tok_emb if self.tied_head else self.lm_head
        wp = head.shape[1]
        if hidden.shape[-1] != wp:
            hidden = nn.functional.pad(hidden, (0, wp - hidden.shape[-1]))
        out = ops.linear(hidden.contiguous(), head)
        out = out[..., : self.dims.vocab_size].float()
        scale = self.dims.logit_scale
        return out if scale == 1.0 else out * scale

    @torch.no_grad()
    def decode_step(self, tokens, cache: LayeredCache, block_tables,
                    ctx_lens, slots=None) -> torch.Tensor:
        """One token for each of B sequences (ctx_lens counts it)."""
        from ..engine.step import StepBatch

        batch = StepBatch.decode(tokens, block_tables, ctx_lens, slots)
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
        slots = None
        if self.state_bytes_per_slot():
            slots = list(range(1, sum(1 for r in rows if r) + 1))
        cache = LayeredCache(self, sum(need) + 1, blk,
                             len(slots) + 1 if slots else 0)
        entries, at = [], 1
        for b, r in enumerate(rows):
            if r:
                entries.append((r, 0, list(range(at, at + need[b]))))
            at += need[b]
        out = torch.zeros(*input_ids.shape, self.dims.hidden_size,
                          dtype=self.dtype, device=self.device)
        if entries:
            batch = StepBatch.build(entries, blk, self.device, slots=slots)
            h = self.forward_step(batch, cache)
            order = torch.cat([torch.as_tensor(r) for r in batch.rows])
            out[mask] = h[order.to(self.device),
                          : self.dims.hidden_size]
        return out

    @property
    def device(self):
        return self.tok_emb.device

    @property
    def dtype(self):
        return self.tok_emb.dtype

    @property
    def embedding_size(self) -> int:
        return self.dims.hidden_size
