"""Parts of decoders that are described layer by layer: what mixers and
feed-forwards have in common, and the latent-attention family.

A mixer maps the rows of a ragged step batch (engine/step.py) to the
sublayer's output and says what it keeps in the cache. Sizes of the
parameters are rounded up to multiples of 64 with zeros, so that the
16-byte loads and MFMA tiles of the kernels never see a partial row; the
zeros leave every product and (with the true sizes passed along) every
norm unchanged.

`tensors` names a part's checkpoint tensors with their (unpadded) shapes,
`checkpoint` maps them to the padded parameters.
"""

from __future__ import annotations

import torch
from torch import nn

from .. import ops
from .config import ClampedGluDims, LatentAttentionDims


def pad64(n: int) -> int:
    return (n + 63) // 64 * 64


def head_pad(n: int) -> int:
    """Head sizes of the packed-prompt attention kernel: 64, 128, 256."""
    for p in (64, 128, 256):
        if n <= p:
            return p
    return pad64(n)


def rank_pad(n: int) -> int:
    """Latent sizes of the MFMA decode kernel, or any multiple of 64."""
    for p in (64, 128, 192, 256, 384, 512):
        if n <= p:
            return p
    return pad64(n)


def padded(w: torch.Tensor, *shape: int) -> torch.Tensor:
    out = w.new_zeros(shape)
    out[tuple(slice(0, n) for n in w.shape)] = w
    return out


def padded_heads(w: torch.Tensor, heads: int, d: int, dp: int,
                 cols: int) -> torch.Tensor:
    """[heads * d, c] -> [heads * dp, cols]."""
    out = w.new_zeros(heads, dp, cols)
    out[:, :d, : w.shape[1]] = w.view(heads, d, -1)
    return out.view(heads * dp, cols)


def expect(name: str, w: torch.Tensor, *shape: int) -> torch.Tensor:
    if tuple(w.shape) != shape:
        raise ValueError(f"checkpoint weight {name} has shape "
                         f"{tuple(w.shape)}, the configuration says {shape}")
    return w


def weight(rows: int, cols: int, dtype) -> nn.Parameter:
    return nn.Parameter(torch.empty(rows, cols, dtype=dtype))


def norm_weight(n: int) -> nn.Parameter:
    # norms are computed in fp32 whatever the model's dtype
    return nn.Parameter(torch.empty(n, dtype=torch.float32))


class Part(nn.Module):
    """A mixer or feed-forward."""

    # a mixer that reads another layer's cache has none of its own
    own = True
    kv_from: int | None = None

    def tensors(self) -> dict[str, tuple[int, ...]]:
        """Checkpoint tensor name (within the part) -> its shape."""
        raise NotImplementedError

    def checkpoint(self, src: dict, pre: str) -> dict[str, torch.Tensor]:
        """Own parameter name -> padded tensor, from a raw checkpoint
        (`checked` has seen to the shapes)."""
        raise NotImplementedError

    def checked(self, src: dict, pre: str) -> dict[str, torch.Tensor]:
        return {n: expect(pre + n, src[pre + n], *shape)
                for n, shape in self.tensors().items()}

    def initial(self) -> dict[str, torch.Tensor]:
        """Checkpoint tensors whose values before training are not the
        usual ones."""
        return {}

    def cache_numel(self) -> int:
        """Numbers that a token keeps in the paged cache."""
        return 0

    def state_numel(self) -> tuple[int, int]:
        """Numbers of a state slot: in fp32, in the model's dtype."""
        return 0, 0

    def make_cache(self, num_blocks: int, blk: int, num_slots: int, dtype,
                   device):
        """What the layer keeps between steps."""
        return None


class Branch(Part):
    """A mechanism between an input and an output product, both of which
    may be shared with other branches (branches.py). It says which rows of
    the input product it wants and what its output columns are multiplied
    with, and fills its columns of the output product's input."""

    in_rows: int   # columns of the input product, padded
    out_cols: int  # columns given to the output product, padded

    def in_weight(self, t: dict) -> torch.Tensor:
        """[in_rows, padded width], from the branch's checked tensors."""
        raise NotImplementedError

    def in_bias(self, t: dict) -> torch.Tensor | None:
        return None

    def out_weight(self, t: dict) -> torch.Tensor:
        """[padded width, out_cols]"""
        raise NotImplementedError

    def out_bias(self, t: dict) -> torch.Tensor | None:
        return None

    def extra(self, t: dict) -> dict[str, torch.Tensor]:
        """The branch's own parameters."""
        raise NotImplementedError

    def run(self, ab, batch, cache, out, scale: float) -> None:
        """ab [M, in_rows]: the branch's columns of the input product;
        out [M, out_cols] takes its result, times `scale`."""
        raise NotImplementedError


class LatentAttention(Part):
    """Latent attention with a sliding window, on paged latents.

    Two forms of the same function:
      folded   queries are taken into the latent space (q' = Uk^T q) and
               every head reads the cached latent itself — single tokens
               and short portions, where reading the cache is the cost;
      expanded keys and values of the visible latents are formed by one
               product and attended by the flash kernel — long portions,
               where the score products are the cost.
    """

    def __init__(self, d: LatentAttentionDims, width: int, eps: float,
                 dtype):
        super().__init__()
        self.d, self.width, self.eps = d, width, eps
        self.wp = pad64(width)
        self.dp, self.vp = head_pad(d.dim), head_pad(d.vdim)
        self.qp, self.rp = pad64(d.q_rank), rank_pad(d.kv_rank)
        self.own = d.kv_from is None
        H = d.heads
        # one product for both down-projections of a layer
        self.wdown = weight(self.qp + (self.rp if self.own else 0),
                             self.wp, dtype)
        self.q_norm = norm_weight(self.qp)
        self.kv_norm = norm_weight(self.rp) if self.own else None
        self.wuq = weight(H * self.dp, self.qp, dtype)
        # all heads' key rows, then all heads' value rows
        self.wukv = weight(H * (self.dp + self.vp), self.rp, dtype)
        self.wo = weight(self.wp, H * self.vp, dtype)
        self._fold: tuple | None = None

    @property
    def kv_from(self):
        return self.d.kv_from

    def tensors(self):
        d, H, W = self.d, self.d.heads, self.width
        t = {"dq": (d.q_rank, W), "dq.norm": (d.q_rank,),
             "uq": (H * d.dim, d.q_rank)}
        if self.own:
            t |= {"dkv": (d.kv_rank, W), "dkv.norm": (d.kv_rank,)}
        return t | {"uk": (H * d.dim, d.kv_rank),
                    "uv": (H * d.vdim, d.kv_rank), "o": (W, H * d.vdim)}

    def checkpoint(self, src, pre):
        d, H = self.d, self.d.heads
        t = self.checked(src, pre)
        down = [padded(t["dq"], self.qp, self.wp)]
        out = {"q_norm": padded(t["dq.norm"], self.qp)}
        if self.own:
            down.append(padded(t["dkv"], self.rp, self.wp))
            out["kv_norm"] = padded(t["dkv.norm"], self.rp)
        out["wdown"] = torch.cat(down)
        out["wuq"] = padded_heads(t["uq"], H, d.dim, self.dp, self.qp)
        out["wukv"] = torch.cat([
            padded_heads(t["uk"], H, d.dim, self.dp, self.rp),
            padded_heads(t["uv"], H, d.vdim, self.vp, self.rp)])
        out["wo"] = padded_heads(t["o"].t(), H, d.vdim, self.vp, self.wp).t()
        return out

    def cache_numel(self):
        return self.rp if self.own else 0

    def make_cache(self, num_blocks, blk, num_slots, dtype, device):
        """Paged latents [blocks, BLK, rank]."""
        return torch.zeros(num_blocks, blk, self.rp, dtype=dtype,
                           device=device)

    def _folded(self) -> tuple[torch.Tensor, torch.Tensor]:
        """(Uk^T [H, R, dim], Uv [H, vdim, R]); Uk^T is a copy, renewed
        when the weights change."""
        w, H = self.wukv, self.d.heads
        key = (w.data_ptr(), w._version)
        if self._fold is None or self._fold[0] != key:
            uk = w[: H * self.dp].view(H, self.dp, self.rp)
            self._fold = (key, uk.detach().transpose(1, 2).contiguous())
        return self._fold[1], w[H * self.dp:].view(H, self.vp, self.rp)

    def expands(self) -> bool:
        """Whether the flash kernel covers this layer's dtype and sizes."""
        w = self.wuq
        return (max(self.dp, self.vp) <= 256
                and (w.dtype == torch.bfloat16 or not w.is_cuda))

    def forward(self, h, batch, latents):
        """h [M, width]; latents: the paged cache [blocks, BLK, rank] of
        the layer that owns it."""
        d, H = self.d, self.d.heads
        M = h.shape[0]
        bt, ctx = batch.block_table, batch.ctx
        ab = ops.linear(h, self.wdown)
        cq = ops.latent_prep(ab, self.qp, d.q_rank, d.kv_rank, self.q_norm,
                             self.kv_norm, self.eps,
                             latents if self.own else None, bt,
                             batch.row_seq, ctx)
        q = ops.linear(cq, self.wuq).view(M, H, self.dp)
        # leading rows folded, then the rows of expanded portions; padding
        # rows trail and count as folded ones that see nothing
        n = batch.n_folded if self.expands() else M
        if n == M:
            o = h.new_empty(M, H, self.vp)
        else:
            o = h.new_zeros(M, H, self.vp)
        if n > 0:
            uk_t, uv = self._folded()
            ql = ops.head_gemm(q[:n], uk_t)
            ol = ops.latent_attn(ql, latents, bt, batch.row_seq[:n],
                                 ctx[:n], d.window, d.scale)
            ops.head_gemm(ol, uv, out=o[:n])
        if n < M:
            e = batch.expansion(d.window)
            c = ops.latent_gather(latents, bt, e.key_seq, e.key_pos)
            kv = ops.linear(c, self.wukv)
            ops.attn_window(q[n:], kv, o[n:], e.cu_q, e.cu_k, e.block_map,
                            d.window, d.scale)
        return ops.linear(o.view(M, H * self.vp), self.wo)


class ClampedGlu(Part):
    def __init__(self, d: ClampedGluDims, width: int, dtype):
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
        return {
            "wgup": torch.cat([padded(t["gate"], self.fp, self.wp),
                               padded(t["up"], self.fp, self.wp)]),
            "wdown": padded(t["down"], self.wp, self.fp),
        }

    def forward(self, h):
        d = self.d
        return ops.linear(
            ops.gateup_clamped_glu(h, self.wgup, d.limit, d.alpha, d.shift),
            self.wdown)
