"""Op dispatch layer: hand-written HIP kernels on GPU, fp32 torch
reference on CPU.

Policy (required by the build rules): on a GPU tensor the HIP extension
is the ONLY path — if its module failed to import, GPU calls raise
immediately instead of silently falling back to eager PyTorch. CPU
tensors use distllm_amd.ops.torch_ref (fp32), which also serves as the
numerics ground truth in tests.
"""

from __future__ import annotations

import math

import torch

from . import torch_ref
from .native import Native

# One namespace over the built extension modules (native.py).
_hip_ops = Native()
HAVE_HIP = not _hip_ops.errors
_HIP_ERR: Exception | None = next(iter(_hip_ops.errors.values()), None)


def _require_hip(name: str = "_hip_ops"):
    _hip_ops.require(name)


# Activation codes shared with csrc/gemm.hip
ACT_NONE, ACT_GELU_TANH, ACT_GELU_ERF, ACT_SILU = 0, 1, 2, 3


def norm_fwd(x, res=None, w=None, b=None, eps=1e-5, rms=False):
    if x.is_cuda:
        _require_hip()
        return _hip_ops.norm_fwd(x, res, w, b, None, eps, rms)
    return torch_ref.norm_fwd(x, res, w, b, eps, rms)


def norm_fwd_sum(x, res, w, b=None, eps=1e-5, rms=False):
    """Fused (x+res) -> norm; returns (normed, x+res). Replaces the
    separate residual-add elementwise pass in pre-norm decoders."""
    if x.is_cuda:
        _require_hip()
        summed = torch.empty_like(x)
        out = _hip_ops.norm_fwd(x, res, w, b, summed, eps, rms)
        return out, summed
    return torch_ref.norm_fwd(x, res, w, b, eps, rms, return_sum=True)


def layer_norm(x, w, b, eps=1e-12, res=None):
    return norm_fwd(x, res=res, w=w, b=b, eps=eps, rms=False)


def rms_norm(x, w, eps=1e-5, res=None):
    return norm_fwd(x, res=res, w=w, b=None, eps=eps, rms=True)


def bias_gelu(x, bias=None, erf=False):
    if x.is_cuda:
        _require_hip()
        return _hip_ops.bias_gelu(x, bias, erf)
    return torch_ref.bias_gelu(x, bias, erf)


def swiglu(gate, up):
    if gate.is_cuda:
        _require_hip()
        return _hip_ops.swiglu(gate.contiguous(), up.contiguous())
    return torch_ref.swiglu(gate, up)


def bias_add(x, bias):
    if x.is_cuda:
        _require_hip()
        return _hip_ops.bias_add(x, bias)
    return torch_ref.bias_add(x, bias)


def mean_pool(hidden, mask, normalize=False):
    mask = mask.int()
    if hidden.is_cuda:
        _require_hip()
        return _hip_ops.mean_pool(hidden.contiguous(), mask.contiguous(),
                                  normalize)
    return torch_ref.mean_pool(hidden, mask, normalize)


def last_token_pool(hidden, mask, left_padded=False, normalize=False):
    mask = mask.int()
    if hidden.is_cuda:
        _require_hip()
        return _hip_ops.last_token_pool(hidden.contiguous(), mask.contiguous(),
                                        left_padded, normalize)
    return torch_ref.last_token_pool(hidden, mask, left_padded, normalize)


def l2_normalize(x):
    if x.is_cuda:
        _require_hip()
        return _hip_ops.l2_normalize(x.float().contiguous())
    return torch_ref.l2_normalize(x)


def adjacent_cosine(emb):
    if emb.is_cuda:
        _require_hip()
        return _hip_ops.adjacent_cosine(emb.float().contiguous())
    return torch_ref.adjacent_cosine(emb)


def gemm(A, B, bias=None, act=ACT_NONE):
    """C = A @ B^T via the hand-written MFMA kernel (GPU, padded shapes)
    or fp32 reference (CPU)."""
    if A.is_cuda:
        _require_hip("_hip_gemm")
        return _hip_ops.gemm_bf16(A, B, bias, act)
    return torch_ref.gemm(A, B, bias, act)


_GEMM_CHOICE: dict[tuple, str] = {}


def _blaslt_path(x2, weight, bias, act):
    out = torch.nn.functional.linear(x2, weight, bias)
    if act == ACT_GELU_TANH:
        out = bias_gelu(out, None, erf=False)
    elif act == ACT_GELU_ERF:
        out = bias_gelu(out, None, erf=True)
    elif act == ACT_SILU:
        out = (
            torch.nn.functional.silu(out.float()).to(out.dtype)
            if not out.is_cuda else _silu_gpu(out)
        )
    return out


def _blt_fused_path(x2, weight, bias, act):
    """ONE hipBLASLt call with the bias/GELU/swish applied in the GEMM
    epilogue — no separate elementwise pass over the [M, N] output."""
    epi = (1 if act in (ACT_GELU_TANH, ACT_GELU_ERF)
           else 2 if act == ACT_SILU else 0)
    return _hip_ops.blt_linear(x2, weight, bias, epi)


def _autotune_gemm(x2, weight, bias, act):
    """Measure hipBLASLt(+epilogue kernel) vs hipBLASLt-fused-epilogue
    vs the fused gemm8 MFMA kernel once per (M-bucket, N, K, act) and
    cache the winner."""
    import time as _t

    def timeit(fn):
        try:
            fn()
        except RuntimeError:
            return float("inf")
        torch.cuda.synchronize()
        t0 = _t.perf_counter()
        for _ in range(5):
            fn()
        torch.cuda.synchronize()
        return _t.perf_counter() - t0

    times = {
        "blaslt": timeit(lambda: _blaslt_path(x2, weight, bias, act)),
        "gemm8": timeit(lambda: _hip_ops.gemm8_bf16(x2, weight, bias, act)),
        "blt_fused": timeit(lambda: _blt_fused_path(x2, weight, bias, act)),
    }
    if x2.shape[1] % 128 == 0:  # gemm16 needs K % 128 == 0
        times["gemm16"] = timeit(
            lambda: _hip_ops.gemm16_bf16(x2, weight, bias, act))
    return min(times, key=times.get)


def _decode_splitk(M, N, K):
    """SPLITK so (N/64)*SPLITK lands near the CU count (256-512):
    narrow projections (k/v heads) need deep K splits to fill the chip."""
    ncb = N // 64
    for sk in (16, 8, 4, 2, 1):
        if ncb * sk <= 512 and K % (64 * sk) == 0:
            return sk
    return 1


def linear(x, weight, bias=None, act=ACT_NONE):
    """Linear layer entry used by models. GPU path: autotuned choice
    between hipBLASLt (plain and fused-epilogue), the hand-written
    MFMA GEMMs (gemm8.hip, 8-phase gemm16.hip) and the skinny-M
    split-K decode GEMM (decode_gemm.hip) for M <= 256. Override with
    DISTLLM_GEMM=blaslt|gemm8|gemm16|decode."""
    import os

    orig_shape = x.shape
    x2 = x.reshape(-1, orig_shape[-1])
    M, K = x2.shape
    N = weight.shape[0]
    if x.is_cuda:
        _require_hip("_hip_gemm")
        mode = os.environ.get("DISTLLM_GEMM", "auto")
        if x2.dtype == torch.float32:  # true 32-bit products
            mode = "blaslt"
        if (mode != "blaslt" and act == ACT_NONE and M <= 256
                and N % 64 == 0 and K % 64 == 0 and x2.is_contiguous()):
            if mode == "decode":  # forced in-chain A/B (profiling)
                sk = _decode_splitk(M, N, K)
                out = _hip_ops.decode_gemm(x2, weight, bias, sk)
                return out.reshape(*orig_shape[:-1], N)
            # bucket by padded M so varying decode/prefill
            # batch sizes reuse one tuning decision
            key = ("dec", 128 if M <= 128 else 256, N, K,
                   bias is not None)
            choice = _GEMM_CHOICE.get(key)
            sk = _decode_splitk(M, N, K)
            if choice is None:
                import time as _t

                def timeit(fn):
                    fn()
                    torch.cuda.synchronize()
                    t0 = _t.perf_counter()
                    for _ in range(10):
                        fn()
                    torch.cuda.synchronize()
                    return _t.perf_counter() - t0

                times = {
                    "blaslt": timeit(lambda: torch.nn.functional.linear(
                        x2, weight, bias)),
                    "decode": timeit(lambda: _hip_ops.decode_gemm(
                        x2, weight, bias, sk)),
                }
                try:  # hipBLASLt with measured algo search (blt_gemm.cpp)
                    times["blt_fused"] = timeit(
                        lambda: _blt_fused_path(x2, weight, bias, act))
                except RuntimeError:
                    pass
                choice = min(times, key=times.get)
                _GEMM_CHOICE[key] = choice
            if choice == "decode":
                out = _hip_ops.decode_gemm(x2, weight, bias, sk)
            elif choice == "blt_fused":
                out = _blt_fused_path(x2, weight, bias, act)
            else:
                out = torch.nn.functional.linear(x2, weight, bias)
            return out.reshape(*orig_shape[:-1], N)
        shapes_ok = (M % 256 == 0 and N % 256 == 0 and K % 64 == 0
                     and x2.is_contiguous())
        if shapes_ok and mode != "blaslt":
            if mode == "gemm8":
                out = _hip_ops.gemm8_bf16(x2, weight, bias, act)
            elif mode == "gemm16":
                out = _hip_ops.gemm16_bf16(x2, weight, bias, act)
            else:  # auto
                # coarse bucket above 16k rows: packed varlen batches
                # produce a different M per batch, and a fresh
                # 4-implementation autotune probe per distinct M
                # (~100ms each) dominated the semantic-chunk pipeline
                key = ("big" if M >= 16384 else M // 4096, N, K, act)
                choice = _GEMM_CHOICE.get(key)
                if choice is None:
                    choice = _autotune_gemm(x2, weight, bias, act)
                    _GEMM_CHOICE[key] = choice
                if choice == "gemm8":
                    out = _hip_ops.gemm8_bf16(x2, weight, bias, act)
                elif choice == "gemm16":
                    out = _hip_ops.gemm16_bf16(x2, weight, bias, act)
                elif choice == "blt_fused":
                    out = _blt_fused_path(x2, weight, bias, act)
                else:
                    out = _blaslt_path(x2, weight, bias, act)
        else:
            out = _blaslt_path(x2, weight, bias, act)
    else:
        out = _blaslt_path(x2, weight, bias, act)
    return out.reshape(*orig_shape[:-1], N)


def _silu_gpu(x):
    # standalone silu via the swiglu kernel with up=1 is wasteful; use a
    # dedicated path: silu(x) = swiglu(x, ones) avoided — bias_gelu
    # kernel family does not cover silu alone, so fall back to torch for
    # this rare case (plain silu without mul is not on any hot path).
    return torch.nn.functional.silu(x)


def attn_fwd(Q, K, V, mask=None, causal=False, scale=None):
    D = Q.shape[-1]
    if scale is None:
        scale = 1.0 / math.sqrt(D)
    if Q.is_cuda:
        _require_hip()
        if D not in (64, 128):
            # head_dim not natively tiled (e.g. small ESM2 variants,
            # D=16/24/32/96): zero-pad to the next native width — exact,
            # since padded dims add 0 to QK^T and produce 0 in O.
            Dp = 64 if D < 64 else 128
            pad = Dp - D
            Qp = torch.nn.functional.pad(Q, (0, pad))
            Kp = torch.nn.functional.pad(K, (0, pad))
            Vp = torch.nn.functional.pad(V, (0, pad))
            O = _hip_ops.attn_fwd(
                Qp, Kp, Vp,
                mask.contiguous() if mask is not None else None,
                causal, scale,
            )
            return O[..., :D].contiguous()
        if Q.stride(-1) != 1 or Q.stride(-2) != D:
            Q = Q.contiguous()
        if K.stride(-1) != 1 or K.stride(-2) != D:
            K = K.contiguous()
        if (V.stride(-1) != 1 or V.stride(-2) != D
                or V.stride(0) != K.stride(0) or V.stride(1) != K.stride(1)):
            V = V.contiguous()
            K = K.contiguous()
        return _hip_ops.attn_fwd(Q, K, V,
                                 mask.contiguous() if mask is not None else None,
                                 causal, scale)
    return torch_ref.attn_fwd(Q, K, V, mask, causal, scale)


def ivf_score(slabs, lens, probes, q):
    """Batched IVF chunk scoring: slabs [nchunks, cap, H] f32, lens
    [nchunks] i32, probes [Q, nprobe] i32, q [Q, H] f32 ->
    [Q, nprobe, cap] f32 (-inf at pad rows)."""
    _require_hip()
    return _hip_ops.ivf_score(slabs, lens, probes, q.contiguous())


def varlen_block_map(cu_seqlens: torch.Tensor, qblk: int = 128):
    """Host-built (seq, qblock) map for attn_varlen: one entry per
    128-row q block of each sequence. cu_seqlens int32 [B+1] (either
    device). Returns (blk_seq, blk_qb) int32 on cu's device."""
    cu = cu_seqlens.to("cpu", torch.int64)
    lens = cu[1:] - cu[:-1]
    nqb = torch.div(lens + qblk - 1, qblk, rounding_mode="floor")
    total = int(nqb.sum())
    blk_seq = torch.repeat_interleave(
        torch.arange(len(lens), dtype=torch.int64), nqb
    )
    # vectorized within-sequence block index: position minus the
    # sequence's first position
    starts = torch.zeros(len(lens), dtype=torch.int64)
    if len(lens) > 1:
        starts[1:] = nqb.cumsum(0)[:-1]
    blk_qb = (torch.arange(total, dtype=torch.int64)
              - torch.repeat_interleave(starts, nqb))
    dev = cu_seqlens.device
    return blk_seq.int().to(dev), blk_qb.int().to(dev)


def attn_varlen(Q, K, V, cu_seqlens, block_map=None, scale=None):
    """Varlen (packed, cu_seqlens) bidirectional attention.
    Q/K/V [total_tokens, H(KV), D]; returns [total_tokens, H, D].
    The protein-path replacement for faesm's flash-attn varlen
    (reference distllm/embed/encoders/esm2.py:41-55)."""
    D = Q.shape[-1]
    if scale is None:
        scale = 1.0 / math.sqrt(D)
    if Q.is_cuda:
        _require_hip()
        if block_map is None:
            block_map = varlen_block_map(cu_seqlens)
        blk_seq, blk_qb = block_map
        if D not in (64, 128):
            Dp = 64 if D < 64 else 128
            pad = Dp - D
            O = _hip_ops.attn_varlen(
                torch.nn.functional.pad(Q, (0, pad)).contiguous(),
                torch.nn.functional.pad(K, (0, pad)).contiguous(),
                torch.nn.functional.pad(V, (0, pad)).contiguous(),
                cu_seqlens.int(), blk_seq, blk_qb, scale)
            return O[..., :D].contiguous()
        return _hip_ops.attn_varlen(Q.contiguous(), K.contiguous(),
                                    V.contiguous(), cu_seqlens.int(),
                                    blk_seq, blk_qb, scale)
    return torch_ref.attn_varlen(Q, K, V, cu_seqlens, scale)


def rope_apply(x, cs, sn, pos, rope_heads: int = -1):
    """Heads >= rope_heads (when >= 0) pass through unchanged — lets a
    fused qkv tensor rope its q|k heads and copy v in ONE launch."""
    if x.is_cuda:
        _require_hip()
        return _hip_ops.rope_apply(x.contiguous(), cs, sn, pos.int(),
                                   rope_heads)
    return torch_ref.rope_apply(x, cs, sn, pos, rope_heads)


def gateup_swiglu(x, wgup, bias=None):
    """silu(x @ Wg^T) * (x @ Wu^T) with Wg|Wu packed as wgup [2I, K].
    Decode path (M <= 256): ONE split-K GEMM with the swiglu fused into
    its reduce; otherwise one big GEMM + packed swiglu."""
    orig_shape = x.shape
    x2 = x.reshape(-1, orig_shape[-1])
    M, K = x2.shape
    I = wgup.shape[0] // 2
    if x.is_cuda:
        _require_hip("_hip_gemm")
        if M <= 256 and wgup.shape[0] % 128 == 0 and x2.is_contiguous():
            sk = _decode_splitk(M, wgup.shape[0], K)
            if sk > 1:
                out = _hip_ops.decode_gemm(x2, wgup, bias, sk, 1)
                return out.reshape(*orig_shape[:-1], I)
    gu = linear(x2, wgup, bias)
    if gu.is_cuda:
        out = _hip_ops.swiglu_packed(gu.contiguous())
    else:
        out = swiglu(gu[:, :I], gu[:, I:])
    return out.reshape(*orig_shape[:-1], I)


def gateup_clamped_glu(x, wgup, limit, alpha, shift):
    """Clamped gated unit of x @ Wg^T and x @ Wu^T, Wg|Wu packed as wgup
    [2I, K]: min(g, limit) * sigmoid(alpha * g) * (clamp(u) + shift), all
    with the clamped g. Decode-sized inputs fuse it into the split-K
    reduce of ONE GEMM, as gateup_swiglu does."""
    M, K = x.shape
    if x.is_cuda:
        _require_hip("_hip_gemm")
        if (M <= 256 and x.dtype == torch.bfloat16 and K % 64 == 0
                and wgup.shape[0] % 128 == 0):
            sk = _decode_splitk(M, wgup.shape[0], K)
            if sk > 1:
                return _hip_ops.decode_gemm(x, wgup, None, sk, 2, limit,
                                            alpha, shift)
        return _hip_ops.clamped_glu(linear(x, wgup), limit, alpha, shift)
    return torch_ref.clamped_glu(linear(x, wgup), limit, alpha, shift)


def quantize_fp8_rows(w: torch.Tensor):
    """Per-output-channel OCP fp8-e4m3 weight quantization for the
    W8A16 decode GEMV: returns (wq uint8 [N, K], scale f32 [N]) with
    scale = absmax/448 so dequant is wq * scale per row."""
    wf = w.detach().float()
    scale = (wf.abs().amax(1) / 448.0).clamp_min(1e-12)
    q = (wf / scale[:, None]).clamp(-448.0, 448.0)
    q = q.to(torch.float8_e4m3fn).view(torch.uint8)
    return q.contiguous(), scale.contiguous()


def gemv_fp8(x, wq, scale, bias=None):
    """out = x @ (dequant(wq) * scale)^T (+bias). x bf16 [M<=8, K],
    wq uint8 fp8-e4m3 [N, K], scale f32 [N]. One wave per output
    column; the fp32 dot runs on the quantized values, the channel
    scale applies after — see csrc/gemv_fp8.hip."""
    _require_hip()
    return _hip_ops.gemv_fp8(x.contiguous(), wq, scale, bias)


rope_tables = torch_ref.rope_tables


def topk(scores, k, chunk=1 << 15):
    """Row-wise top-k over a [Q, N] f32 score matrix.

    GPU: chunked radix-select kernel + candidate-merge round. The
    32k default chunk keeps the grid >= 1024 workgroups even for a few
    queries (the chip needs >> 256 workgroups to fill).
    Returns (values [Q,k] f32 desc-sorted, indices [Q,k] int32).
    """
    if scores.is_cuda:
        _require_hip()
        Q, N = scores.shape
        k_eff = min(k, N)
        v, i = _hip_ops.topk_chunked(scores.contiguous(), None, k_eff, chunk)
        if v.shape[1] > k_eff:  # merge candidates from multiple chunks
            v2, i2 = _hip_ops.topk_chunked(v.contiguous(), i.contiguous(),
                                           k_eff, v.shape[1])
            v, i = v2, i2
        if k_eff < k:
            pad_v = torch.full((Q, k - k_eff), float("-inf"),
                               device=v.device)
            pad_i = torch.full((Q, k - k_eff), -1, dtype=torch.int32,
                               device=v.device)
            v = torch.cat([v, pad_v], 1)
            i = torch.cat([i, pad_i], 1)
        return v[:, :k], i[:, :k]
    return torch_ref.topk(scores, min(k, scores.shape[1]))


def hamming_score(qcodes, codes_t):
    if qcodes.is_cuda:
        _require_hip()
        return _hip_ops.hamming_score(qcodes.contiguous(),
                                      codes_t.contiguous())
    return torch_ref.hamming_score(qcodes, codes_t)


def sample_tokens(logits, rand, temp, min_p=0.0):
    if logits.is_cuda:
        _require_hip()
        return _hip_ops.sample_tokens(logits.float().contiguous(),
                                      rand.float(), temp, min_p)
    return torch_ref.sample_tokens(logits, rand, temp, min_p)


def paged_attn(q, kcache, vcache, block_table, ctx_len, scale=None):
    if scale is None:
        scale = 1.0 / math.sqrt(q.shape[-1])
    if q.is_cuda:
        _require_hip()
        return _hip_ops.paged_attn(q.contiguous(), kcache, vcache,
                                   block_table.int(), ctx_len.int(), scale)
    return torch_ref.paged_attn(q, kcache, vcache, block_table, ctx_len,
                                scale)


def cache_put(knew, vnew, kcache, vcache, block_table, slot):
    if knew.is_cuda:
        _require_hip()
        _hip_ops.cache_put(knew.contiguous(), vnew.contiguous(), kcache,
                           vcache, block_table.int(), slot.int())
        return
    # CPU reference: scatter
    B, HKV, D = knew.shape
    BLK = kcache.shape[2]
    for b in range(B):
        pos = int(slot[b])
        blk = int(block_table[b, pos // BLK])
        kcache[blk, :, pos % BLK] = knew[b]
        vcache[blk, :, pos % BLK] = vnew[b]


# ---- sandwich-norm / latent-attention decoder -----------------------------

def embed_norm(tokens, table, w_next, n, eps):
    """Start of the residual stream: x = table[token] in fp32 and h =
    rms(x) * w_next, statistics over the first n columns. -> (h, x)"""
    if table.is_cuda:
        _require_hip("_hip_residual")
        x = torch.empty(tokens.shape[0], table.shape[1],
                        dtype=torch.float32, device=table.device)
        h = _hip_ops.sandwich_norm(table, tokens, x, None, w_next, n, eps)
        return h, x
    return torch_ref.embed_norm(tokens, table, w_next, n, eps)


def post_norm_add(y, x, w_post, w_next, n, eps):
    """End of a sandwich-normed sublayer: x += rms(y) * w_post (x fp32,
    in place), returns the next sublayer's input rms(x) * w_next."""
    if y.is_cuda:
        _require_hip("_hip_residual")
        return _hip_ops.sandwich_norm(y, None, x, w_post, w_next, n, eps)
    return torch_ref.post_norm_add(y, x, w_post, w_next, n, eps)


def latent_prep(ab, q_cols, q_rank, rank, wq, wc, eps, cache, block_table,
                row_seq, ctx):
    """Norm both down-projections of a latent-attention layer in one
    launch: the query latent (first q_cols columns of ab) is returned,
    the key/value latent goes straight to its cache slot (position
    ctx - 1 of block-table row row_seq; ctx 0 writes nothing). cache
    None: the layer has no latent of its own."""
    if ab.is_cuda:
        _require_hip("_hip_latent")
        return _hip_ops.latent_prep(ab, q_cols, q_rank, rank, wq, wc, eps,
                                    cache, block_table, row_seq, ctx)
    return torch_ref.latent_prep(ab, q_cols, q_rank, rank, wq, wc, eps,
                                 cache, block_table, row_seq, ctx)


def rotary_latent_prep(ab, heads, dp, tp, rank, wc, eps, table, cache,
                       block_table, row_seq, ctx, ql):
    """What precedes latent attention with rotated parts, on a projection
    ab [M, heads * (dp unrotated, tp rotated numbers) | latent | key part |
    ...], in one launch: the rotated numbers of the queries of the first
    len(ql) rows go to the last tp columns of ql [n, heads, latent + tp],
    those of the others back to ab; normed latents (statistics over rank
    numbers) and rotated key parts go to their cache rows (position ctx - 1;
    ctx 0 writes nothing). cache None: the layer has none of its own."""
    if ab.is_cuda:
        _require_hip("_hip_latent")
        _hip_ops.rotary_latent_prep(ab, heads, dp, tp, rank, wc, eps, table,
                                    cache, block_table, row_seq, ctx, ql)
        return
    torch_ref.rotary_latent_prep(ab, heads, dp, tp, rank, wc, eps, table,
                                 cache, block_table, row_seq, ctx, ql)


def latent_gather(cache, block_table, key_seq, key_pos, rank=None):
    """Cached latents of (sequence, position) pairs, packed. With rank
    (fewer columns than a cache row has): the first rank columns and the
    others, as two tensors."""
    if cache.is_cuda:
        _require_hip("_hip_latent")
        c, rest = _hip_ops.latent_gather(cache, block_table, key_seq,
                                         key_pos, rank or cache.shape[2])
        return c if rank is None else (c, rest)
    c = torch_ref.latent_gather(cache, block_table, key_seq, key_pos)
    return c if rank is None else (c[:, :rank].contiguous(),
                                   c[:, rank:].contiguous())


def head_gemm(x, w, out=None):
    """One product per head: x [M, H, K], w [H, N, K] -> [M, H, N]. Rows
    and heads of x and out may be strided."""
    if x.is_cuda and x.dtype == torch.bfloat16:
        _require_hip("_hip_latent")
        if out is None:
            out = x.new_empty(x.shape[0], x.shape[1], w.shape[1])
        _hip_ops.head_gemm(x, w, out)
        return out
    if x.is_cuda:  # true 32-bit product
        res = torch.bmm(x.transpose(0, 1), w.transpose(1, 2))
        res = res.transpose(0, 1).contiguous()
    else:
        res = torch_ref.head_gemm(x, w)
    if out is None:
        return res
    return out.copy_(res)


def latent_attn(q, cache, block_table, row_seq, ctx, window, scale,
                nsplit=0, rank=None, sink=None, gate=None):
    """Attention of single-token rows over paged latents, queries folded
    into the latent space: q [M, H, R] -> [M, H, R]. A row sees the last
    `window` positions of its sequence up to its own (ctx - 1). nsplit:
    workgroups that share a row's keys (0: chosen from the sizes). With
    rank, only the first rank columns of a cache row are the value. sink
    [H]: exp(sink) is part of the softmax's denominator; gate [M, H]: head
    outputs are multiplied by its sigmoid."""
    rank = rank or cache.shape[2]
    if q.is_cuda:
        _require_hip("_hip_latent")
        return _hip_ops.latent_attn(q, cache, block_table, row_seq, ctx,
                                    window, scale, nsplit, rank, sink, gate)
    return torch_ref.latent_attn(q, cache, block_table, row_seq, ctx,
                                 window, scale, rank, sink, gate)


def attn_window(q, kv, out, cu_q, cu_k, block_map, window, scale, kr=None,
                sink=None, gate=None):
    """Sliding-window causal attention of packed queries that are the
    last ones of their packed keys (a prompt portion after its cached
    part). q [Tq, H, DK], kv [Tk, H*DK + H*DV], out [Tq, H, DV]. With kr
    [Tk, DR], key numbers that all heads share, queries have DK + DR
    numbers. sink, gate: as for latent_attn."""
    if q.is_cuda:
        _require_hip("_hip_latent")
        blk_seq, blk_qb = block_map
        _hip_ops.attn_window(q, kv, out, cu_q, cu_k, blk_seq, blk_qb,
                             window, scale, kr, sink, gate)
        return out
    return out.copy_(torch_ref.attn_window(q, kv, out.shape[2], cu_q, cu_k,
                                           window, scale, kr, sink, gate))


# ---- chunked attention / delta rule / experts decoder -----------------------

def embed_positions(tokens, ctx, table, pos):
    """Start of a residual stream with position vectors: x = table[token]
    + pos[ctx - 1] in fp32. -> (x in the table's dtype, x)"""
    if table.is_cuda:
        _require_hip("_hip_residual")
        x = torch.empty(tokens.shape[0], table.shape[1],
                        dtype=torch.float32, device=table.device)
        return _hip_ops.embed_positions(tokens, ctx, table, pos, x), x
    return torch_ref.embed_positions(tokens, ctx, table, pos)


def layer_norm_add(y, x, w, b, n, eps, final=None, mix=None):
    """End of a sublayer whose output is layer-normed: x += norm(y) (x
    fp32, in place; statistics over n columns). Returns x in y's dtype,
    normed by final = (weight, bias) if given. With mix [M, top] the
    sublayer output is sum_k mix[m, k] * y[m * top + k]."""
    if y.is_cuda:
        _require_hip("_hip_residual")
        wf, bf = final if final is not None else (None, None)
        return _hip_ops.layer_norm_add(y, x, w, b, n, eps, wf, bf, mix)
    return torch_ref.layer_norm_add(y, x, w, b, n, eps, final, mix)


def attn_prep(ab, heads, kv_heads, dp, vp, dim, wq, wk, eps, pages,
              block_table, row_seq, ctx):
    """Norm the query heads of a fused projection (returned, [M, heads,
    dp]) and its key heads, and write keys and values to their pages
    (position ctx - 1; ctx 0 writes nothing). pages None: the layer has
    no keys and values of its own."""
    if ab.is_cuda:
        _require_hip("_hip_hybrid")
        kp, vpg = pages if pages is not None else (None, None)
        return _hip_ops.attn_prep(ab, heads, kv_heads, dp, vp, dim, wq, wk,
                                  eps, kp, vpg, block_table, row_seq, ctx)
    return torch_ref.attn_prep(ab, heads, kv_heads, dp, vp, dim, wq, wk, eps,
                               pages, block_table, row_seq, ctx)


def paged_attn_rows(q, kpages, vpages, ab, gate_at, out, block_table,
                    row_seq, ctx, chunk, scale, softcap, dist, nsplit=0):
    """Attention of single-token rows over paged keys and values. A row
    sees the positions of its chunk up to its own. The output is gated by
    the sigmoid of ab's columns from gate_at on."""
    if q.is_cuda:
        _require_hip("_hip_chunked")
        _hip_ops.paged_attn_rows(q, kpages, vpages, ab, gate_at, out,
                                 block_table, row_seq, ctx, chunk, scale,
                                 softcap, dist, nsplit)
        return out
    return torch_ref.paged_attn_rows(q, kpages, vpages, ab, gate_at, out,
                                     block_table, row_seq, ctx, chunk, scale,
                                     softcap, dist)


def paged_attn_prompts(q, kpages, vpages, ab, gate_at, out, block_table,
                       prompts, chunk, scale, softcap, dist):
    """The same for the rows of prompt portions (step.PromptBlocks)."""
    if q.is_cuda:
        _require_hip("_hip_chunked")
        _hip_ops.paged_attn_prompts(q, kpages, vpages, ab, gate_at, out,
                                    block_table, prompts.portions,
                                    prompts.blocks, chunk, scale, softcap,
                                    dist)
        return out
    return torch_ref.paged_attn_prompts(q, kpages, vpages, ab, gate_at, out,
                                        block_table, prompts, chunk, scale,
                                        softcap, dist)


def gated_delta(ab, heads, kv_heads, dp, vp, dim, vdim, conv_w, decay,
                o_norm, unit_eps, eps, state, conv, segments, row_seq, ctx):
    """Gated delta rule of a ragged step on the fused projection ab
    [M, queries | keys | values | gates | b | a]: short convolutions, unit
    queries and keys, recurrence in fp32, gated output norm.
    -> [M, heads * vp]; state and convolution slots are updated."""
    if ab.is_cuda:
        _require_hip("_hip_hybrid")
        return _hip_ops.gated_delta(
            ab, heads, kv_heads, dp, vp, dim, vdim, conv_w, decay, o_norm,
            unit_eps, eps, state, conv, segments.row0, segments.rows,
            segments.slot, segments.longest, row_seq, ctx, segments.longs,
            segments.chunks, segments.SHORT)
    return torch_ref.gated_delta(
        ab, heads, kv_heads, dp, vp, dim, vdim, conv_w, decay, o_norm,
        unit_eps, eps, state, conv, segments, row_seq, ctx)


def up_xielu(x, wup, act):
    """xielu(x @ wup^T); act: the activation's two raw numbers."""
    M, K = x.shape
    if x.is_cuda:
        _require_hip("_hip_gemm")
        _require_hip("_hip_experts")
        if (M <= 256 and x.dtype == torch.bfloat16 and K % 64 == 0
                and wup.shape[0] % 64 == 0):
            sk = _decode_splitk(M, wup.shape[0], K)
            if sk > 1:
                return _hip_ops.decode_gemm(x, wup, None, sk, 3,
                                            act_nums=act)
        return _hip_ops.xielu(linear(x, wup), act)
    return torch_ref.xielu(linear(x, wup), act)


def route(h, router, ctx, top, groups, keep):
    """Experts of every row: ids [M, top] int32 and their softmax scores.
    Only experts of the `keep` groups with the largest scores count; rows
    with ctx 0 get ids -1 and weights 0."""
    if h.is_cuda:
        _require_hip("_hip_experts")
        if h.dtype == torch.bfloat16 and router.shape[0] <= 256:
            return _hip_ops.route(h, router, ctx, top, groups, keep)
        logits = torch.nn.functional.linear(h.float(), router.float())
        return _hip_ops.route(logits, None, ctx, top, groups, keep)
    return torch_ref.route(h, router, ctx, top, groups, keep)


def experts(h, ids, wup, wdown, gated=True):
    """Experts: row m * top + k of the result is expert ids[m, k] of row m
    (undefined for id -1). Gated units, wup [E, 2F, W]: gate and up rows
    alternate in groups of 16; else squared ReLU, wup [E, F, W]."""
    if h.is_cuda:
        _require_hip("_hip_experts")
        return _hip_ops.experts(h, ids, wup, wdown, gated)
    return torch_ref.experts(h, ids, wup, wdown, gated)


def route_sigmoid(h, router, correction, ctx, top, scale, shards=0):
    """Experts of every row by sigmoid scores: ids [M, top] int32 of the
    largest sums of score and correction, and scale times their scores
    without it. One more row of the router than corrections is the gate of
    an expert that serves every row: its sigmoid is a further column of the
    weights, or, with shards, the weight of that many further choices, the
    experts behind the others. Rows with ctx 0 get ids -1 and weights 0."""
    if h.is_cuda:
        _require_hip("_hip_experts")
        if h.dtype == torch.bfloat16 and router.shape[0] <= 256:
            return _hip_ops.route_sigmoid(h, router, correction, ctx, top,
                                          scale, shards)
        logits = torch.nn.functional.linear(h.float(), router.float())
        return _hip_ops.route_sigmoid(logits, None, correction, ctx, top,
                                      scale, shards)
    return torch_ref.route_sigmoid(h, router, correction, ctx, top, scale,
                                   shards)


def up_relu2(x, wup):
    """The square of relu(x @ wup^T)."""
    M, K = x.shape
    if x.is_cuda:
        _require_hip("_hip_gemm")
        if (M <= 256 and x.dtype == torch.bfloat16 and K % 64 == 0
                and wup.shape[0] % 64 == 0):
            sk = _decode_splitk(M, wup.shape[0], K)
            if sk > 1:
                return _hip_ops.decode_gemm(x, wup, None, sk, 5)
        return _hip_ops.relu2(linear(x, wup))
    return torch_ref.relu2(linear(x, wup))


# ---- parallel attention and delta rule / linear recurrent decoder -----------

def residual_step(x, y=None, bias=None, rms=None, embed=None, vec=None,
                  act=None, fresh=False, dtype=None):
    """One boundary of an fp32 residual stream x [M, W], in place:
      x += y + bias (fp32 vector), or rms(y) * w with rms = (w, n, eps),
           statistics over n columns
      x += scale * table[token] with embed = (tokens, table, scale)
      x += vec (fp32 vector)
    all of them optional; with `fresh` x starts from zeros. Returns x, or
    tanh(alpha x) * w + b with act = (w, b, alpha), in `dtype` (default:
    that of y, of the table without y)."""
    if dtype is None:
        dtype = y.dtype if y is not None else embed[1].dtype
    if x.is_cuda:
        _require_hip("_hip_residual")
        tokens, table, scale = embed if embed is not None else (None, None,
                                                                1.0)
        w_rms, n, eps = rms if rms is not None else (None, x.shape[1], 0.0)
        w, b, alpha = act if act is not None else (None, None, None)
        h = torch.empty(x.shape, dtype=dtype, device=x.device)
        _hip_ops.residual_step(x, y, bias, w_rms, n, eps, tokens, table,
                               scale, vec, w, b, alpha, fresh, h)
        return h
    return torch_ref.residual_step(x, y, bias, rms, embed, vec, act, fresh,
                                   dtype)


def gated_rows(x, wgate, tokens, table, col0, n):
    """gelu_tanh(x @ wgate^T) * table[token, col0: col0 + n], zeros in the
    columns of wgate behind n."""
    if x.is_cuda:
        _require_hip("_hip_gemm")
        M, K = x.shape
        if (M <= 256 and x.dtype == torch.bfloat16 and K % 64 == 0):
            sk = _decode_splitk(M, wgate.shape[0], K)
            if sk > 1:
                return _hip_ops.decode_gemm_rows(x, wgate, sk, tokens, table,
                                                 col0, n)
        return _hip_ops.gelu_rows(linear(x, wgate), tokens, table, col0, n)
    return torch_ref.gelu_rows(linear(x, wgate), tokens, table, col0, n)


def rotation_table(ctx, freq, mult):
    """mult * (cos, sin) of freq (fp64) times the position ctx - 1 of every
    row: [M, pairs, 2] fp32."""
    if ctx.is_cuda:
        _require_hip("_hip_residual")
        return _hip_ops.rotation_table(ctx, freq, mult)
    return torch_ref.rotation_table(ctx, freq, mult)


def rotary_prep(ab, heads, kv_heads, dp, dim, wq, wk, eps, table, pages,
                block_table, row_seq, ctx):
    """Norm and rotate the query heads of a projection ab [M, queries |
    keys] (returned, [M, heads, dp]) and its key heads; those go to the key
    pages, keys as projected to the value pages (position ctx - 1; ctx 0
    writes nothing). The first 2 * pairs numbers of a head rotate."""
    if ab.is_cuda:
        _require_hip("_hip_hybrid")
        return _hip_ops.rotary_prep(ab, heads, kv_heads, dp, dim, wq, wk,
                                    eps, table, pages[0], pages[1],
                                    block_table, row_seq, ctx)
    return torch_ref.rotary_prep(ab, heads, kv_heads, dp, dim, wq, wk, eps,
                                 table, pages, block_table, row_seq, ctx)


def sink_attn_rows(q, kpages, vpages, out, block_table, row_seq, ctx, scale,
                   sink, out_scale, nsplit=0):
    """Causal attention of single-token rows over paged keys and values;
    exp(sink) of the head is part of the softmax's denominator. out
    [M, heads * vdim] (rows may be strided) takes the result times
    out_scale."""
    if q.is_cuda:
        _require_hip("_hip_hybrid")
        _hip_ops.sink_attn_rows(q, kpages, vpages, out, block_table, row_seq,
                                ctx, scale, sink, out_scale, nsplit)
        return out
    return torch_ref.sink_attn_rows(q, kpages, vpages, out, block_table,
                                    row_seq, ctx, scale, sink, out_scale)


def sink_attn_prompts(q, kpages, vpages, out, block_table, prompts, scale,
                      sink, out_scale):
    """The same for the rows of prompt portions (step.PromptBlocks)."""
    if q.is_cuda:
        _require_hip("_hip_hybrid")
        _hip_ops.sink_attn_prompts(q, kpages, vpages, out, block_table,
                                   prompts.portions, prompts.blocks, scale,
                                   sink, out_scale)
        return out
    return torch_ref.sink_attn_prompts(q, kpages, vpages, out, block_table,
                                       prompts, scale, sink, out_scale)


def channel_delta(ab, ag, heads, kv_heads, dp, vp, dim, vdim, conv_w, a_log,
                  dt_bias, o_norm, unit_eps, eps, out_scale, state, conv,
                  segments, row_seq, ctx, out):
    """Delta rule with a decay per key channel of a ragged step, on the
    projection ab [M, queries | keys | values | b] and the second product
    ag [M, decays | gates]: short convolutions, unit queries and keys,
    recurrence in fp32, output norm, sigmoid gate, out_scale. out
    [M, heads * vp] (rows may be strided); state and convolution slots are
    updated."""
    if ab.is_cuda:
        _require_hip("_hip_hybrid")
        _hip_ops.channel_delta(
            ab, ag, heads, kv_heads, dp, vp, dim, vdim, conv_w, a_log,
            dt_bias, o_norm, unit_eps, eps, out_scale, state, conv,
            segments.row0, segments.rows, segments.slot, segments.longest,
            row_seq, ctx, segments.longs, segments.chunks, segments.SHORT,
            out)
        return out
    return torch_ref.channel_delta(
        ab, ag, heads, kv_heads, dp, vp, dim, vdim, conv_w, a_log, dt_bias,
        o_norm, unit_eps, eps, out_scale, state, conv, segments, row_seq,
        ctx, out)


def lru_gate_order(w):
    """Gate weights [.., out, in] in the order in which the MFMA takes them
    (32 outputs by 32 inputs at a time), in the same shape; sizes % 32."""
    n = w.shape[-1]
    t = w.reshape(-1, n // 32, 16, 2, n // 32, 4, 8)
    return t.permute(0, 1, 4, 3, 5, 2, 6).reshape(w.shape)


def gated_lru(ab, conv_w, conv_b, gates, gates_b, decay, state, conv,
              segments, row_seq, ctx, chunk):
    """Linear recurrent unit of a ragged step on the projection ab [M,
    GELU branch | recurrent branch]: convolution, block-diagonal gates,
    recurrence in fp32, times the GELU branch. -> [M, width]; state and
    convolution slots are updated. Long segments run in chunks of `chunk`
    rows."""
    if ab.is_cuda:
        _require_hip("_hip_lru")
        longs, chunks = segments.chunk_lists(chunk)
        return _hip_ops.gated_lru(
            ab, conv_w, conv_b, gates, gates_b, decay, state, conv,
            segments.row0, segments.rows, segments.slot, segments.longest,
            row_seq, ctx, longs, chunks, chunk, segments.SHORT)
    return torch_ref.gated_lru(ab, conv_w, conv_b, gates, gates_b, decay,
                               state, conv, segments, row_seq, ctx)


# ---- retention / rotary latent attention decoder on several streams ---------

def stream_step(x, y=None, writes=None, mix=None, shared=None, embed=None,
                read=None, norm=None, store=True, dtype=None):
    """One boundary of fp32 residual streams x [M, S, W], in place. With a
    sublayer's output y [M, W] and writes = (out [S], then the matrix mix,
    from-major), x_t becomes sum_s mix[s, t] x_s + out[t] y. With mix
    [M, top] (+ 1 column with shared [M, W]), y [M * top, W] is summed with
    these weights first. With embed = (tokens, table) every old stream is
    the token's row and x is not read; without `store` x is not written.
    Returns rms(sum_s read[s] x_s) * w (read None: the plain sum) with norm
    = (w, n, eps), statistics over n columns, in `dtype` (default: y's)."""
    w, n, eps = norm
    if dtype is None:
        dtype = y.dtype
    if x.is_cuda:
        _require_hip("_hip_residual")
        tokens, table = embed if embed is not None else (None, None)
        h = torch.empty(x.shape[0], x.shape[2], dtype=dtype, device=x.device)
        _hip_ops.stream_step(x, y, writes, mix, shared, tokens, table, read,
                             w, n, eps, store, h)
        return h
    return torch_ref.stream_step(x, y, writes, mix, shared, embed, read,
                                 norm, store, dtype)


def retention(ab, heads, dp, vp, dim, vdim, decay, table, eps, state,
              segments, ctx):
    """Linear attention with a fixed decay per head (decay [2, heads]: the
    decays, their base-2 logarithms) of a ragged step, on the projection
    ab [M, queries | keys | values | gates]: rotation by table, recurrence
    in fp32, heads normed over vdim and gated by silu. -> [M, heads * vp];
    the sequences' slots of state [slots, heads, vp, dp] are updated."""
    if ab.is_cuda:
        _require_hip("_hip_retention")
        return _hip_ops.retention(
            ab, heads, dp, vp, dim, vdim, decay, table, eps, state,
            segments.row0, segments.rows, segments.slot, ctx,
            *segments.pieces(heads), segments.SHORT)
    return torch_ref.retention(ab, heads, dp, vp, dim, vdim, decay, table,
                               eps, state, segments, ctx)
