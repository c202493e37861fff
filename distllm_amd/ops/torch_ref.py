"""Plain-PyTorch fp32 reference implementations of every HIP op.

These are the ground truth for kernel numerics tests (GPU: HIP kernel vs
this in fp32) and the CPU execution path for the no-GPU test tier. They
define the op semantics exactly; the HIP kernels in csrc/ must match
within bf16 tolerance.
"""

from __future__ import annotations

import math

import torch
import torch.nn.functional as F


def norm_fwd(
    x: torch.Tensor,
    res: torch.Tensor | None,
    w: torch.Tensor,
    b: torch.Tensor | None,
    eps: float,
    rms: bool,
    return_sum: bool = False,
):
    xf = x.float()
    if res is not None:
        xf = xf + res.float()
    summed = xf
    if rms:
        inv = torch.rsqrt(xf.pow(2).mean(-1, keepdim=True) + eps)
        out = xf * inv * w.float()
        if b is not None:
            out = out + b.float()
    else:
        mean = xf.mean(-1, keepdim=True)
        var = xf.var(-1, unbiased=False, keepdim=True)
        out = (xf - mean) * torch.rsqrt(var + eps) * w.float()
        if b is not None:
            out = out + b.float()
    out = out.to(x.dtype)
    if return_sum:
        return out, summed.to(x.dtype)
    return out


def bias_gelu(x: torch.Tensor, bias: torch.Tensor | None, erf: bool = False):
    xf = x.float()
    if bias is not None:
        xf = xf + bias.float()
    out = F.gelu(xf) if erf else F.gelu(xf, approximate="tanh")
    return out.to(x.dtype)


def swiglu(gate: torch.Tensor, up: torch.Tensor):
    return (F.silu(gate.float()) * up.float()).to(gate.dtype)


def bias_add(x: torch.Tensor, bias: torch.Tensor):
    return (x.float() + bias.float()).to(x.dtype)


def mean_pool(hidden: torch.Tensor, mask: torch.Tensor, normalize: bool):
    """Masked mean excluding BOS (pos 0) and the last real token (pos L-1).

    Role of reference distllm/embed/poolers/mean.py:13-49, with ONE
    deliberate divergence: the reference's `attention_mask[:, L-1] = 0`
    uses a VECTOR column index, so for a mixed-length batch it zeroes
    the column at every row's length-1 across ALL rows (excluding
    interior tokens of longer rows). We exclude each row's OWN last
    real token only — the per-row behavior the reference intends
    ("Set the attention mask to 0 for start and end tokens"). Equal
    results for uniform-length batches.
    hidden [R, S, H]; mask [R, S] int -> [R, H] fp32.
    """
    hf = hidden.float()
    m = mask.clone().to(hf.dtype)
    L = mask.sum(dim=1).long()
    m[:, 0] = 0
    rows = torch.arange(m.size(0), device=m.device)
    last = (L - 1).clamp(min=0)
    m[rows, last] = 0
    summed = (hf * m.unsqueeze(-1)).sum(dim=1)
    count = m.sum(dim=1, keepdim=True).clamp(min=1)
    out = summed / count
    if normalize:
        out = F.normalize(out, p=2, dim=-1)
    return out


def last_token_pool(
    hidden: torch.Tensor, mask: torch.Tensor, left_padded: bool, normalize: bool
):
    """reference distllm/embed/poolers/last_token.py:12-38 semantics."""
    hf = hidden.float()
    R, S, H = hf.shape
    if left_padded:
        out = hf[:, -1]
    else:
        idx = (mask.sum(dim=1).long() - 1).clamp(min=0)
        out = hf[torch.arange(R, device=hf.device), idx]
    if normalize:
        out = F.normalize(out, p=2, dim=-1)
    return out


def l2_normalize(x: torch.Tensor):
    return F.normalize(x.float(), p=2, dim=-1)


def adjacent_cosine(emb: torch.Tensor):
    """reference embed/embedders/semantic_chunk.py:24-55: 1 - cosine of
    adjacent rows."""
    e = emb.float()
    if e.size(0) < 2:
        return torch.empty(0, dtype=torch.float32, device=e.device)
    a, b = e[:-1], e[1:]
    num = (a * b).sum(-1)
    den = a.norm(dim=-1).clamp(min=1e-15) * b.norm(dim=-1).clamp(min=1e-15)
    return 1.0 - num / den


def gemm(A: torch.Tensor, B: torch.Tensor, bias=None, act: int = 0):
    """C = A @ B^T (+bias) (+activation). act: 0 none, 1 gelu_tanh,
    2 gelu_erf, 3 silu."""
    C = A.float() @ B.float().t()
    if bias is not None:
        C = C + bias.float()
    if act == 1:
        C = F.gelu(C, approximate="tanh")
    elif act == 2:
        C = F.gelu(C)
    elif act == 3:
        C = F.silu(C)
    return C.to(A.dtype)


def attn_fwd(
    Q: torch.Tensor,
    K: torch.Tensor,
    V: torch.Tensor,
    mask: torch.Tensor | None,
    causal: bool,
    scale: float,
):
    """BSHD layout; mask f32 [B, SKV] additive; GQA by head repeat."""
    B, SQ, H, D = Q.shape
    SKV, HKV = K.shape[1], K.shape[2]
    q = Q.float().permute(0, 2, 1, 3)  # B H S D
    k = K.float().permute(0, 2, 1, 3)
    v = V.float().permute(0, 2, 1, 3)
    if HKV != H:
        rep = H // HKV
        k = k.repeat_interleave(rep, dim=1)
        v = v.repeat_interleave(rep, dim=1)
    s = (q @ k.transpose(-1, -2)) * scale  # B H SQ SKV
    if mask is not None:
        s = s + mask.float()[:, None, None, :]
    if causal:
        cm = torch.full((SQ, SKV), float("-inf"), device=s.device)
        cm = torch.triu(cm, diagonal=1)
        s = s + cm
    p = torch.softmax(s, dim=-1)
    p = torch.nan_to_num(p, nan=0.0)  # fully-masked rows -> 0
    o = p @ v
    return o.permute(0, 2, 1, 3).contiguous().to(Q.dtype)


def attn_varlen(Q, K, V, cu_seqlens, scale: float):
    """Packed [T, H(KV), D] varlen bidirectional attention reference:
    per-sequence slices through attn_fwd (fp32)."""
    cu = cu_seqlens.to("cpu", torch.int64).tolist()
    out = torch.empty_like(Q)
    for b in range(len(cu) - 1):
        lo, hi = cu[b], cu[b + 1]
        if hi <= lo:
            continue
        o = attn_fwd(Q[lo:hi][None], K[lo:hi][None], V[lo:hi][None],
                     None, False, scale)
        out[lo:hi] = o[0]
    return out


def rope_tables(max_pos: int, D: int, theta: float = 10000.0, device="cpu"):
    inv = 1.0 / (
        theta ** (torch.arange(0, D, 2, dtype=torch.float32, device=device) / D)
    )
    pos = torch.arange(max_pos, dtype=torch.float32, device=device)
    ang = pos[:, None] * inv[None, :]  # [S, D/2]
    return ang.cos().contiguous(), ang.sin().contiguous()


def rope_apply(x: torch.Tensor, cs: torch.Tensor, sn: torch.Tensor,
               pos: torch.Tensor, rope_heads: int = -1):
    """x [..., S, Hx, D] flattened rows [B,S,Hx,D]; pos int32 [B*S].
    Heads >= rope_heads (when >= 0) pass through unchanged."""
    shape = x.shape
    D = shape[-1]
    Hx = shape[-2]
    xf = x.float().reshape(-1, Hx, D)
    p = pos.long().reshape(-1)
    c = cs[p].unsqueeze(1)  # [rows, 1, D/2]
    s = sn[p].unsqueeze(1)
    x1, x2 = xf[..., : D // 2], xf[..., D // 2 :]
    out = torch.cat([x1 * c - x2 * s, x2 * c + x1 * s], dim=-1)
    if 0 <= rope_heads < Hx:
        out[:, rope_heads:] = xf[:, rope_heads:]
    return out.reshape(shape).to(x.dtype)


def topk(scores: torch.Tensor, k: int):
    v, i = torch.topk(scores.float(), k, dim=-1)
    return v, i.int()


def hamming_score(qcodes: torch.Tensor, codes_t: torch.Tensor):
    """qcodes [Q, W] int64 (bit-packed), codes_t [W, N] int64 word-major."""
    Q, W = qcodes.shape
    N = codes_t.shape[1]
    out = torch.zeros(Q, N, dtype=torch.float32, device=qcodes.device)
    for w in range(W):
        x = qcodes[:, w : w + 1] ^ codes_t[w][None, :]
        # popcount on int64 via bit tricks (no torch.popcount on this ver)
        cnt = torch.zeros_like(x)
        for shift in range(0, 64, 8):
            byte = (x >> shift) & 0xFF
            cnt += _POPCNT_TABLE.to(x.device)[byte.long()]
        out -= cnt.float()
    return out


_POPCNT_TABLE = torch.tensor(
    [bin(i).count("1") for i in range(256)], dtype=torch.int64
)


def sample_tokens(logits: torch.Tensor, rand: torch.Tensor, temp: float,
                  min_p: float):
    lf = logits.float()
    if temp <= 0:
        return lf.argmax(dim=-1).int()
    mx = lf.max(dim=-1, keepdim=True).values
    if min_p > 0:
        cut = mx + temp * math.log(min_p)
        lf = torch.where(lf >= cut, lf, torch.full_like(lf, float("-inf")))
    p = torch.softmax((lf - mx) / temp, dim=-1)
    cdf = p.cumsum(dim=-1)
    r = rand.float().unsqueeze(-1)
    idx = (cdf < r).sum(dim=-1).clamp(max=lf.size(-1) - 1)
    return idx.int()


def paged_attn(q, kcache, vcache, block_table, ctx_len, scale):
    """q [B,H,D]; caches [nblk, HKV, BLK, D]; reference decode attention."""
    B, H, D = q.shape
    HKV = kcache.shape[1]
    BLK = kcache.shape[2]
    out = torch.empty_like(q)
    for b in range(B):
        L = int(ctx_len[b])
        nb = (L + BLK - 1) // BLK
        blocks = block_table[b, :nb].long()
        k = kcache[blocks].permute(1, 0, 2, 3).reshape(HKV, -1, D)[:, :L]
        v = vcache[blocks].permute(1, 0, 2, 3).reshape(HKV, -1, D)[:, :L]
        rep = H // HKV
        k = k.repeat_interleave(rep, dim=0).float()
        v = v.repeat_interleave(rep, dim=0).float()
        s = (q[b].float().unsqueeze(1) * k).sum(-1) * scale  # [H, L]
        p = torch.softmax(s, dim=-1)
        out[b] = (p.unsqueeze(-1) * v).sum(1).to(q.dtype)
    return out


# ---- sandwich-norm / latent-attention decoder -----------------------------

def embed_norm(tokens, table, w_next, n, eps):
    """x = table[token] (fp32), h = rms(x) over the first n columns."""
    x = table[tokens.long()].float()
    ms = x.pow(2).sum(-1, keepdim=True) / n
    return (x / torch.sqrt(ms + eps) * w_next).to(table.dtype), x


def post_norm_add(y, x, w_post, w_next, n, eps):
    """x += rms(y) * w_post in place; returns h = rms(x) * w_next."""
    yf = y.float()
    ms = yf.pow(2).sum(-1, keepdim=True) / n
    x += yf / torch.sqrt(ms + eps) * w_post
    ms = x.pow(2).sum(-1, keepdim=True) / n
    return (x / torch.sqrt(ms + eps) * w_next).to(y.dtype)


def _cache_rows(block_table, row_seq, pos, blk):
    """Flat cache row of position pos[i] of sequence row_seq[i]."""
    p = pos.long()
    page = block_table.long()[row_seq.long(), p // blk]
    return page * blk + p % blk


def latent_prep(ab, q_cols, q_rank, rank, wq, wc, eps, cache, block_table,
                row_seq, ctx):
    """Norm of the query latent (returned) and of the cached latent
    (written to the cache at position ctx - 1 of each live row)."""

    def norm(v, n, w):
        v = v.float()
        ms = v.pow(2).sum(-1, keepdim=True) / n
        return (v / torch.sqrt(ms + eps) * w).to(ab.dtype)

    if cache is not None:
        live = ctx > 0
        rows = _cache_rows(block_table, row_seq[live], ctx[live] - 1,
                           cache.shape[1])
        cache.view(-1, cache.shape[2])[rows] = norm(
            ab[live, q_cols:], rank, wc)
    return norm(ab[:, :q_cols], q_rank, wq)


def _rotate(x, table):
    """x [M, .., n]: its first 2 * pairs numbers turned by table [M, pairs,
    2], in fp32."""
    x, half = x.float(), table.shape[1]
    cs = table.view(len(x), *[1] * (x.dim() - 2), half, 2)
    a, b = x[..., :half], x[..., half: 2 * half]
    cos, sin = cs[..., 0], cs[..., 1]
    return torch.cat([a * cos - b * sin, b * cos + a * sin,
                      x[..., 2 * half:]], -1)


def rotary_latent_prep(ab, heads, dp, tp, rank, wc, eps, table, cache,
                       block_table, row_seq, ctx, ql):
    M, n = ab.shape[0], ql.shape[0]
    qr = ab[:, : heads * (dp + tp)].view(M, heads, dp + tp)[..., dp:]
    turned = _rotate(qr, table).to(ab.dtype)
    ql[..., ql.shape[2] - tp:] = turned[:n]
    qr[n:] = turned[n:]
    if cache is None:
        return
    live = ctx > 0
    at, R = heads * (dp + tp), cache.shape[2] - tp
    c = ab[live, at: at + R].float()
    ms = c.pow(2).sum(-1, keepdim=True) / rank
    c = (c / torch.sqrt(ms + eps) * wc).to(ab.dtype)
    kr = _rotate(ab[live, at + R: at + R + tp], table[live]).to(ab.dtype)
    rows = _cache_rows(block_table, row_seq[live], ctx[live] - 1,
                       cache.shape[1])
    cache.view(-1, R + tp)[rows] = torch.cat([c, kr], 1)


def latent_gather(cache, block_table, key_seq, key_pos):
    rows = _cache_rows(block_table, key_seq, key_pos, cache.shape[1])
    return cache.view(-1, cache.shape[2])[rows]


def head_gemm(x, w):
    """[M, H, K] x [H, N, K] -> [M, H, N]."""
    out = torch.bmm(x.float().transpose(0, 1),
                    w.float().transpose(1, 2).contiguous())
    return out.transpose(0, 1).to(x.dtype).contiguous()


def _softmax_sink(s, sink):
    """Softmax over the last axis of s [H, .., n], with exp(sink) of the
    head in the denominator."""
    if sink is None:
        return torch.softmax(s, -1)
    own = sink.float().view(-1, *[1] * (s.dim() - 1)).expand(
        *s.shape[:-1], 1)
    return torch.softmax(torch.cat([s, own], -1), -1)[..., :-1]


def latent_attn(q, cache, block_table, row_seq, ctx, window, scale,
                rank=None, sink=None, gate=None):
    """q [M, H, R] against the cached latents of each row's sequence; the
    key is the whole cache row, the value its first rank (or all) columns."""
    rank = rank or cache.shape[2]
    out = q.new_zeros(q.shape[0], q.shape[1], rank)
    for r in range(q.shape[0]):
        L = int(ctx[r])
        if L <= 0:
            continue
        pos = torch.arange(max(0, L - window), L)
        c = latent_gather(cache, block_table,
                          row_seq[r].expand(len(pos)), pos).float()
        p = _softmax_sink(q[r].float() @ c.t() * scale, sink)
        o = p @ c[:, :rank]
        if gate is not None:
            o = o * torch.sigmoid(gate[r].float())[:, None]
        out[r] = o.to(q.dtype)
    return out


def attn_window(q, kv, dv, cu_q, cu_k, window, scale, kr=None, sink=None,
                gate=None):
    """Packed continuation attention: the queries of a sequence are the
    last ones of its keys. q [Tq, H, DK (+ DR)]; kv [Tk, H*DK + H*DV]; kr
    [Tk, DR]."""
    Tq, H, dk = q.shape
    dk -= 0 if kr is None else kr.shape[1]
    k = kv[:, : H * dk].view(-1, H, dk).float()
    v = kv[:, H * dk:].view(-1, H, dv).float()
    if kr is not None:
        k = torch.cat([k, kr[:, None].float().expand(-1, H, -1)], -1)
    out = torch.zeros(Tq, H, dv, dtype=q.dtype)
    for b in range(len(cu_q) - 1):
        q0, q1 = int(cu_q[b]), int(cu_q[b + 1])
        k0, k1 = int(cu_k[b]), int(cu_k[b + 1])
        i = torch.arange(q1 - q0)[:, None] + (k1 - k0) - (q1 - q0)
        j = torch.arange(k1 - k0)[None]
        s = torch.einsum("qhd,khd->hqk", q[q0:q1].float(),
                         k[k0:k1]) * scale
        s = s.masked_fill((j > i) | (j <= i - window), float("-inf"))
        o = torch.einsum("hqk,khd->qhd", _softmax_sink(s, sink), v[k0:k1])
        if gate is not None:
            o = o * torch.sigmoid(gate[q0:q1].float())[..., None]
        out[q0:q1] = o.to(q.dtype)
    return out


def clamped_glu(gu, limit, alpha, shift):
    F_ = gu.shape[-1] // 2
    g = gu[..., :F_].float().clamp(max=limit)
    u = gu[..., F_:].float().clamp(-limit, limit)
    return (g * torch.sigmoid(alpha * g) * (u + shift)).to(gu.dtype)


# ---- chunked attention / delta rule / experts decoder -----------------------

def embed_positions(tokens, ctx, table, pos):
    p = (ctx.long() - 1).clamp(min=0)
    x = table[tokens.long()].float() + pos[p].float()
    return x.to(table.dtype), x


def _layer_norm_n(v, w, b, n, eps):
    """Layer norm over the first n columns; w and b are 0 beyond."""
    mean = v[:, :n].mean(-1, keepdim=True)
    var = (v[:, :n] - mean).pow(2).mean(-1, keepdim=True)
    return (v - mean) / torch.sqrt(var + eps) * w + b


def layer_norm_add(y, x, w, b, n, eps, final=None, mix=None):
    """x += layer_norm(y) in place; returns x (normed by final's weight
    and bias, if given) in y's dtype. With mix [M, top], y [M * top, W]
    is first summed with these weights."""
    yf = y.float()
    if mix is not None:
        yf = yf.view(*mix.shape, -1).masked_fill(mix[..., None] == 0, 0)
        yf = (yf * mix[..., None]).sum(1)
    x += _layer_norm_n(yf, w, b, n, eps)
    if final is None:
        return x.to(y.dtype)
    return _layer_norm_n(x, final[0], final[1], n, eps).to(y.dtype)


def attn_prep(ab, heads, kv_heads, dp, vp, dim, wq, wk, eps, pages,
              block_table, row_seq, ctx):
    """Per-head norm of the queries (returned) and keys; keys and values
    go to their pages."""

    def norm(v, w):
        v = v.float()
        ms = v.pow(2).sum(-1, keepdim=True) / dim
        return (v / torch.sqrt(ms + eps) * w).to(ab.dtype)

    M = ab.shape[0]
    if pages is not None:
        kp, vpg = pages
        blk = kp.shape[2]
        live = ctx > 0
        rows = _cache_rows(block_table, row_seq[live], ctx[live] - 1, blk)
        at = heads * dp
        k = ab[live, at: at + kv_heads * dp].view(-1, kv_heads, dp)
        v = ab[live, at + kv_heads * dp:][:, : kv_heads * vp]
        kp[rows // blk, :, rows % blk] = norm(k, wk)
        vpg[rows // blk, :, :, rows % blk] = v.reshape(-1, kv_heads, vp)
    return norm(ab[:, : heads * dp].reshape(M, heads, dp), wq)


def paged_attn_rows(q, kpages, vpages, ab, gate_at, out, block_table,
                    row_seq, ctx, chunk, scale, softcap, dist):
    """Attention of single-token rows over the visible part of the pages:
    the positions of the row's chunk up to its own."""
    M, H, _ = q.shape
    G, blk, dv = kpages.shape[1], kpages.shape[2], vpages.shape[2]
    gate = torch.sigmoid(ab[:, gate_at: gate_at + H * dv].float()
                         .reshape(M, H, dv))
    for r in range(M):
        p = int(ctx[r]) - 1
        if p < 0:
            out[r] = 0
            continue
        pos = torch.arange(p // chunk * chunk, p + 1)
        rows = _cache_rows(block_table, row_seq[r].expand(len(pos)), pos,
                           blk)
        k = kpages[rows // blk, :, rows % blk].float()
        v = vpages[rows // blk, :, :, rows % blk].float()
        k = k.repeat_interleave(H // G, 1).transpose(0, 1)   # [H, n, d]
        v = v.repeat_interleave(H // G, 1).transpose(0, 1)
        s = (k * q[r].float()[:, None]).sum(-1) * scale
        s = softcap * torch.tanh(s / softcap)
        s = s - dist[0][:, None] * torch.log1p(
            dist[1][:, None] * (p - pos)[None].float())
        w = torch.softmax(s, -1)
        out[r] = ((w[..., None] * v).sum(1) * gate[r]).to(q.dtype)
    return out


def paged_attn_prompts(q, kpages, vpages, ab, gate_at, out, block_table,
                       prompts, chunk, scale, softcap, dist):
    for seq, row0, start, n in prompts.portions.tolist():
        r = slice(row0, row0 + n)
        paged_attn_rows(q[r], kpages, vpages, ab[r], gate_at, out[r],
                        block_table,
                        torch.full((n,), seq, dtype=torch.int32),
                        torch.arange(start + 1, start + n + 1), chunk, scale,
                        softcap, dist)
    return out


def gated_delta(ab, heads, kv_heads, dp, vp, dim, vdim, conv_w, decay,
                o_norm, unit_eps, eps, state, conv, segments, row_seq, ctx):
    """Convolutions, recurrence and gated output norm of every segment;
    state and conv slots are read and written."""
    M, C, taps = ab.shape[0], conv_w.shape[1], conv_w.shape[0]
    G, H = kv_heads, heads
    out = torch.zeros(M, H * vp, dtype=ab.dtype)
    own = torch.arange(H) // (H // G)
    for row0, n, slot in zip(segments.row0.tolist(), segments.rows.tolist(),
                             segments.slot.tolist()):
        if n == 0:
            continue
        start = int(ctx[row0]) - 1
        S = state[slot] * (start > 0)                  # [H, vp, dp]
        past = conv[slot] * (start > 0)
        x = torch.cat([past, ab[row0: row0 + n, :C]])
        conv[slot] = x[n:]
        z = sum(x[a: a + n].float() * conv_w[a] for a in range(taps))
        z = torch.nn.functional.silu(z)
        qk = z[:, : 2 * G * dp].view(n, 2, G, dp)
        qk = qk / torch.sqrt(qk.pow(2).sum(-1, keepdim=True) + unit_eps)
        q, k = qk[:, 0, own] * dim ** -0.5, qk[:, 1, own]
        v = z[:, 2 * G * dp:].to(ab.dtype).float().view(n, H, vp)
        gate = ab[row0: row0 + n, C: C + H * vp].float().view(n, H, vp)
        ba = ab[row0: row0 + n, C + H * vp:][:, : 2 * H].float()
        beta = torch.sigmoid(ba[:, :H])
        g = torch.exp(-torch.exp(decay[0]) * torch.nn.functional.softplus(
            ba[:, H:] + decay[1]))
        for i in range(n):
            S = S * g[i, :, None, None]
            u = beta[i, :, None] * (v[i] - (S * k[i, :, None]).sum(-1))
            S = S + u[..., None] * k[i, :, None]
            o = (S * q[i, :, None]).sum(-1)            # [H, vp]
            ms = o.pow(2).sum(-1, keepdim=True) / vdim
            y = o / torch.sqrt(ms + eps) * o_norm
            y = y * torch.nn.functional.silu(gate[i])
            out[row0 + i] = y.reshape(-1).to(ab.dtype)
        state[slot] = S
    return out


def xielu(z, act):
    p, q = torch.nn.functional.softplus(act.float())
    f = z.float()
    pos = p * f * f + 0.5 * f
    neg = (0.5 + q) * (torch.expm1(f.clamp(max=0)) - f) + 0.5 * f
    return torch.where(f > 0, pos, neg).to(z.dtype)


def route(h, router, ctx, top, groups, keep):
    """-> expert ids [M, top] int32 (-1: none) and weights [M, top]."""
    s = torch.softmax(h.float() @ router.float().t(), -1)
    M, E = s.shape
    best = s.view(M, groups, -1).amax(-1).topk(keep, -1).indices
    allowed = torch.zeros(M, groups, dtype=torch.bool).scatter(1, best, True)
    allowed = allowed.repeat_interleave(E // groups, 1)
    w, ids = s.masked_fill(~allowed, -1).topk(top, -1)
    dead = (ctx <= 0)[:, None]
    return ids.int().masked_fill(dead, -1), w.masked_fill(dead, 0)


def route_sigmoid(h, router, correction, ctx, top, scale, shards=0):
    """-> expert ids [M, top + shards] int32 (-1: none) and weights."""
    E = correction.shape[0]
    s = torch.sigmoid(h.float() @ router.float().t())
    ids = (s[:, :E] + correction).topk(top, -1).indices
    w = torch.cat([s.gather(1, ids) * scale,
                   s[:, E:].repeat(1, max(shards, 1))], 1)
    ids = torch.cat([ids, (E + torch.arange(shards)).expand(len(ids), -1)],
                    1)
    dead = (ctx <= 0)[:, None]
    return ids.int().masked_fill(dead, -1), w.masked_fill(dead, 0)


def relu2(z):
    return z.float().clamp(min=0).square().to(z.dtype)


def experts(h, ids, wgup, wdown, gated=True, unit=16):
    M, top = ids.shape
    out = torch.zeros(M * top, wdown.shape[1], dtype=h.dtype)
    flat = ids.reshape(-1)
    for e in flat.unique().tolist():
        if e < 0:
            continue
        rows = (flat == e).nonzero()[:, 0]
        gu = h[rows // top].float() @ wgup[e].float().t()
        if gated:
            gu = gu.view(len(rows), -1, 2, unit)
            a = torch.nn.functional.silu(gu[:, :, 0]) * gu[:, :, 1]
            a = a.reshape(len(rows), -1).to(h.dtype)
        else:
            a = relu2(gu).to(h.dtype)
        out[rows] = (a.float() @ wdown[e].float().t()).to(h.dtype)
    return out


# ---- parallel attention and delta rule / linear recurrent decoder -----------

def residual_step(x, y, bias, rms, embed, vec, act, fresh, dtype):
    if fresh:
        x.zero_()
    if y is not None:
        v = y.float()
        if rms is not None:
            w, n, eps = rms
            ms = v.pow(2).sum(-1, keepdim=True) / n
            v = v / torch.sqrt(ms + eps) * w
        x += v if bias is None else v + bias
    if embed is not None:
        tokens, table, scale = embed
        x += table[tokens.long()].float() * scale
    if vec is not None:
        x += vec
    if act is None:
        return x.to(dtype)
    w, b, alpha = act
    return (torch.tanh(alpha * x) * w + b).to(dtype)


def gelu_rows(z, tokens, table, col0, n):
    e = table[tokens.long(), col0: col0 + n].float()
    out = torch.zeros_like(z)
    out[:, :n] = (F.gelu(z[:, :n].float(), approximate="tanh") * e).to(
        z.dtype)
    return out


def rotation_table(ctx, freq, mult):
    a = (ctx.double() - 1).clamp(min=0)[:, None] * freq
    return (torch.stack([a.cos(), a.sin()], -1) * mult).float()


def rotary_prep(ab, heads, kv_heads, dp, dim, wq, wk, eps, table, pages,
                block_table, row_seq, ctx):
    M, half = ab.shape[0], table.shape[1]
    cos, sin = table[:, None, :, 0], table[:, None, :, 1]

    def prep(v, w):
        v = v.reshape(M, -1, dp).float()
        ms = v.pow(2).sum(-1, keepdim=True) / dim
        v = v / torch.sqrt(ms + eps) * w
        a, b = v[..., :half], v[..., half: 2 * half]
        return torch.cat([a * cos - b * sin, b * cos + a * sin,
                          v[..., 2 * half:]], -1).to(ab.dtype)

    kp, vpg = pages
    blk = kp.shape[2]
    live = ctx > 0
    rows = _cache_rows(block_table, row_seq[live], ctx[live] - 1, blk)
    k = ab[:, heads * dp: (heads + kv_heads) * dp]
    kp[rows // blk, :, rows % blk] = prep(k, wk)[live]
    vpg[rows // blk, :, :, rows % blk] = k[live].reshape(-1, kv_heads, dp)
    return prep(ab[:, : heads * dp], wq)


def sink_attn_rows(q, kpages, vpages, out, block_table, row_seq, ctx, scale,
                   sink, out_scale):
    M, H, _ = q.shape
    G, blk = kpages.shape[1], kpages.shape[2]
    for r in range(M):
        n = int(ctx[r])
        if n <= 0:
            out[r] = 0
            continue
        rows = _cache_rows(block_table, row_seq[r].expand(n),
                           torch.arange(n), blk)
        k = kpages[rows // blk, :, rows % blk].float()
        v = vpages[rows // blk, :, :, rows % blk].float()
        k = k.repeat_interleave(H // G, 1).transpose(0, 1)   # [H, n, d]
        v = v.repeat_interleave(H // G, 1).transpose(0, 1)
        s = (k * q[r].float()[:, None]).sum(-1) * scale
        w = torch.softmax(torch.cat([s, sink.float()[:, None]], 1), -1)
        o = (w[:, :n, None] * v).sum(1) * out_scale
        out[r] = o.reshape(-1).to(q.dtype)
    return out


def sink_attn_prompts(q, kpages, vpages, out, block_table, prompts, scale,
                      sink, out_scale):
    for seq, row0, start, n in prompts.portions.tolist():
        r = slice(row0, row0 + n)
        sink_attn_rows(q[r], kpages, vpages, out[r], block_table,
                       torch.full((n,), seq, dtype=torch.int32),
                       torch.arange(start + 1, start + n + 1), scale, sink,
                       out_scale)
    return out


def _short_conv(x, conv_w, slot, conv, start):
    """Causal convolution of one segment's rows x [n, C] (fp32 result); its
    slot of last inputs is read and renewed."""
    n, taps = x.shape[0], conv_w.shape[0]
    x = torch.cat([conv[slot] * (start > 0), x])
    conv[slot] = x[n:]
    return sum(x[a: a + n].float() * conv_w[a] for a in range(taps))


def channel_delta(ab, ag, heads, kv_heads, dp, vp, dim, vdim, conv_w, a_log,
                  dt_bias, o_norm, unit_eps, eps, out_scale, state, conv,
                  segments, row_seq, ctx, out):
    C = conv_w.shape[1]
    G, H = kv_heads, heads
    own = torch.arange(H) // (H // G)
    for row0, n, slot in zip(segments.row0.tolist(), segments.rows.tolist(),
                             segments.slot.tolist()):
        if n == 0:
            continue
        r = slice(row0, row0 + n)
        start = int(ctx[row0]) - 1
        S = state[slot] * (start > 0)                  # [H, vp, dp]
        z = F.silu(_short_conv(ab[r, :C], conv_w, slot, conv, start))
        qk = z[:, : 2 * G * dp].view(n, 2, G, dp)
        qk = qk / torch.sqrt(qk.pow(2).sum(-1, keepdim=True) + unit_eps)
        q, k = qk[:, 0, own] * dim ** -0.5, qk[:, 1, own]
        v = z[:, 2 * G * dp:].to(ab.dtype).float().view(n, H, vp)
        beta = torch.sigmoid(ab[r, C: C + H].float())
        a = F.softplus(ag[r, : H * dp].float() + dt_bias).view(n, H, dp)
        g = torch.exp(-torch.exp(a_log)[:, None] * a)
        gate = torch.sigmoid(ag[r, H * dp:].float()).view(n, H, vp)
        for i in range(n):
            S = S * g[i, :, None]
            u = beta[i, :, None] * (v[i] - (S * k[i, :, None]).sum(-1))
            S = S + u[..., None] * k[i, :, None]
            o = (S * q[i, :, None]).sum(-1)            # [H, vp]
            ms = o.pow(2).sum(-1, keepdim=True) / vdim
            y = o / torch.sqrt(ms + eps) * o_norm * gate[i] * out_scale
            out[row0 + i] = y.reshape(-1).to(ab.dtype)
        state[slot] = S
    return out


def gated_lru(ab, conv_w, conv_b, gates, gates_b, decay, state, conv,
              segments, row_seq, ctx):
    M, C = ab.shape[0], conv_w.shape[1]
    B, bs = gates.shape[1], gates.shape[2]
    # [gate, block, in, out] from the stored order (ops.lru_gate_order)
    w = gates.float().view(2, B, bs // 32, bs // 32, 2, 4, 16, 8)
    w = w.permute(0, 1, 3, 5, 7, 2, 6, 4).reshape(2, B, bs, bs)
    out = torch.zeros(M, C, dtype=ab.dtype)
    for row0, n, slot in zip(segments.row0.tolist(), segments.rows.tolist(),
                             segments.slot.tolist()):
        if n == 0:
            continue
        r = slice(row0, row0 + n)
        start = int(ctx[row0]) - 1
        S = state[slot] * (start > 0)
        u = _short_conv(ab[r, C:], conv_w, slot, conv, start) + conv_b
        u = u.to(ab.dtype).float()
        z = torch.zeros(2, n, C)
        z[..., : B * bs] = torch.matmul(
            u[:, : B * bs].view(n, B, bs).transpose(0, 1), w
        ).transpose(1, 2).reshape(2, n, B * bs)
        z = torch.sigmoid(z + gates_b[:, None])
        log_a = decay * z[0]
        drive = torch.sqrt(-torch.expm1(2 * log_a)) * z[1] * u
        a = torch.exp(log_a)
        y = F.gelu(ab[r, :C].float(), approximate="tanh")
        for i in range(n):
            S = a[i] * S + drive[i]
            out[row0 + i] = (S * y[i]).to(ab.dtype)
        state[slot] = S
    return out


# ---- retention / rotary latent attention decoder on several streams ---------

def stream_step(x, y, writes, mix, shared, embed, read, norm, store, dtype):
    S = x.shape[1]
    old = x
    if embed is not None:
        tokens, table = embed
        old = table[tokens.long()].float()[:, None].expand(-1, S, -1)
    new = old
    if y is not None:
        v = y.float()
        if mix is not None:
            top = mix.shape[1] - (shared is not None)
            w = mix[:, :top, None]
            v = (v.view(len(x), top, -1).masked_fill(w == 0, 0) * w).sum(1)
            if shared is not None:
                v = v + shared.float() * mix[:, top:]
        out, m = writes[:S], writes[S:].view(S, S)
        new = (old[:, :, None] * m[None, :, :, None]).sum(1) \
            + out[None, :, None] * v[:, None]
        if store:
            x.copy_(new)
    u = new.sum(1) if read is None else (new * read[None, :, None]).sum(1)
    w, n, eps = norm
    ms = u.pow(2).sum(-1, keepdim=True) / n
    return (u / torch.sqrt(ms + eps) * w).to(dtype)


def retention(ab, heads, dp, vp, dim, vdim, decay, table, eps, state,
              segments, ctx):
    M, H = ab.shape[0], heads
    out = torch.zeros(M, H * vp, dtype=ab.dtype)
    qk = _rotate(ab[:, : 2 * H * dp].reshape(M, 2 * H, dp), table)
    q, k = qk[:, :H], qk[:, H:] * dim ** -0.5
    v = ab[:, 2 * H * dp: 2 * H * dp + H * vp].float().view(M, H, vp)
    gate = F.silu(ab[:, 2 * H * dp + H * vp:].float()).view(M, H, vp)
    g = decay[0][:, None, None]
    for row0, n, slot in zip(segments.row0.tolist(), segments.rows.tolist(),
                             segments.slot.tolist()):
        if n == 0:
            continue
        S = state[slot] * (int(ctx[row0]) > 1)         # [H, vp, dp]
        for i in range(row0, row0 + n):
            S = g * S + v[i, :, :, None] * k[i, :, None]
            o = (S * q[i, :, None]).sum(-1)            # [H, vp]
            ms = o.pow(2).sum(-1, keepdim=True) / vdim
            y = o / torch.sqrt(ms + eps) * gate[i]
            out[i] = y.reshape(-1).to(ab.dtype)
        state[slot] = S
    return out
