"""Kedelorn on the GPU: the HIP kernels against fp32 references of the same
op, and the engine path in bf16 and fp32 against the plain
implementation."""

import json
import os
import subprocess
import sys
from pathlib import Path

import pytest
import torch

import kedelorn_cases as cases
import kedelorn_oracle as oracle
from distllm_amd import ops
from distllm_amd.engine.step import Segments
from distllm_amd.models.config import RotaryDims
from distllm_amd.ops import torch_ref
from test_bufulorn_gpu import _close, _i32, _rand
from test_kanotar_gpu import _paged
from test_tebasun_gpu import _batch_of

pytestmark = pytest.mark.gpu

F32, BF16 = torch.float32, torch.bfloat16
DTYPES = [BF16, F32]
ids = {BF16: "bf16", F32: "fp32"}.get
dtypes = pytest.mark.parametrize("dtype", DTYPES, ids=ids)


def _table(rot, ctx):
    f, mult = RotaryDims(**rot).frequencies()
    return ops.rotation_table(ctx.cuda(), torch.tensor(
        f, dtype=torch.float64).cuda(), mult)


# ---- kernels ---------------------------------------------------------------

@dtypes
@pytest.mark.parametrize("S", [1, 2, 3, 4, 6, 8, 13])
@pytest.mark.parametrize("M, W, n", [(1, 64, 1), (7, 320, 300),
                                     (5, 1024, 1024), (3, 4096, 4000),
                                     (2, 8192, 8192), (2, 12288, 12288)])
def test_stream_step(device, dtype, S, M, W, n):
    top = 3
    x0 = _rand(M, S, W) * torch.logspace(-3, 1, M).cuda()[:, None, None]
    y, one = _rand(M * top, W, seed=1, dtype=dtype), _rand(M, W, seed=2,
                                                           dtype=dtype)
    table, w = _rand(11, W, seed=3, dtype=dtype), _rand(W, seed=4)
    coef, mix = _rand(S * (S + 2), seed=5), _rand(M, top + 1, seed=6)
    for t in (x0, y, one, table, w):
        t[..., n:] = 0
    mix[0, 1], y[1] = 0, float("nan")  # no expert: not looked at
    tok = torch.arange(M, device="cuda") % 11
    embed, reads, writes = (tok, table), coef[:S], coef[S:]
    for kw in ({"embed": embed, "read": reads, "dtype": dtype},
               {"y": one, "writes": writes, "embed": embed, "read": reads},
               {"y": one, "writes": writes, "read": reads},
               {"y": y, "writes": writes, "read": reads, "shared": one,
                "mix": mix},
               {"y": y, "writes": writes, "mix": mix[:, :top].contiguous()},
               {"y": one, "writes": writes, "store": False}):
        x, xr = x0.clone(), x0.clone()
        h = ops.stream_step(x, norm=(w, n, 0.01), **kw)
        args = {"y": None, "writes": None, "mix": None, "shared": None,
                "embed": None, "read": None, "store": True, **kw}
        args["dtype"] = F32
        want = torch_ref.stream_step(xr, norm=(w, n, 0.01), **args)
        assert h.dtype == dtype
        _close(x, xr, F32)
        _close(h, want, dtype, None if dtype == BF16 else 2e-4)  # sums cancel
    x = x0.clone()
    ops.stream_step(x, one, writes, read=reads, norm=(w, n, 0.01),
                    store=False)
    assert torch.equal(x, x0)


@dtypes
@pytest.mark.parametrize("M, N, K", [(1, 64, 64), (37, 192, 256),
                                     (300, 128, 128), (256, 64, 1024),
                                     (8, 512, 4096)])
def test_up_relu2(device, dtype, M, N, K):
    x, w = _rand(M, K, dtype=dtype), (_rand(N, K, seed=1) * 0.2).to(dtype)
    z = (x.double() @ w.double().t()).cpu()
    _close(ops.up_relu2(x, w), torch.clamp(z, min=0) ** 2, dtype, 4e-2
           if dtype == BF16 else None)


@dtypes
@pytest.mark.parametrize("E, top, gates", [
    (1, 1, 0), (6, 2, 1), (16, 16, 1), (47, 5, 0), (64, 8, 1), (79, 3, 1),
    (128, 8, 1), (200, 20, 0), (255, 4, 1), (300, 6, 1), (1000, 9, 1)])
def test_route_sigmoid(device, dtype, E, top, gates):
    M, W = 45, 192
    h = _rand(M, W, dtype=dtype)
    router = (_rand(E + gates, W, seed=1) * 0.2).to(dtype)
    corr = _rand(E, seed=2) - 2
    ctx = torch.arange(1, M + 1).int()
    ctx[7] = 0
    got, w = ops.route_sigmoid(h, router, corr, ctx.cuda(), top, 1.6)
    s = oracle.sigmoid(h.double().cpu() @ router.double().cpu().T)
    choice = s[:, :E] + corr.double().cpu()
    close = 0
    for m in range(M):
        if m == 7:
            assert (got[m] == -1).all() and not w[m].any()
            continue
        own = got[m].long().cpu()
        assert len(set(own.tolist())) == top
        want = choice[m].topk(top).indices
        if not torch.equal(own, want):  # fp32 may swap equal scores
            close += 1
            assert torch.allclose(choice[m, own], choice[m, want], rtol=1e-4)
        assert torch.allclose(w[m, :top].double().cpu(), 1.6 * s[m, own],
                              rtol=1e-4)
        assert torch.allclose(w[m, top:].double().cpu(), s[m, E:], rtol=1e-4)
    assert close < 3
    if gates:  # the shared expert as two more choices
        ids2, w2 = ops.route_sigmoid(h, router, corr, ctx.cuda(), top, 1.6, 2)
        live = (ctx > 0).cuda()
        assert torch.equal(ids2[:, :top], got)
        assert (ids2[live, top:] == torch.tensor([E, E + 1]).cuda()).all()
        assert torch.equal(w2, torch.cat([w[:, :top], w[:, top:].expand(
            -1, 2)], 1))
        assert (ids2[7] == -1).all()


@dtypes
@pytest.mark.parametrize("M, E, top, W, ff", [
    (1, 6, 2, 64, 64), (9, 6, 3, 192, 128), (40, 8, 2, 256, 192),
    (130, 8, 2, 128, 64), (300, 4, 2, 320, 192), (700, 5, 2, 128, 320),
    (1100, 4, 2, 256, 256), (1300, 4, 2, 512, 384), (1200, 3, 2, 256, 512)])
def test_squared_relu_experts(device, dtype, M, E, top, W, ff):
    """Every tile size of the grouped product; uneven experts, one of them
    without a row, padding rows."""
    h = _rand(M, W, dtype=dtype)
    up = (_rand(E, ff, W, seed=1) / W ** 0.5).to(dtype)
    down = (_rand(E, W, ff, seed=2) / ff ** 0.5).to(dtype)
    g = torch.Generator().manual_seed(3)
    p = torch.rand(M, E, generator=g) + torch.linspace(0, 0.8, E)
    p[:, 1] = -1
    chosen = p.topk(top, -1).indices.int()
    chosen[M // 2] = -1 if M > 1 else chosen[0]
    y = ops.experts(h, chosen.cuda(), up, down, gated=False)
    want = torch_ref.experts(h.cpu().float(), chosen, up.cpu().float(),
                             down.cpu().float(), gated=False)
    live = (chosen >= 0).reshape(-1)
    _close(y[live.cuda()], want[live], dtype, 3e-2 if dtype == BF16 else None)


@dtypes
@pytest.mark.parametrize("M, E, top", [
    (16384, 3, 2), (16385, 64, 2), (9000, 100, 4), (20000, 200, 2),
    (8200, 500, 5), (40000, 1000, 1)])
def test_plan_of_many_rows(device, dtype, M, E, top):
    """Pairs sorted in blocks; uneven experts, some without a row."""
    h = _rand(M, 64, dtype=dtype)
    up, down = _rand(E, 64, 64, seed=1), _rand(E, 64, 64, seed=2)
    g = torch.Generator().manual_seed(3)
    p = torch.rand(M, E, generator=g) + torch.linspace(0, 0.8, E)
    p[:, 1] = -1
    ids = p.topk(top, -1).indices.int()
    ids[M // 2], ids[M - 1] = -1, -1
    y = ops.experts(h, ids.cuda(), (up / 8).to(dtype), (down / 8).to(dtype),
                    gated=False)
    few = torch.randperm(M - 1, generator=g)[:200]
    few = few[few != M // 2]
    want = torch_ref.experts(h[few.cuda()].cpu().float(), ids[few],
                             (up / 8).to(dtype).cpu().float(),
                             (down / 8).to(dtype).cpu().float(), gated=False)
    got = y.view(M, top, -1)[few.cuda()].flatten(0, 1)
    _close(got, want, dtype, 3e-2 if dtype == BF16 else None)
    # every pair has a place: none of its rows is left as it was
    live = (ids >= 0).reshape(-1).cuda()
    assert torch.isfinite(y[live]).all() and (y[live].abs().sum(1) > 0).all()


@dtypes
@pytest.mark.parametrize("rank, R, rot_dim, tp", [
    (40, 64, 8, 64), (512, 512, 64, 64), (130, 192, 6, 64),
    (600, 640, 72, 128), (1100, 1152, 64, 64), (33, 64, 2, 64)])
@pytest.mark.parametrize("H, n", [(3, 0), (40, 3), (1, 6)])
def test_rotary_latent_prep(device, dtype, rank, R, rot_dim, tp, H, n):
    dp, M, rot = 64, 6, oracle.yarn(rot_dim, 500.0)
    _, bt = _paged(64, [40, 7], dtype)
    ctx, seq = _i32(40, 17, 7, 0, 1, 39), _i32(0, 0, 1, 0, 1, 0)
    ab = _rand(M, H * (dp + tp) + R + tp + 64, dtype=dtype)
    q, kv = ab[:, : H * (dp + tp)].view(M, H, -1), ab[:, H * (dp + tp):]
    q[..., dp + rot_dim:], kv[:, rank: R] = 0, 0
    kv[:, R + rot_dim: R + tp] = 0
    wc = _rand(R, seed=1)
    table = _table(rot, ctx)
    cache = torch.zeros(8, 16, R + tp, dtype=dtype, device="cuda")
    ql = torch.full((n, H, R + tp), 7.0, dtype=dtype, device="cuda")
    ra, rc, rq = ab.cpu().float(), cache.cpu().float(), ql.cpu().float()
    ops.rotary_latent_prep(ab, H, dp, tp, rank, wc, 1e-3, table, cache,
                           bt.cuda(), seq.cuda(), ctx.cuda(), ql)
    torch_ref.rotary_latent_prep(ra, H, dp, tp, rank, wc.cpu(), 1e-3,
                                 table.cpu(), rc, bt, seq, ctx, rq)
    _close(ab, ra, dtype)
    _close(cache, rc, dtype)
    if n:
        _close(ql, rq, dtype)
    c, kr = ops.latent_gather(cache, bt.cuda(), _i32(1, 0).cuda(),
                              _i32(6, 39).cuda(), R)
    for i, (s, p) in enumerate(((1, 6), (0, 39))):
        row = cache[bt[s, p // 16].item(), p % 16]
        assert torch.equal(c[i], row[:R]) and torch.equal(kr[i], row[R:])
    # a layer without latents of its own
    own = torch.full((n, H, R + tp), 7.0, dtype=dtype, device="cuda")
    ab2 = _rand(M, H * (dp + tp) + 64, seed=5, dtype=dtype)
    ab2[:, : H * (dp + tp)].view(M, H, -1)[..., dp + rot_dim:] = 0
    ra, rq = ab2.cpu().float(), own.cpu().float()
    ops.rotary_latent_prep(ab2, H, dp, tp, rank, None, 1e-3, table, None,
                           bt.cuda(), seq.cuda(), ctx.cuda(), own)
    torch_ref.rotary_latent_prep(ra, H, dp, tp, rank, None, 1e-3,
                                 table.cpu(), None, bt, seq, ctx, rq)
    _close(ab2, ra, dtype)
    assert n == 0 or _close(own, rq, dtype) is None


def test_head_gemm_strided(device):
    wide = _rand(20, 5, 192, dtype=BF16)
    w = _rand(5, 128, 64, seed=1, dtype=BF16)
    out = torch.full((20, 5, 256), 7.0, dtype=BF16, device="cuda")
    ops.head_gemm(wide[..., 64:128], w, out=out[..., 64:192])
    want = torch_ref.head_gemm(wide[..., 64:128].cpu().float(),
                               w.cpu().float())
    _close(out[..., 64:192], want, BF16)
    assert (out[..., :64] == 7).all() and (out[..., 192:] == 7).all()


@dtypes
@pytest.mark.parametrize("R, rot", [(64, 64), (128, 64), (192, 64),
                                    (256, 64), (384, 64), (512, 64),
                                    (640, 128), (64, 0), (512, 0)])
@pytest.mark.parametrize("H", [1, 16, 20, 40, 70])
def test_latent_attn(device, dtype, R, rot, H):
    """Scores over the whole row, values from its first numbers, sinks that
    take all or nothing, gates."""
    lens = [1, 15, 16, 33, 200, 517]
    cache, bt = _paged(R + rot, lens, dtype)
    row_seq = _i32(5, 0, 1, 2, 3, 4, 5, 4, 0)
    ctx = _i32(517, 1, 15, 16, 33, 200, 300, 97, 0)
    q = _rand(9, H, R + rot, seed=2, dtype=dtype)
    sink = _rand(H, seed=3) * 3
    if H > 2:
        sink[1], sink[2] = 90.0, -95.0
    wide = _rand(9, H + 24, seed=4, dtype=dtype)
    gate = wide[:, 8: 8 + H]
    scale = 2.0 / (R + rot) ** 0.5
    for window in (33, 1 << 30):
        want = torch_ref.latent_attn(
            q.cpu().float(), cache.cpu().float(), bt, row_seq, ctx, window,
            scale, R, sink.cpu(), gate.cpu().float())
        for nsplit in (0, 1, 3):
            got = ops.latent_attn(q, cache, bt.cuda(), row_seq.cuda(),
                                  ctx.cuda(), window, scale, nsplit, R, sink,
                                  gate)
            assert got.shape == (9, H, R)
            _close(got, want, dtype, None if dtype == BF16 else 5e-5)
            assert not got[8].any()  # a padding row sees nothing


@dtypes
@pytest.mark.parametrize("R, H", [(64, 3), (512, 40)])
@pytest.mark.parametrize("part", ["latent", "rotated"])
def test_latent_attn_far_key(device, dtype, R, H, part):
    """A key that matches the query in one of its two parts comes back
    whole, from every place and at page and tile borders."""
    cache, bt = _paged(R + 64, [400], dtype)
    cache *= 0.05
    at = slice(0, R) if part == "latent" else slice(R, R + 64)
    q = torch.zeros(3, H, R + 64, dtype=dtype, device="cuda")
    q[..., at] = 4.0
    sink = torch.full((H,), 30.0, device="cuda")
    for pos in (0, 15, 16, 31, 32, 100, 127, 128, 398):
        c = cache.clone()
        c[bt[0, pos // 16].item(), pos % 16, at] = 4.0
        c[bt[0, pos // 16].item(), pos % 16, :R] = 4.0
        ctx = _i32(pos, pos + 1, 400).cuda()
        out = ops.latent_attn(q, c, bt.cuda(), _i32(0, 0, 0).cuda(), ctx,
                              1 << 30, 1.0, 0, R, sink).float()
        assert (out[1:] > 3.9).all() and (out[0].abs() < 1).all(), pos


@pytest.mark.parametrize("dk, dv", [(64, 64), (64, 128), (128, 64),
                                    (128, 128), (256, 64), (128, 256),
                                    (256, 256)])
def test_attn_window(device, dk, dv):
    """Prompt continuations with a shared key part, sinks and gates;
    queries are columns of a wider product."""
    H = 3
    nq, nk = [130, 33, 1, 300], [130, 170, 65, 411]
    cu_q = torch.tensor([0] + nq).cumsum(0).int()
    cu_k = torch.tensor([0] + nk).cumsum(0).int()
    wide = _rand(sum(nq), H * (dk + 64) + 64, dtype=BF16)
    q = wide[:, : H * (dk + 64)].view(-1, H, dk + 64)
    kv = _rand(sum(nk), H * (dk + dv), seed=1, dtype=BF16)
    kr = _rand(sum(nk), 64, seed=2, dtype=BF16)
    gate = wide[:, H * (dk + 64):][:, :H]
    sink = torch.tensor([0.5, 300.0, -95.0], device="cuda")
    bm = tuple(t.cuda() for t in ops.varlen_block_map(cu_q))
    scale = 2.0 / dk ** 0.5
    for window in (97, 1 << 30):
        out = torch.full((sum(nq), H, dv), 7.0, dtype=BF16, device="cuda")
        ops.attn_window(q, kv, out, cu_q.cuda(), cu_k.cuda(), bm, window,
                        scale, kr, sink, gate)
        want = torch_ref.attn_window(
            q.cpu().float(), kv.cpu().float(), dv, cu_q, cu_k, window, scale,
            kr.cpu().float(), sink.cpu(), gate.cpu().float())
        _close(out, want, BF16)
        assert not out[:, 1].any()


def test_attn_window_far_key(device):
    """One key that matches in its shared part, at every kind of place."""
    H, d, Tk, Tq = 2, 64, 400, 333
    cu_q, cu_k = _i32(0, Tq), _i32(0, Tk)
    bm = tuple(t.cuda() for t in ops.varlen_block_map(cu_q))
    base = _rand(Tk, 2 * H * d, dtype=BF16) * 0.05
    q = torch.zeros(Tq, H, d + 64, dtype=BF16, device="cuda")
    q[..., d:] = 4.0
    for pos in (0, 63, 64, 127, 200, 255, 269, 399):
        kv, kr = base.clone(), _rand(Tk, 64, seed=3, dtype=BF16) * 0.05
        kv[pos, H * d:], kr[pos] = 4.0, 4.0
        out = torch.empty(Tq, H, d, dtype=BF16, device="cuda")
        ops.attn_window(q, kv, out, cu_q.cuda(), cu_k.cuda(), bm, 1 << 30,
                        1.0, kr)
        seen = torch.arange(Tq) + Tk - Tq >= pos
        got = out.float().mean((1, 2)).cpu() > 3.9
        assert torch.equal(got, seen), pos


def _retention_inputs(H, dp, vp, dim, vdim, rot, ctx, slots, dtype, seed=0):
    M = len(ctx)
    wide = _rand(M, 2 * H * (dp + vp) + 64, seed=seed, dtype=dtype)
    ab = wide[:, 64:]
    cols = torch.arange(2 * H * (dp + vp))
    pad = torch.where(cols < 2 * H * dp, cols % dp >= dim,
                      (cols - 2 * H * dp) % vp >= vdim).cuda()
    ab[:, pad] = 0
    state = _rand(slots, H, vp, dp, seed=seed + 1)
    state[:, :, vdim:], state[..., dim:] = 0, 0
    g = 1 - torch.logspace(-0.5, -3, H, dtype=torch.float64)
    g[0] = 1.0 if H > 1 else g[0]
    return {"ab": ab, "decay": torch.stack([g, g.log2()]).float().cuda(),
            "table": _table(rot, ctx), "state": state}


def _run_retention(r, H, dp, vp, dim, vdim, seg, ctx, ref=False):
    f = torch_ref if ref else ops
    return f.retention(r["ab"], H, dp, vp, dim, vdim, r["decay"], r["table"],
                       1e-5, r["state"], seg, ctx)


@dtypes
@pytest.mark.parametrize("H, dp, vp, half, rows", [
    (2, 64, 64, 8, [1, 1, 1]), (4, 128, 128, 60, [3, 150, 1, 2]),
    (3, 64, 128, 27, [70, 5]), (2, 128, 64, 3, [64, 65, 63]),
    (4, 64, 256, 16, [33, 200]), (2, 256, 64, 124, [40, 129]),
    (2, 256, 256, 120, [66, 2]), (1, 128, 256, 7, [300]),
    (6, 128, 128, 32, [16, 17, 32, 31, 1]), (64, 64, 128, 28, [95]),
    (32, 128, 128, 56, [33] * 8), (3, 64, 64, 24, [700, 20, 1]),
    (2, 128, 128, 48, [1200]), (2, 256, 128, 60, [300, 17]),
    (2, 64, 320, 20, [40, 1]), (3, 448, 64, 33, [1, 50])])
def test_retention(device, dtype, H, dp, vp, half, rows):
    """Segments of one row to several pieces, from the start or going on,
    with padding rows behind; the sequence's slots and no others change."""
    starts = [(0, 5, 2, 0)[i % 4] for i in range(len(rows))]
    seg, ctx, _ = _batch_of(rows, starts)
    S, dim, vdim, n = len(rows), dp - 7, vp - 3, sum(rows)
    rot = {"base": 1e4, "dims": 2 * half}
    r = _retention_inputs(H, dp, vp, dim, vdim, rot, ctx, S + 2, dtype)
    host = {k: v.cpu().clone() for k, v in r.items()}
    host["ab"] = host["ab"].float()
    want = _run_retention(host, H, dp, vp, dim, vdim, seg, ctx, True)
    before = r["state"].clone()
    dseg = Segments.build(seg.row0.tolist(), rows, seg.slot.tolist(), "cuda")
    got = _run_retention(r, H, dp, vp, dim, vdim, dseg, ctx.cuda())
    assert got.dtype == dtype
    _close(got[:n], want[:n], dtype, None if dtype == BF16 else 1e-4)
    _close(r["state"], host["state"], F32, 1e-4)
    assert torch.equal(r["state"][0], before[0])
    assert torch.equal(r["state"][S + 1], before[S + 1])


@pytest.mark.parametrize("H, dp, vp, rows", [
    (4, 128, 128, [200, 17, 3]), (64, 64, 64, [64, 31]),
    (3, 256, 256, [70, 600]), (32, 128, 128, [33] * 8),
    (2, 128, 64, [2500, 900])])
def test_retention_chunks(device, H, dp, vp, rows):
    """The chunked form and its pieces against the token-by-token form,
    both in fp32 behind the same bf16 inputs."""
    row0 = torch.tensor([0] + rows).cumsum(0)[:-1].tolist()
    S = len(rows)
    ctx = torch.cat([torch.arange(n) + 1 + 4 * (i % 2)
                     for i, n in enumerate(rows)]).int()
    r = _retention_inputs(H, dp, vp, dp, vp, {"base": 1e4, "dims": dp}, ctx,
                          S + 1, BF16)
    got = []
    for chunked in (True, False):
        seg = Segments.build(row0, rows, range(1, S + 1), "cuda")
        if not chunked:
            seg._lists[("pieces", H)] = (None, None, False)
        c = {k: v.clone() for k, v in r.items()}
        y = _run_retention(c, H, dp, vp, dp, vp, seg, ctx.cuda())
        got.append((y, c["state"]))
    _close(got[0][0], got[1][0], BF16, 4e-3)
    _close(got[0][1], got[1][1], F32, 1e-4)


@dtypes
def test_retention_remembers(device, dtype):
    """One key that matches all queries: its value comes back from every
    later row, weaker by the decay, through chunks, pieces and slots."""
    D, n = 64, 700
    ctx = torch.arange(1, n + 1).int()
    g = torch.tensor([1.0, 0.998046875], dtype=torch.float64)
    for pos in (0, 15, 31, 32, 255, 256, 511, 600):
        ab = torch.zeros(n, 2 * 2 * (D + D), dtype=dtype, device="cuda")
        v = ab.view(n, 4, 2, D)
        v[:, 0, :, D - 1] = 1.0              # queries, number not rotated
        v[:, 3] = 3.0                        # gates
        v[:, 1, :, 8], v[:, 2, :, 7] = 0.5, 1.0
        v[pos, 1, :, D - 1], v[pos, 2, :, 3] = 100.0, 100.0
        table = _table({"base": 1e4, "dims": 4}, ctx)
        decay = torch.stack([g, g.log2()]).float().cuda()
        state = torch.zeros(2, 2, D, D, device="cuda")
        outs = []
        for a, b in ((0, 300), (300, 310), (310, 700)):
            seg = Segments.build([0], [b - a], [1], "cuda")
            outs.append(ops.retention(
                ab[a:b], 2, D, D, D, D, decay, table[a:b].contiguous(), 0.1,
                state, seg, ctx[a:b].cuda()))
        y = torch.cat(outs).view(n, 2, D).float().cpu()
        i = torch.arange(n)
        for h in range(2):
            # what is read out: value 3 of the matching key; the norm of a
            # vector with one number x is x / sqrt(x^2 / D + eps)
            x = torch.where(i >= pos, 100.0 * 100.0 / 8 * g[h].float()
                            ** (i - pos), 0.0)
            want = x / torch.sqrt(x * x / D + 0.1) * 3.0 / (
                1 + torch.exp(torch.tensor(-3.0)))
            _close(y[:, h, 3], want, dtype, 2e-2)
        S = state[1, 1, 3, D - 1].item()
        assert abs(S / (1250 * 100 / 100 * g[1].item() ** (n - 1 - pos))
                   - 1) < 1e-4


# ---- the model ---------------------------------------------------------------

@pytest.fixture(scope="module", params=DTYPES, ids=ids)
def case(request, device, tmp_path_factory):
    return cases.Case(tmp_path_factory.mktemp("k"), "cuda:0", request.param)


def test_residual_stream(case):
    cases.check_residuals(case)


def test_whole_prompt(case):
    cases.check_whole(case)


def test_first_tokens(case):
    cases.check_first_tokens(case)


def test_portions(case):
    cases.check_portions(case)


def test_mixed_batches(case):
    cases.check_batches(case)


def test_page_and_slot_reuse(case):
    cases.check_reuse(case)


def test_long_prompt(case):
    """Several pieces of a retention layer, many tiles of keys."""
    toks = case.tokens(900, 50)
    for cuts in ([900], [600, 1, 299]):
        case.passes(cases.run_cut(case.engine(tokens=1024), toks, cuts),
                    toks)


@dtypes
@pytest.mark.parametrize("rotated", [False, True])
def test_far_key(device, tmp_path, dtype, rotated):
    cases.check_far_key(tmp_path, "cuda:0", dtype, rotated=rotated)


@dtypes
def test_sink_and_gate(device, tmp_path, dtype):
    cases.check_sink_and_gate(tmp_path, "cuda:0", dtype)


@dtypes
def test_shared_latents(device, tmp_path, dtype):
    cases.check_shared_latents(tmp_path, "cuda:0", dtype)


@dtypes
def test_state_memory(device, tmp_path, dtype):
    cases.check_state_memory(tmp_path, "cuda:0", dtype)


@dtypes
def test_streams(device, tmp_path, dtype):
    cases.check_streams(tmp_path, "cuda:0", dtype)


def test_router(device, tmp_path):
    cases.check_router(tmp_path, "cuda:0", F32)


@dtypes
def test_other_sizes(device, tmp_path, dtype):
    cases.check_sizes(tmp_path, "cuda:0", dtype)


def test_greedy_generation(case):
    cases.check_greedy(case)


def test_greedy_generation_loop(case):
    cases.check_greedy(case, use_loop=True)


def test_long_decode(case):
    cases.check_long_decode(case)


def test_decode_graph_replays(case):
    """Captured decode steps against eager ones, replay after replay, with
    other work and other batches in between."""
    toks = case.tokens(60, 97)
    graph, eager = case.engine(), case.engine(use_graphs=False)
    a, b = [cases.common._Seq(i, []) for i in range(2)]
    cases.feed(graph, a, toks[:30])
    cases.feed(eager, b, toks[:30])
    for i in range(30, 60):
        got = cases.feed(graph, a, toks[i: i + 1])
        want = cases.feed(eager, b, toks[i: i + 1])
        assert cases.rel(got, want.double().cpu()) < cases.TOL[case.dtype]
        torch.cuda.synchronize()
        torch.randn(512, 512, device="cuda").sum().item()
        if i % 7 == 0:
            other = cases.common._Seq(9, [])
            cases.feed(graph, other, toks[: i - 20])
            graph.release(other)
    assert graph._graphs and graph.use_graphs


def test_listed_extensions_suffice(case, monkeypatch):
    """A step finds all of its kernels in the extensions that are compiled
    for this design."""
    from distllm_amd.build_ext import needed_for

    need = needed_for(str(case.path))
    native = ops._hip_ops
    monkeypatch.setattr(native, "modules", {
        k: v for k, v in native.modules.items() if k in need})
    assert set(native.modules) == set(need)
    toks = case.tokens(70, 101)
    case.passes(cases.run_cut(case.engine(), toks, [40, 28, 1, 1]), toks)


def test_trace_run_program(device, tmp_path):
    """bin/trace_run as a program, both dtypes."""
    import numpy as np

    root = Path(__file__).resolve().parents[1]
    c = cases.Case(tmp_path, "cuda:0", F32, seed=9)
    cases.decide(c.tensors, 9)
    from safetensors.torch import save_file
    save_file(c.tensors, str(c.path / "model.safetensors"))
    t1, t2 = c.tokens(70, 98), c.tokens(4, 99)
    steps = [
        {"step": 0, "entries": [{"id": "p", "tokens": t1[:50],
                                 "want": [49]}], "end": []},
        {"step": 1, "entries": [{"id": "q", "tokens": t2, "want": [0, 3]},
                                {"id": "p", "tokens": t1[50:69],
                                 "want": []}], "end": ["q"]},
        {"step": 2, "entries": [{"id": "p", "tokens": t1[69:],
                                 "want": [0]}], "end": ["p"]},
    ]
    for dtype in DTYPES:
        out = tmp_path / str(dtype)
        out.mkdir()
        run = subprocess.run(
            [sys.executable, str(root / "bin" / "trace_run"), "--model",
             str(c.path), "--dtype", str(dtype).split(".")[1], "--out",
             str(out), "--max-tokens", "128"],
            input="\n".join(json.dumps(s) for s in steps) + "\n",
            capture_output=True, text=True, timeout=100,
            env=dict(os.environ))
        assert run.returncode == 0, run.stderr[-2000:]
        assert [x for x in run.stdout.splitlines() if x.startswith("done")] \
            == ["done 0", "done 1", "done 2"]
        got = torch.from_numpy(np.concatenate(
            [np.fromfile(out / f"{i}.f32", "<f4") for i in range(3)]))
        want = torch.cat([c.want(t1)[49:50], c.want(t2)[[0, 3]],
                          c.want(t1)[69:]])
        assert cases.rel(got.view(4, -1), want) < cases.TOL[dtype]
