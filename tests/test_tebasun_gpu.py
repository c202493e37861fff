"""Tebasun on the GPU: the HIP kernels against fp32 references of the same
op, and the engine path in bf16 and fp32 against the plain
implementation."""

import json
import os
import subprocess
import sys
from pathlib import Path

import pytest
import torch

import tebasun_cases as cases
import tebasun_oracle as oracle
from distllm_amd import ops
from distllm_amd.engine.step import PromptBlocks, Segments, StepBatch
from distllm_amd.ops import torch_ref
from test_bufulorn_gpu import _close, _i32, _pages, _rand, _tables

pytestmark = pytest.mark.gpu

F32, BF16 = torch.float32, torch.bfloat16
DTYPES = [BF16, F32]
ids = {BF16: "bf16", F32: "fp32"}.get
dtypes = pytest.mark.parametrize("dtype", DTYPES, ids=ids)


# ---- kernels ---------------------------------------------------------------

@dtypes
@pytest.mark.parametrize("M, W, n", [(1, 64, 1), (7, 320, 300),
                                     (5, 1024, 1024), (3, 1088, 1030),
                                     (9, 4096, 4096), (2, 8192, 8000),
                                     (2, 12288, 12288)])
def test_residual_step(device, dtype, M, W, n):
    vecs = [_rand(W, seed=i) for i in range(5)]
    table, y = _rand(11, W, seed=6, dtype=dtype), _rand(M, W, seed=7,
                                                        dtype=dtype)
    x0 = _rand(M, W, seed=8) * torch.logspace(-4, 1, M).cuda()[:, None]
    for t in vecs + [table, y, x0]:
        t[..., n:] = 0
    bias, w, vec, aw, ab = vecs
    alpha = torch.tensor([0.6], device="cuda")
    tok = torch.arange(M, device="cuda") % 11
    embed, act = (tok, table, 2.5), (aw, ab, alpha)
    for kw in ({"embed": embed, "fresh": True, "act": act},
               {"embed": embed, "fresh": True, "act": act, "vec": vec},
               {"y": y, "bias": bias, "act": act}, {"y": y},
               {"y": y, "rms": (w, n, 0.01), "act": act},
               {"y": y, "rms": (w, n, 0.01), "act": act, "vec": vec,
                "embed": embed},
               {"act": act, "dtype": dtype},
               {"vec": vec, "dtype": dtype}):
        x, xr = x0.clone(), x0.clone()
        h = ops.residual_step(x, **kw)
        args = {"y": None, "bias": None, "rms": None, "embed": None,
                "vec": None, "act": None, "fresh": False, **kw, "dtype": F32}
        want = torch_ref.residual_step(xr, **args)
        assert h.dtype == dtype
        _close(x, xr, F32)
        _close(h, want, dtype)


@dtypes
@pytest.mark.parametrize("M, dim, K", [(1, 16, 64), (37, 70, 256),
                                       (300, 100, 128), (256, 1, 1024)])
def test_gated_rows(device, dtype, M, dim, K):
    N = (dim + 63) // 64 * 64
    x, w = _rand(M, K, dtype=dtype), _rand(N, K, seed=1) * 0.1
    w[dim:] = 0
    w = w.to(dtype)
    table = _rand(9, 3 * dim, seed=2, dtype=dtype)
    tok = torch.arange(M, device="cuda") % 9
    got = ops.gated_rows(x, w, tok, table, 2 * dim, dim)
    z = (x.double() @ w.double().t()).cpu()[:, :dim]
    want = oracle.gelu_tanh(z) * table.double().cpu()[tok.cpu()][:, 2 * dim:]
    _close(got[:, :dim], want, dtype, 4e-2 if dtype == BF16 else None)
    assert not got[:, dim:].any()


def test_rotation_table(device):
    """Positions of a long context keep their angles to 32-bit rounding."""
    f, mult = oracle.frequencies(oracle.rotation(64, 1e4, 16.0, 4096, 32., 1.))
    ctx = _i32(1, 2, 5000, 131072, 1048576, 0)
    got = ops.rotation_table(ctx.cuda(), f.cuda(), mult).cpu()
    want = torch_ref.rotation_table(ctx, f, mult)
    assert (got - want).abs().max() < 1e-6


@dtypes
@pytest.mark.parametrize("dp, dim, half, H, long", [
    (64, 33, 8, 6, 70), (128, 128, 64, 6, 70), (128, 100, 21, 6, 70),
    (256, 200, 100, 6, 70), (320, 300, 2, 6, 70), (576, 560, 280, 2, 40),
    (64, 64, 16, 30, 2301), (128, 100, 32, 30, 2301)])
def test_rotary_prep(device, dtype, dp, dim, half, H, long):
    """Runs of rows in one page, whole pages, single rows, padding rows;
    what the step does not bring stays."""
    G = 2
    lens = [long, 7, 33]
    nb, bt = _tables(lens)
    ctx = _i32(*range(14, long + 1), 7, 0, *range(1, 34), 0)
    row_seq = _i32(*[0] * (long - 13), 1, 0, *[2] * 33, 0)
    M = len(ctx)
    wide = _rand(M, (H + G) * dp + 128, dtype=dtype)
    ab = wide[:, 64: 64 + (H + G) * dp]  # columns of a wider product
    for h in range(H + G):
        ab[:, h * dp + dim: (h + 1) * dp] = 0
    wq, wk = _rand(dp, seed=1), _rand(dp, seed=2)
    f, mult = oracle.frequencies(oracle.rotation(2 * half, 500.0))
    table = ops.rotation_table(ctx.cuda(), f.cuda(), mult)
    kp = torch.full((nb, G, 16, dp), 3.0, dtype=dtype, device="cuda")
    vpg = torch.full((nb, G, dp, 16), 3.0, dtype=dtype, device="cuda")
    rk, rv = kp.cpu().float(), vpg.cpu().float()
    q = ops.rotary_prep(ab, H, G, dp, dim, wq, wk, 1e-3, table, (kp, vpg),
                        bt.cuda(), row_seq.cuda(), ctx.cuda())
    want = torch_ref.rotary_prep(ab.cpu().float(), H, G, dp, dim, wq.cpu(),
                                 wk.cpu(), 1e-3, table.cpu(), (rk, rv), bt,
                                 row_seq, ctx)
    _close(q, want, dtype)
    _close(kp, rk, dtype)
    assert torch.equal(vpg.cpu().float(), rv)


@dtypes
@pytest.mark.parametrize("D", [64, 128, 256, 320])
@pytest.mark.parametrize("H, G", [(1, 1), (4, 4), (8, 2), (34, 2)])
def test_sink_rows(device, dtype, D, H, G):
    """Single-token rows: heads per key head up to more than a tile, every
    split of the keys, sinks that take all or nothing."""
    lens = [1, 15, 16, 33, 200, 517]
    kp, vp, bt = _pages(lens, G, D, D, dtype)
    row_seq = _i32(5, 0, 1, 2, 3, 4, 5, 4, 0)
    ctx = _i32(517, 1, 15, 16, 33, 200, 300, 97, 0)
    q = _rand(9, H, D, seed=4, dtype=dtype)
    sink = _rand(H, seed=5) * 3
    if H > 2:
        sink[1], sink[2] = 80.0, -90.0
    scale = 2.0 / D ** 0.5
    want = torch_ref.sink_attn_rows(
        q.cpu().float(), kp.cpu().float(), vp.cpu().float(),
        torch.zeros(9, H * D), bt, row_seq, ctx, scale, sink.cpu(), 0.6)
    for nsplit in (0, 1, 3):
        wide = torch.full((9, H * D + 64), 7.0, dtype=dtype, device="cuda")
        ops.sink_attn_rows(q, kp, vp, wide[:, 64:], bt.cuda(),
                           row_seq.cuda(), ctx.cuda(), scale, sink, 0.6,
                           nsplit)
        _close(wide[:, 64:], want, dtype)
        assert not wide[8, 64:].any()  # a padding row sees nothing
        assert (wide[:, :64] == 7).all()


@pytest.mark.parametrize("D", [64, 128, 256])
@pytest.mark.parametrize("H, G", [(2, 2), (6, 2)])
def test_sink_prompts(device, D, H, G):
    """Portions after their cached part, among other rows."""
    starts, rows = [0, 137, 64, 111], [130, 33, 1, 300]
    kp, vp, bt = _pages([s + n for s, n in zip(starts, rows)], G, D, D, BF16)
    M = 5 + sum(rows)
    q = _rand(M, H, D, seed=4, dtype=BF16)
    sink = torch.linspace(-60.0, 6.0, H).cuda()
    scale = 2.0 / D ** 0.5
    batch = StepBatch(tokens=torch.zeros(M, device="cuda"), ctx=None,
                      row_seq=None, block_table=None, n_folded=5,
                      portions=[(i, s, n) for i, (s, n) in
                                enumerate(zip(starts, rows))])
    p = batch.prompt_blocks(1 << 30)
    wide = torch.full((M, H * D + 64), 7.0, dtype=BF16, device="cuda")
    ops.sink_attn_prompts(q, kp, vp, wide[:, : H * D], bt.cuda(), p, scale,
                          sink, 1.7)
    want = torch_ref.sink_attn_prompts(
        q.cpu().float(), kp.cpu().float(), vp.cpu().float(),
        torch.full((M, H * D), 7.0), bt,
        PromptBlocks(p.portions.cpu(), p.blocks.cpu()), scale, sink.cpu(),
        1.7)
    _close(wide[:, : H * D], want, BF16)
    assert (wide[:5] == 7).all() and (wide[:, H * D:] == 7).all()


@dtypes
def test_sink_far_key(device, dtype):
    """One matching key, at page and tile borders: its value comes back
    from every later place and from none before."""
    D, T = 64, 400
    kp, vp, bt = _pages([T], 1, D, D, dtype)
    kp, vp = kp * 0.01, vp * 0
    q = torch.full((T, 3, D), 4.0, dtype=dtype, device="cuda")
    sink = torch.tensor([-20.0, 0.0, 4000.0], device="cuda")
    ctx = torch.arange(1, T + 1).int().cuda()
    seq = torch.zeros(T, dtype=torch.int32, device="cuda")
    i = torch.arange(T)
    batch = StepBatch(tokens=q, ctx=None, row_seq=None, block_table=None,
                      n_folded=0, portions=[(0, 0, T)])
    for pos in (0, 15, 16, 31, 32, 63, 64, 127, 255, 256, 399):
        k, v = kp.clone(), vp.clone()
        k[bt[0, pos // 16].item(), :, pos % 16] = 4.0
        v[bt[0, pos // 16].item(), :, :, pos % 16] = 5.0
        for nsplit in (1, 2, 0):
            out = torch.zeros(T, 3 * D, dtype=dtype, device="cuda")
            if nsplit or dtype == F32:
                ops.sink_attn_rows(q, k, v, out, bt.cuda(), seq, ctx, 1.0,
                                   sink, 1.0, nsplit)
            else:
                ops.sink_attn_prompts(q, k, v, out, bt.cuda(),
                                      batch.prompt_blocks(1 << 30), 1.0,
                                      sink, 1.0)
            got = out.float().cpu().view(T, 3, D).mean(2)
            assert torch.equal(got[:, 0] > 4.9, i >= pos), pos
            assert torch.equal(got[:, 1] > 4.9, i >= pos), pos
            assert got[i < pos].abs().sum() < 1e-3
            assert not got[:, 2].any()


def _batch_of(rows, starts, pad=3):
    """Row offsets, ctx, row_seq and slots of segments."""
    S = len(rows)
    row0 = torch.tensor([0] + rows).cumsum(0)[:-1].int()
    slots = torch.arange(S).flip(0).int() + 1
    ctx = torch.cat([torch.arange(s + 1, s + n + 1)
                     for s, n in zip(starts, rows)]
                    + [torch.zeros(pad)]).int()
    row_seq = torch.cat([torch.full((n,), i) for i, n in enumerate(rows)]
                        + [torch.zeros(pad)]).int()
    return Segments(row0, torch.tensor(rows).int(), slots, max(rows)), \
        ctx, row_seq


def _delta_inputs(H, G, dp, vp, dim, vdim, taps, M, slots, dtype, seed=0):
    C = 2 * G * dp + H * vp
    r = {"ab": _rand(M, C + 64, seed=seed, dtype=dtype),
         "ag": _rand(M, H * (dp + vp), seed=seed + 1, dtype=dtype),
         "conv_w": _rand(taps, C, seed=seed + 2) * 0.6,
         "a_log": _rand(H, seed=seed + 3) * 0.5 - 1,
         "dt": _rand(H * dp, seed=seed + 4) * 1.5 - 1,
         "norm": _rand(vp, seed=seed + 5),
         "state": _rand(slots, H, vp, dp, seed=seed + 6),
         "conv": _rand(slots, taps - 1, C, seed=seed + 7, dtype=dtype)}
    cols = torch.arange(C)
    pad = torch.where(cols < 2 * G * dp, cols % dp >= dim,
                      (cols - 2 * G * dp) % vp >= vdim).cuda()
    r["ab"][:, :C][:, pad] = 0
    r["conv"][..., pad] = 0
    r["norm"][vdim:] = 0
    r["state"][:, :, vdim:], r["state"][..., dim:] = 0, 0
    return r


def _run_delta(r, H, G, dp, vp, dim, vdim, seg, row_seq, ctx, out, ref):
    f = torch_ref if ref else ops
    return f.channel_delta(r["ab"], r["ag"], H, G, dp, vp, dim, vdim,
                           r["conv_w"], r["a_log"], r["dt"], r["norm"], 1e-6,
                           1e-5, 0.8, r["state"], r["conv"], seg, row_seq,
                           ctx, out)


@dtypes
@pytest.mark.parametrize("H, G, dp, vp, taps, rows", [
    (2, 1, 64, 64, 4, [1, 1, 1]), (4, 2, 128, 128, 4, [3, 150, 1, 2]),
    (3, 3, 64, 128, 1, [70, 5]), (2, 1, 128, 64, 2, [64, 65, 63]),
    (4, 1, 64, 256, 7, [33, 200]), (2, 2, 256, 64, 3, [40, 129]),
    (2, 1, 256, 256, 4, [66, 2]), (2, 2, 128, 256, 4, [300]),
    (6, 2, 128, 128, 4, [16, 17, 32, 31, 1]), (64, 8, 64, 128, 4, [95]),
    (32, 32, 128, 128, 4, [33] * 8)])
def test_channel_delta(device, dtype, H, G, dp, vp, taps, rows):
    """Segments of one row to several chunks, from the start or going on,
    with padding rows behind; the sequence's slots and no others change."""
    starts = [(0, 5, 2, 0)[i % 4] for i in range(len(rows))]
    seg, ctx, row_seq = _batch_of(rows, starts)
    M, S, dim, vdim = len(ctx), len(rows), dp - 7, vp - 3
    r = _delta_inputs(H, G, dp, vp, dim, vdim, taps, M, S + 2, dtype)
    for i, s in enumerate(starts):  # no inputs before a sequence's start
        r["conv"][S - i, : max(0, taps - 1 - s)] = 0
    host = {k: v.cpu().clone() for k, v in r.items()}
    want = _run_delta(host, H, G, dp, vp, dim, vdim, seg, row_seq, ctx,
                      torch.zeros(M, H * vp, dtype=dtype), True)
    before = r["state"].clone()
    dseg = Segments.build(seg.row0.tolist(), rows, seg.slot.tolist(), "cuda")
    wide = torch.full((M, H * vp + 64), 7.0, dtype=dtype, device="cuda")
    got = wide[:, 64:]
    _run_delta(r, H, G, dp, vp, dim, vdim, dseg, row_seq.cuda(), ctx.cuda(),
               got, False)
    n = sum(rows)
    _close(got[:n], want[:n], dtype, 2e-2 if dtype == BF16 else 1e-4)
    assert (wide[:, :64] == 7).all()
    _close(r["state"], host["state"], F32, 1e-2 if dtype == BF16 else 1e-4)
    for i, s in enumerate(seg.slot.tolist()):
        live = min(taps - 1, starts[i] + rows[i])
        if live:
            assert torch.equal(r["conv"][s, -live:].cpu(),
                               host["conv"][s, -live:])
    assert torch.equal(r["state"][0], before[0])
    assert torch.equal(r["state"][S + 1], before[S + 1])


@pytest.mark.parametrize("H, G, dp, vp, rows", [
    (4, 2, 128, 128, [200, 17, 3]), (64, 64, 64, 64, [64, 31]),
    (3, 1, 256, 256, [70]), (32, 8, 128, 128, [33] * 8)])
@pytest.mark.parametrize("rates", [(-6, -2), (-6, 3), (2, 5)])
def test_channel_chunks(device, H, G, dp, vp, rows, rates):
    """The chunked form against the token-by-token form, both in fp32
    behind the same bf16 inputs. Weak decays are split into two factors,
    strong ones are formed pair by pair; heads with one and the other."""
    M, S = sum(rows), len(rows)
    r = _delta_inputs(H, G, dp, vp, dp, vp, 4, M, S + 1, BF16)
    r["a_log"] = torch.linspace(*rates, H).cuda()
    row0 = torch.tensor([0] + rows).cumsum(0)[:-1].tolist()
    ctx = torch.cat([torch.arange(n) + 1 + 4 * (i % 2)
                     for i, n in enumerate(rows)]).int().cuda()
    row_seq = torch.cat([torch.full((n,), i)
                         for i, n in enumerate(rows)]).int().cuda()
    got = []
    for chunked in (True, False):
        seg = Segments.build(row0, rows, range(1, S + 1), "cuda")
        if not chunked:
            seg.longs = seg.chunks = None
        c = {k: v.clone() for k, v in r.items()}
        y = torch.zeros(M, H * vp, dtype=BF16, device="cuda")
        _run_delta(c, H, G, dp, vp, dp, vp, seg, row_seq, ctx, y, False)
        got.append((y, c["state"], c["conv"]))
    assert torch.isfinite(got[0][0]).all()
    _close(got[0][0], got[1][0], BF16, 4e-3)
    _close(got[0][1], got[1][1], F32, 1e-4)
    assert torch.equal(got[0][2], got[1][2])


def _lru_inputs(blocks, bs, taps, M, slots, dtype, seed=0):
    C = (blocks * bs + 63) // 64 * 64
    r = {"ab": _rand(M, 2 * C, seed=seed, dtype=dtype),
         "conv_w": _rand(taps, C, seed=seed + 1) * 0.6,
         "conv_b": _rand(C, seed=seed + 2) * 0.3,
         "gates": (_rand(2, blocks, bs, bs, seed=seed + 3) / bs ** 0.5).to(
             dtype),
         "gates_b": _rand(2, C, seed=seed + 4),
         "decay": -8 * torch.nn.functional.softplus(
             _rand(C, seed=seed + 5) * 2 - 3),
         "state": _rand(slots, C, seed=seed + 6),
         "conv": _rand(slots, taps - 1, C, seed=seed + 7, dtype=dtype)}
    for k, v in r.items():  # columns of padding
        if k not in ("gates", "decay"):
            v.view(-1, C)[:, blocks * bs:] = 0
    return r


@dtypes
@pytest.mark.parametrize("blocks, bs, taps, rows", [
    (2, 32, 4, [1, 1, 1]), (3, 32, 4, [3, 150, 1, 2]), (1, 64, 1, [70, 5]),
    (2, 96, 2, [64, 65, 63]), (5, 64, 7, [33, 200]), (1, 256, 3, [40, 129]),
    (4, 256, 4, [66, 2, 17]), (16, 64, 4, [16, 17, 64, 31, 1, 400]),
    (2, 160, 5, [1] * 40), (2, 384, 4, [70, 3]), (1, 320, 2, [65, 1]),
    (1, 512, 4, [130, 16]), (3, 128, 4, [64, 40])])
def test_gated_lru(device, dtype, blocks, bs, taps, rows):
    """Segments of one row to several chunks, from the start or going on,
    with padding rows behind; the sequence's slots and no others change."""
    starts = [(0, 5, 2, 0)[i % 4] for i in range(len(rows))]
    seg, ctx, row_seq = _batch_of(rows, starts)
    M, S, n = len(ctx), len(rows), sum(rows)
    r = _lru_inputs(blocks, bs, taps, M, S + 2, dtype)
    for i, s in enumerate(starts):
        r["conv"][S - i, : max(0, taps - 1 - s)] = 0
    host = {k: v.cpu().clone() for k, v in r.items()}
    before = r["state"].clone()
    dseg = Segments.build(seg.row0.tolist(), rows, seg.slot.tolist(), "cuda")
    want = torch_ref.gated_lru(*host.values(), seg, row_seq, ctx)
    got = ops.gated_lru(*r.values(), dseg, row_seq.cuda(), ctx.cuda(), 64)
    _close(got[:n], want[:n], dtype, 2e-2 if dtype == BF16 else 1e-4)
    C = r["decay"].numel()
    _close(r["state"], host["state"], F32, 1e-2 if dtype == BF16 else 1e-4)
    assert not got[:n, blocks * bs:].any() or C == blocks * bs
    for i, s in enumerate(seg.slot.tolist()):
        live = min(taps - 1, starts[i] + rows[i])
        if live:
            assert torch.equal(r["conv"][s, -live:].cpu(),
                               host["conv"][s, -live:])
    assert torch.equal(r["state"][0], before[0])
    assert torch.equal(r["state"][S + 1], before[S + 1])


@pytest.mark.parametrize("rows", [[200, 17, 3], [64, 65], [1000]])
@pytest.mark.parametrize("shift", [-14.0, -3.0, 3.0])
def test_lru_chunks(device, rows, shift):
    """The chunked recurrence against the one row by row, behind the same
    bf16 inputs: decays from nearly none to nearly everything."""
    M, S = sum(rows), len(rows)
    r = _lru_inputs(4, 64, 4, M, S + 1, BF16)
    r["decay"] = -8 * torch.nn.functional.softplus(
        _rand(256, seed=9) + shift)
    row0 = torch.tensor([0] + rows).cumsum(0)[:-1].tolist()
    ctx = torch.cat([torch.arange(n) + 1 + 4 * (i % 2)
                     for i, n in enumerate(rows)]).int().cuda()
    row_seq = torch.cat([torch.full((n,), i)
                         for i, n in enumerate(rows)]).int().cuda()
    got = []
    for chunked in (True, False):
        seg = Segments.build(row0, rows, range(1, S + 1), "cuda")
        if not chunked:
            seg._lists[64] = (None, None)
        c = {k: v.clone() for k, v in r.items()}
        y = ops.gated_lru(*c.values(), seg, row_seq, ctx, 64)
        got.append((y, c["state"]))
    _close(got[0][0], got[1][0], BF16, 4e-3)
    _close(got[0][1], got[1][1], F32, 1e-4)


# ---- the model ---------------------------------------------------------------

@pytest.fixture(scope="module", params=DTYPES, ids=ids)
def case(request, device, tmp_path_factory):
    return cases.Case(tmp_path_factory.mktemp("t"), "cuda:0", request.param)


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


@dtypes
def test_far_key(device, tmp_path, dtype):
    cases.check_far_key(tmp_path, "cuda:0", dtype)


@dtypes
def test_sink(device, tmp_path, dtype):
    cases.check_sink(tmp_path, "cuda:0", dtype)


@dtypes
@pytest.mark.parametrize("kind", ["rglru", "delta"])
def test_state_memory(device, tmp_path, dtype, kind):
    cases.check_state_memory(tmp_path, "cuda:0", dtype, kind)


@dtypes
def test_strong_decay(device, tmp_path, dtype):
    cases.check_strong_decay(tmp_path, "cuda:0", dtype)


@dtypes
def test_loop(device, tmp_path, dtype):
    cases.check_loop(tmp_path, "cuda:0", dtype)


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
    a, b = [cases._Seq(i, []) for i in range(2)]
    cases.feed(graph, a, toks[:30])
    cases.feed(eager, b, toks[:30])
    for i in range(30, 60):
        got = cases.feed(graph, a, toks[i: i + 1])
        want = cases.feed(eager, b, toks[i: i + 1])
        assert cases.rel(got, want.double().cpu()) < cases.TOL[case.dtype]
        torch.cuda.synchronize()
        torch.randn(512, 512, device="cuda").sum().item()
        if i % 7 == 0:
            other = cases._Seq(9, [])
            cases.feed(graph, other, toks[: i - 20])
            graph.release(other)
    assert graph._graphs and graph.use_graphs


def test_trace_run_program(device, tmp_path):
    """bin/trace_run as a program, both dtypes."""
    import numpy as np

    root = Path(__file__).resolve().parents[1]
    c = cases.Case(tmp_path, "cuda:0", F32, seed=9)
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
