"""Bufulorn on the GPU: the HIP kernels against fp32 references of the
same op, and the engine path in bf16 and fp32 against the plain
implementation."""

import json
import os
import subprocess
import sys
from pathlib import Path

import pytest
import torch

import bufulorn_cases as cases
import bufulorn_oracle as oracle
from distllm_amd import ops
from distllm_amd.engine.step import PromptBlocks, Segments, StepBatch
from distllm_amd.ops import torch_ref

pytestmark = pytest.mark.gpu

F32, BF16 = torch.float32, torch.bfloat16
DTYPES = [BF16, F32]
ids = {BF16: "bf16", F32: "fp32"}.get


@pytest.fixture(scope="module", params=DTYPES, ids=ids)
def case(request, device, tmp_path_factory):
    return cases.Case(tmp_path_factory.mktemp("b"), "cuda:0", request.param,
                      gain=1.5 if request.param == F32 else 1.0)


def test_whole_prompt(case):
    cases.check_whole(case)


def test_residual_stream(case):
    cases.check_residuals(case)


def test_first_tokens(case):
    cases.check_first_tokens(case)


def test_portions(case):
    cases.check_portions(case)


def test_mixed_batches(case):
    cases.check_batches(case)


def test_page_and_slot_reuse(case):
    cases.check_reuse(case)


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("size", [1, 2, 16, 33, 130])
def test_chunk_edges(device, tmp_path, dtype, size):
    c = cases.edge_case(tmp_path, "cuda:0", dtype, size)
    if dtype == BF16 and size > 33:
        # one key of many: the kernels' own tests make it stand out
        toks = c.tokens(300, 1)
        got = cases.run_cut(c.engine(), toks, [200, 3, 40, 1])
        assert cases.rel(got, c.want(toks)) < cases.TOL[BF16]
    else:
        cases.check_edges(c, 100 if size < 100 else 180)


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
def test_state_memory(device, tmp_path, dtype):
    cases.check_state_memory(tmp_path, "cuda:0", dtype)


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
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


# ---- kernels ---------------------------------------------------------------

def _rand(*shape, seed=0, dtype=F32):
    g = torch.Generator().manual_seed(seed)
    return torch.randn(*shape, generator=g).to(dtype).to("cuda")


def _i32(*v):
    return torch.tensor(v, dtype=torch.int32)


def _close(got, want, dtype, tol=None):
    got, want = got.float().cpu(), want.float().cpu()
    assert torch.isfinite(got).all()
    scale = want.pow(2).mean().sqrt().clamp_min(1e-6)
    d = (got - want).abs()
    if dtype == BF16:  # the output's own rounding comes on top
        d = d - want.abs() / 128
    err = (d.max() / scale).item()
    assert err < (tol or (2e-2 if dtype == BF16 else 2e-5)), err


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("M, W, n", [(1, 64, 1), (7, 320, 300),
                                     (5, 1024, 1024), (3, 1088, 1030),
                                     (9, 4096, 4096), (2, 8192, 8000),
                                     (2, 12288, 12288)])
def test_residual_norms(device, dtype, M, W, n):
    v = [_rand(W, seed=i) for i in range(4)]
    table, pos = _rand(11, W, dtype=dtype), _rand(6, W, seed=5, dtype=dtype)
    for t in v + [table, pos]:
        t[..., n:] = 0
    tok = torch.arange(M, device="cuda") % 11
    ctx = (torch.arange(M, device="cuda") % 7).int()
    h, x = ops.embed_positions(tok, ctx, table, pos)
    h_ref, x_ref = torch_ref.embed_positions(tok, ctx, table, pos)
    assert torch.equal(x, x_ref) and torch.equal(h, h_ref)
    for top in (0, 3):
        y = _rand(M * max(top, 1), W, seed=7, dtype=dtype)
        y[:, n:] = 0
        mix = None
        if top:
            mix = torch.rand(M, top, device="cuda") + 0.1
            mix[M // 2] = 0
            y[M // 2 * top: (M // 2 + 1) * top] = float("nan")
        for final in (None, (v[2], v[3])):
            h = ops.layer_norm_add(y, x, v[0], v[1], n, 0.01, final, mix)
            h_ref = torch_ref.layer_norm_add(y.float(), x_ref, v[0], v[1], n,
                                             0.01, final, mix)
            _close(x, x_ref, F32)
            _close(h, h_ref, dtype)


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("M, ff", [(1, 64), (37, 448), (300, 1024)])
def test_xielu(device, dtype, M, ff):
    x = _rand(M, 256, dtype=dtype)
    w = (_rand(ff, 256, seed=1) * 0.15).to(dtype)
    act = torch.tensor([-0.7, 0.9], device="cuda")
    z = (x.double() @ w.double().t()).cpu()
    want = oracle.xielu(z, *act.double().cpu())
    # (in bf16 the product is rounded on its way to the activation)
    _close(ops.up_xielu(x, w, act), want, dtype,
           4e-2 if dtype == BF16 else None)


def _tables(lens, blk=16, seed=0):
    """Page tables with the pages of sequences interleaved."""
    pages = [(n + blk - 1) // blk for n in lens]
    g = torch.Generator().manual_seed(seed)
    order = torch.randperm(sum(pages) + 2, generator=g).int()
    bt = torch.zeros(len(lens), max(pages) + 1, dtype=torch.int32)
    at = 0
    for i, p in enumerate(pages):
        bt[i, :p] = order[at: at + p]
        at += p
    return sum(pages) + 2, bt


def _pages(lens, G, dk, dv, dtype, seed=0):
    nb, bt = _tables(lens, seed=seed)
    return (_rand(nb, G, 16, dk, seed=seed + 1, dtype=dtype),
            _rand(nb, G, dv, 16, seed=seed + 2, dtype=dtype), bt)


HEADS = [(1, 1), (4, 4), (8, 2), (20, 1), (34, 2)]


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("dk, dv", [(64, 64), (128, 64), (64, 128),
                                    (128, 128), (256, 128), (128, 256),
                                    (256, 256), (320, 64)])
@pytest.mark.parametrize("H, G", HEADS)
def test_attn_rows(device, dtype, dk, dv, H, G):
    """Single-token rows: heads per key head up to more than a tile, every
    split of the keys, chunks from one key to everything."""
    lens = [1, 15, 16, 33, 200, 517]
    kp, vp, bt = _pages(lens, G, dk, dv, dtype)
    row_seq = _i32(5, 0, 1, 2, 3, 4, 5, 4, 0)
    ctx = _i32(517, 1, 15, 16, 33, 200, 300, 97, 0)
    q = _rand(9, H, dk, seed=4, dtype=dtype)
    ab = _rand(9, 64 + H * dv, seed=5, dtype=dtype)
    dist = torch.rand(2, H, device="cuda") + 0.1
    scale = 2.0 / dk ** 0.5
    for chunk in (1, 31, 64, 200, 10 ** 12):
        want = torch_ref.paged_attn_rows(
            q.cpu().float(), kp.cpu().float(), vp.cpu().float(),
            ab.cpu().float(), 64, torch.zeros(9, H, dv), bt, row_seq, ctx,
            chunk, scale, 5.0, dist.cpu())
        for nsplit in (0, 1, 3):
            out = torch.full((9, H, dv), 7.0, dtype=dtype, device="cuda")
            got = ops.paged_attn_rows(
                q, kp, vp, ab, 64, out, bt.cuda(), row_seq.cuda(),
                ctx.cuda(), chunk, scale, 5.0, dist, nsplit)
            _close(got, want, dtype)
            assert not got[8].any()  # a padding row sees nothing


@pytest.mark.parametrize("dk, dv", [(64, 64), (64, 128), (128, 64),
                                    (128, 128), (256, 64), (128, 256),
                                    (256, 256)])
@pytest.mark.parametrize("H, G", [(2, 2), (6, 2)])
def test_attn_prompts(device, dk, dv, H, G):
    """Portions after their cached part, among other rows."""
    starts, rows = [0, 137, 64, 111], [130, 33, 1, 300]
    kp, vp, bt = _pages([s + n for s, n in zip(starts, rows)], G, dk, dv,
                        BF16)
    M = 5 + sum(rows)
    q = _rand(M, H, dk, seed=4, dtype=BF16)
    ab = _rand(M, H * dv + 64, seed=5, dtype=BF16)
    dist = torch.rand(2, H, device="cuda") + 0.1
    scale = 2.0 / dk ** 0.5
    batch = StepBatch(tokens=torch.zeros(M, device="cuda"), ctx=None,
                      row_seq=None, block_table=None, n_folded=5,
                      portions=[(i, s, n) for i, (s, n) in
                                enumerate(zip(starts, rows))])
    for chunk in (1, 2, 64, 97, 128, 300, 10 ** 9):
        p = batch.prompt_blocks(chunk)
        out = torch.full((M, H, dv), 7.0, dtype=BF16, device="cuda")
        ops.paged_attn_prompts(q, kp, vp, ab, 0, out, bt.cuda(), p, chunk,
                               scale, 5.0, dist)
        want = torch_ref.paged_attn_prompts(
            q.cpu().float(), kp.cpu().float(), vp.cpu().float(),
            ab.cpu().float(), 0, torch.full((M, H, dv), 7.0), bt,
            PromptBlocks(p.portions.cpu(), p.blocks.cpu()), chunk, scale,
            5.0, dist.cpu())
        _close(out, want, BF16)
        assert (out[:5] == 7).all()


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("D", [64, 128])
def test_far_key(device, dtype, D):
    """One matching key, at page and tile borders and at the edges of a
    chunk: its value comes back in its whole chunk and nowhere else, for
    decoded rows and prompt rows."""
    size, T = 150, 400
    kp, vp, bt = _pages([T], 1, D, D, dtype)
    kp, vp = kp * 0.01, vp * 0
    ab = torch.full((T, 3 * D), 30.0, dtype=dtype, device="cuda")
    dist = torch.tensor([[0.5] * 3, [0.2] * 3], device="cuda")
    q = torch.full((T, 3, D), 4.0, dtype=dtype, device="cuda")
    ctx = torch.arange(1, T + 1).int().cuda()
    seq = torch.zeros(T, dtype=torch.int32, device="cuda")
    i = torch.arange(T)
    batch = StepBatch(tokens=q, ctx=None, row_seq=None, block_table=None,
                      n_folded=0, portions=[(0, 0, T)])
    for pos in (0, 15, 16, 31, 32, 63, 64, 127, 149, 150, 255, 256, 299,
                300, 399):
        k, v = kp.clone(), vp.clone()
        k[bt[0, pos // 16].item(), :, pos % 16] = 4.0
        v[bt[0, pos // 16].item(), :, :, pos % 16] = 5.0
        seen = (i >= pos) & (i // size == pos // size)
        for nsplit in (1, 2):
            out = torch.zeros(T, 3, D, dtype=dtype, device="cuda")
            ops.paged_attn_rows(q, k, v, ab, 0, out, bt.cuda(), seq, ctx,
                                size, 1.0, 30.0, dist, nsplit)
            got = out.float().cpu().mean((1, 2))
            assert torch.equal(got > 4.9, seen), pos
            assert got[~seen].abs().max() < 1e-3
        if dtype == BF16:
            out = torch.zeros(T, 3, D, dtype=dtype, device="cuda")
            ops.paged_attn_prompts(q, k, v, ab, 0, out, bt.cuda(),
                                   batch.prompt_blocks(size), size, 1.0,
                                   30.0, dist)
            got = out.float().cpu().mean((1, 2))
            assert torch.equal(got > 4.9, seen), pos
            assert got[~seen].abs().max() < 1e-3


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("dp, dim, vp, H, long", [
    (64, 33, 128, 6, 70), (128, 128, 64, 6, 70), (256, 200, 256, 6, 70),
    (320, 300, 64, 6, 70), (64, 64, 64, 30, 2301), (128, 100, 256, 30, 2301)])
def test_attn_prep(device, dtype, dp, dim, vp, H, long):
    """Runs of rows in one page, whole pages, single rows, padding rows;
    what the step does not bring stays."""
    G = 2
    lens = [long, 7, 33]
    nb, bt = _tables(lens)
    ctx = _i32(*range(14, long + 1), 7, 0, *range(1, 34), 0)
    row_seq = _i32(*[0] * (long - 13), 1, 0, *[2] * 33, 0)
    M = len(ctx)
    ab = _rand(M, H * dp + G * (dp + vp) + 64, dtype=dtype)
    for h in range(H + G):
        ab[:, h * dp + dim: (h + 1) * dp] = 0
    wq, wk = _rand(dp, seed=1), _rand(dp, seed=2)
    kp = torch.full((nb, G, 16, dp), 3.0, dtype=dtype, device="cuda")
    vpg = torch.full((nb, G, vp, 16), 3.0, dtype=dtype, device="cuda")
    rk, rv = kp.cpu().float(), vpg.cpu().float()
    q = ops.attn_prep(ab, H, G, dp, vp, dim, wq, wk, 1e-3, (kp, vpg),
                      bt.cuda(), row_seq.cuda(), ctx.cuda())
    want = torch_ref.attn_prep(ab.cpu().float(), H, G, dp, vp, dim, wq.cpu(),
                               wk.cpu(), 1e-3, (rk, rv), bt, row_seq, ctx)
    _close(q, want, dtype)
    _close(kp, rk, dtype)
    assert torch.equal(vpg.cpu().float(), rv)
    # a layer without its own keys norms the queries only
    q2 = ops.attn_prep(ab[:, : H * dp + 64], H, G, dp, vp, dim, wq, None,
                       1e-3, None, bt.cuda(), row_seq.cuda(), ctx.cuda())
    assert torch.equal(q, q2)


def _delta_inputs(H, G, dp, vp, taps, M, slots, dtype, seed=0):
    C = 2 * G * dp + H * vp
    ab = _rand(M, (C + H * vp + 2 * H + 63) // 64 * 64, seed=seed,
               dtype=dtype)
    conv_w = _rand(taps, C, seed=seed + 1) * 0.6
    decay = torch.stack([_rand(H, seed=seed + 2) * 0.5 - 2,
                         _rand(H, seed=seed + 3) * 0.5 - 1])
    norm = _rand(vp, seed=seed + 4)
    state = _rand(slots, H, vp, dp, seed=seed + 5)
    conv = _rand(slots, taps - 1, C, seed=seed + 6, dtype=dtype)
    return ab, conv_w, decay, norm, state, conv


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("H, G, dp, vp, taps, rows", [
    (2, 1, 64, 64, 4, [1, 1, 1]), (4, 2, 128, 128, 4, [3, 150, 1, 2]),
    (3, 3, 64, 128, 1, [70, 5]), (2, 1, 128, 64, 2, [64, 65, 63]),
    (4, 1, 64, 256, 7, [33, 200]), (2, 2, 256, 64, 3, [40, 129]),
    (2, 1, 256, 256, 4, [66, 2]), (2, 2, 128, 256, 4, [300]),
    (6, 2, 128, 128, 4, [16, 17, 32, 31, 1]), (64, 8, 64, 128, 4, [95]),
    (64, 64, 64, 64, 3, [50, 40]), (32, 32, 128, 128, 4, [33] * 8)])
def test_gated_delta(device, dtype, H, G, dp, vp, taps, rows):
    """Segments of one row to several chunks, from the start or going on,
    with padding rows behind; the sequence's slots and no others change."""
    starts = [(0, 5, 2, 0)[i % 4] for i in range(len(rows))]
    M, S = sum(rows) + 3, len(rows)
    slots = S + 2
    dim, vdim = dp - 7, vp - 3
    ab, cw, decay, norm, state, conv = _delta_inputs(H, G, dp, vp, taps, M,
                                                     slots, dtype)
    C = cw.shape[1]
    cols = torch.arange(C + H * vp)
    pad = torch.where(cols < 2 * G * dp, cols % dp >= dim,
                      (cols - 2 * G * dp) % vp >= vdim).cuda()
    ab[:, : C + H * vp][:, pad] = 0
    conv[..., pad[:C]] = 0
    norm[vdim:] = 0
    for i, s in enumerate(starts):  # no inputs before a sequence's start
        conv[S - i, : max(0, taps - 1 - s)] = 0
    state[:, :, vdim:], state[..., dim:] = 0, 0
    row0 = torch.tensor([0] + rows).cumsum(0)[:-1].int()
    seg = Segments(row0, torch.tensor(rows).int(),
                   torch.arange(S).flip(0).int() + 1, max(rows))
    ctx = torch.cat([torch.arange(s + 1, s + n + 1)
                     for s, n in zip(starts, rows)]
                    + [torch.zeros(3)]).int()
    row_seq = torch.cat([torch.full((n,), i)
                         for i, n in enumerate(rows)]
                        + [torch.zeros(3)]).int()
    # (in bf16 the reference rounds the values behind the convolutions, too)
    rs, rc = state.cpu().clone(), conv.cpu().clone()
    want = torch_ref.gated_delta(
        ab.cpu(), H, G, dp, vp, dim, vdim, cw.cpu(), decay.cpu(),
        norm.cpu(), 1e-6, 1e-5, rs, rc, seg, row_seq, ctx)
    before = state.clone()
    dseg = Segments.build(seg.row0.tolist(), rows, seg.slot.tolist(), "cuda")
    got = ops.gated_delta(ab, H, G, dp, vp, dim, vdim, cw, decay, norm,
                          1e-6, 1e-5, state, conv, dseg, row_seq.cuda(),
                          ctx.cuda())
    n = sum(rows)
    # a value next to a rounding border may go the other way
    _close(got[:n], want[:n], dtype, 2e-2 if dtype == BF16 else 1e-4)
    _close(state, rs, F32, 1e-2 if dtype == BF16 else 1e-4)
    for i, s in enumerate(seg.slot.tolist()):
        live = taps - 1 if starts[i] + rows[i] >= taps - 1 else \
            starts[i] + rows[i]
        if live:
            assert torch.equal(conv[s, -live:].cpu(), rc[s, -live:])
    assert torch.equal(state[0], before[0])
    assert torch.equal(state[S + 1], before[S + 1])


@pytest.mark.parametrize("H, G, dp, vp, rows", [
    (4, 2, 128, 128, [200, 17, 3]), (64, 64, 64, 64, [64, 31]),
    (2, 1, 256, 256, [70]), (32, 8, 128, 128, [33] * 8)])
def test_delta_chunks(device, H, G, dp, vp, rows):
    """The chunked form against the token-by-token form, both in fp32
    behind the same bf16 inputs; strong and weak decays."""
    M, S = sum(rows), len(rows)
    ab, cw, decay, norm, state, conv = _delta_inputs(H, G, dp, vp, 4, M,
                                                     S + 1, BF16)
    decay[0] = torch.linspace(-6, 3, H)
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
        s, c = state.clone(), conv.clone()
        y = ops.gated_delta(ab, H, G, dp, vp, dp, vp, cw, decay, norm, 1e-6,
                            1e-5, s, c, seg, row_seq, ctx)
        got.append((y, s, c))
    _close(got[0][0], got[1][0], BF16, 1e-3)
    _close(got[0][1], got[1][1], F32)
    assert torch.equal(got[0][2], got[1][2])


@pytest.mark.parametrize("E, top, count, keep", [
    (1, 1, 1, 1), (6, 2, 3, 2), (24, 4, 4, 1), (64, 8, 8, 4),
    (100, 5, 10, 9), (256, 8, 8, 3), (300, 6, 3, 2)])
@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
def test_route(device, dtype, E, top, count, keep):
    M, W = 45, 192
    h = _rand(M, W, dtype=dtype)
    router = (_rand(E, W, seed=1) * 0.2).to(dtype)
    ctx = torch.arange(1, M + 1).int()
    ctx[7] = 0
    got, w = ops.route(h, router, ctx.cuda(), top, count, keep)
    s = oracle.softmax(h.double().cpu() @ router.double().cpu().T)
    close = 0
    for m in range(M):
        if m == 7:
            assert (got[m] == -1).all() and not w[m].any()
            continue
        want = oracle.choose(s[m], top, count, keep)
        if got[m].tolist() != want:  # fp32 may swap equal scores
            close += 1
            assert torch.allclose(s[m, got[m].long().cpu()], s[m, want],
                                  rtol=1e-4)
        assert torch.allclose(w[m].double().cpu(), s[m, want], rtol=1e-4)
    assert close < 3


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("M, E, top, W, ff", [
    (1, 6, 2, 64, 64), (9, 6, 3, 192, 128), (40, 8, 2, 256, 192),
    (130, 8, 2, 128, 64), (300, 4, 2, 320, 192), (700, 5, 2, 128, 320),
    (1100, 4, 2, 256, 128), (1300, 4, 2, 512, 384)])
def test_experts(device, dtype, M, E, top, W, ff):
    """Every tile size of the grouped product; uneven experts, one of them
    without a row, padding rows."""
    h = _rand(M, W, dtype=dtype)
    wgup = (_rand(E, 2 * ff, W, seed=1) / W ** 0.5).to(dtype)
    wdown = (_rand(E, W, ff, seed=2) / ff ** 0.5).to(dtype)
    g = torch.Generator().manual_seed(3)
    p = torch.rand(M, E, generator=g) + torch.linspace(0, 0.8, E)
    p[:, 1] = -1
    chosen = p.topk(top, -1).indices.int()
    chosen[M // 2] = -1 if M > 1 else chosen[0]
    y = ops.experts(h, chosen.cuda(), wgup, wdown)
    want = torch_ref.experts(h.cpu().float(), chosen, wgup.cpu().float(),
                             wdown.cpu().float())
    live = (chosen >= 0).reshape(-1)
    _close(y[live.cuda()], want[live], dtype, 3e-2 if dtype == BF16 else None)


def test_trace_run_program(device, tmp_path):
    """bin/trace_run as a program, both dtypes."""
    import numpy as np

    root = Path(__file__).resolve().parents[1]
    c = cases.Case(tmp_path, "cuda:0", F32, seed=9, gain=1.0)
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
