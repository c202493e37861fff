"""Kanotar on the GPU: the HIP kernels against fp32 references of the same
op, and the engine path in bf16 and fp32 against the plain
implementation."""

import os
import subprocess
import sys
from pathlib import Path

import pytest
import torch

import kanotar_cases as cases
import kanotar_oracle as oracle
from distllm_amd import ops
from distllm_amd.ops import torch_ref

pytestmark = pytest.mark.gpu

F32, BF16 = torch.float32, torch.bfloat16
DTYPES = [BF16, F32]
ids = {BF16: "bf16", F32: "fp32"}.get


@pytest.fixture(scope="module", params=DTYPES, ids=ids)
def case(request, device, tmp_path_factory):
    return cases.Case(tmp_path_factory.mktemp("k"), "cuda:0", request.param,
                      gain=2.0 if request.param == F32 else 1.0)


def test_whole_prompt(case):
    cases.check_whole(case)


def test_residual_stream(case):
    cases.check_residuals(case)


def test_portions(case):
    cases.check_portions(case)


def test_mixed_batches(case):
    cases.check_batches(case)


def test_page_reuse(case):
    cases.check_reuse(case)


def test_wanted_places(case):
    cases.check_wanted(case)


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("size", [1, 2, 16, 33, 130])
def test_window_edges(device, tmp_path, dtype, size):
    c = cases.edge_case(tmp_path, "cuda:0", dtype, size)
    if dtype == BF16 and size > 33:
        # one key of many: the kernels' own tests make it stand out
        toks = c.tokens(300, 1)
        got = cases.run_cut(c.engine(), toks, [200, 3, 40, 1])
        assert cases.rel(got, c.want(toks)) < cases.TOL[BF16]
    else:
        cases.check_edges(c, 100 if size < 100 else 180)


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


def test_capture_without_garbage_collection(case, monkeypatch):
    """Nothing may be collected while a decode graph is captured, and a
    dead engine's graphs go with it instead of waiting for a collection."""
    import gc
    import weakref

    states = []
    inner = type(case.model).decode_step

    def spy(self, *a):
        if torch.cuda.is_current_stream_capturing():
            states.append(gc.isenabled())
        return inner(self, *a)

    monkeypatch.setattr(type(case.model), "decode_step", spy)
    engine = case.engine()
    engine.warm_graphs([1, 2])
    assert states == [False, False] and gc.isenabled()
    refs = [weakref.ref(g) for g in engine._graphs.values()]
    gc.disable()
    try:
        del engine
        assert all(r() is None for r in refs)
    finally:
        gc.enable()


# ---- kernels ---------------------------------------------------------------

def _rand(*shape, seed=0, dtype=F32):
    g = torch.Generator().manual_seed(seed)
    return torch.randn(*shape, generator=g).to(dtype).to("cuda")


def _close(got, want, dtype):
    got, want = got.float().cpu(), want.float().cpu()
    scale = want.pow(2).mean().sqrt().clamp_min(1e-6)
    d = (got - want).abs()
    if dtype == BF16:  # the output's own rounding comes on top
        d = d - want.abs() / 128
    err = (d.max() / scale).item()
    assert err < (2e-2 if dtype == BF16 else 2e-5), err


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("M, W, n", [(1, 64, 1), (7, 320, 300),
                                     (5, 1024, 1024), (3, 1088, 1030),
                                     (9, 4096, 4096), (2, 8192, 8000),
                                     (2, 12288, 12288)])
def test_sandwich_norm(device, dtype, M, W, n):
    table, y = _rand(11, W, dtype=dtype), _rand(M, W, seed=1, dtype=dtype)
    wn, wp = _rand(W, seed=2), _rand(W, seed=3)
    for t in (table, y, wn, wp):
        t[..., n:] = 0
    tok = torch.arange(M, device="cuda") % 11
    h, x = ops.embed_norm(tok, table, wn, n, 0.01)
    h_ref, x_ref = torch_ref.embed_norm(tok, table.float(), wn, n, 0.01)
    assert torch.equal(x, x_ref)
    _close(h, h_ref, dtype)
    h = ops.post_norm_add(y, x, wp, wn, n, 0.01)
    h_ref = torch_ref.post_norm_add(y.float(), x_ref, wp, wn, n, 0.01)
    _close(x, x_ref, F32)
    _close(h, h_ref, dtype)


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("M, ff", [(1, 64), (37, 448), (300, 1024)])
def test_clamped_glu(device, dtype, M, ff):
    x = _rand(M, 256, dtype=dtype)
    w = (_rand(2 * ff, 256, seed=1) * 0.15).to(dtype)
    got = ops.gateup_clamped_glu(x, w, 1.1, 1.702, 1.0)
    gu = (x.double() @ w.double().t()).float()
    assert (gu.abs() > 1.1).any()
    _close(got, torch_ref.clamped_glu(gu, 1.1, 1.702, 1.0), dtype)


@pytest.mark.parametrize("M", [1, 16, 17, 40, 100, 200])
@pytest.mark.parametrize("N, K", [(64, 64), (512, 128), (128, 512),
                                  (192, 256)])
def test_head_gemm(device, M, N, K):
    x, w = _rand(M, 5, K, dtype=BF16), _rand(5, N, K, seed=1, dtype=BF16)
    _close(ops.head_gemm(x, w), torch_ref.head_gemm(x.cpu().float(),
                                                    w.cpu().float()), BF16)


def _paged(R, lens, dtype, blk=16, seed=0):
    """Cache with the pages of sequences interleaved, and its table."""
    pages = [(n + blk - 1) // blk for n in lens]
    g = torch.Generator().manual_seed(seed)
    order = torch.randperm(sum(pages) + 2, generator=g).int()
    bt = torch.zeros(len(lens), max(pages) + 1, dtype=torch.int32)
    at = 0
    for i, p in enumerate(pages):
        bt[i, :p] = order[at: at + p]
        at += p
    return _rand(sum(pages) + 2, blk, R, seed=seed + 1, dtype=dtype), bt


RANKS = [64, 128, 192, 256, 320, 384, 512, 576]


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("R", RANKS)
@pytest.mark.parametrize("H", [1, 16, 20, 40, 70])
def test_latent_attn(device, dtype, R, H):
    lens = [1, 15, 16, 33, 200, 517]
    cache, bt = _paged(R, lens, dtype)
    row_seq = torch.tensor([5, 0, 1, 2, 3, 4, 5, 4, 0], dtype=torch.int32)
    ctx = torch.tensor([517, 1, 15, 16, 33, 200, 300, 97, 0],
                       dtype=torch.int32)
    q = _rand(9, H, R, seed=2, dtype=dtype)
    scale = 2.0 / R ** 0.5
    for window in (1, 31, 32, 200, 10 ** 12):
        want = torch_ref.latent_attn(
            q.cpu().float(), cache.cpu().float(), bt, row_seq, ctx, window,
            scale)
        for nsplit in (0, 1, 3):
            got = ops.latent_attn(q, cache, bt.cuda(), row_seq.cuda(),
                                  ctx.cuda(), window, scale, nsplit)
            _close(got, want, dtype)
            assert not got[8].any()  # a padding row sees nothing


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("R, H", [(64, 3), (512, 40)])
def test_latent_attn_far_key(device, dtype, R, H):
    """A key that matches the query comes back whole just inside the
    window and not at all just outside, at page and tile borders."""
    W = 150
    cache, bt = _paged(R, [400], dtype)
    cache *= 0.05
    for pos in (0, 15, 16, 31, 32, 100, 127, 128):
        c = cache.clone()
        c[bt[0, pos // 16].item(), pos % 16] = 4.0
        ctx = torch.tensor([pos + 1, pos + W, pos + W + 1, 399],
                           dtype=torch.int32, device="cuda")
        out = ops.latent_attn(
            torch.full((4, H, R), 4.0, dtype=dtype, device="cuda"), c,
            bt.cuda(), torch.zeros(4, dtype=torch.int32, device="cuda"),
            ctx, W, 1.0).float()
        assert (out[:2] > 3.9).all() and (out[2:].abs() < 1).all(), pos


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
def test_latent_prep_and_gather(device, dtype):
    QP, qn, R, rn = 128, 100, 192, 130
    _, bt = _paged(R, [40, 7], dtype)
    cache = torch.zeros(8, 16, R, dtype=dtype, device="cuda")
    ab = _rand(5, QP + R, dtype=dtype)
    ab[:, qn:QP] = 0
    ab[:, QP + rn:] = 0
    wq, wc = _rand(QP, seed=1), _rand(R, seed=2)
    row_seq = torch.tensor([0, 0, 1, 0, 1], dtype=torch.int32)
    ctx = torch.tensor([40, 17, 7, 0, 1], dtype=torch.int32)
    cq = ops.latent_prep(ab, QP, qn, rn, wq, wc, 1e-3, cache, bt.cuda(),
                         row_seq.cuda(), ctx.cuda())
    ref = torch.zeros(8, 16, R)
    want = torch_ref.latent_prep(ab.cpu().float(), QP, qn, rn, wq.cpu(),
                                 wc.cpu(), 1e-3, ref, bt, row_seq, ctx)
    _close(cq, want, dtype)
    _close(cache, ref, dtype)
    got = ops.latent_gather(
        cache, bt.cuda(), torch.tensor([1, 0], dtype=torch.int32).cuda(),
        torch.tensor([6, 39], dtype=torch.int32).cuda())
    assert torch.equal(got[1].cpu(), cache[bt[0, 2].item(), 7].cpu())
    assert torch.equal(got[0].cpu(), cache[bt[1, 0].item(), 6].cpu())
    # a layer without its own latent norms the query latent only
    cq2 = ops.latent_prep(ab[:, :QP].contiguous(), QP, qn, rn, wq, None,
                          1e-3, None, bt.cuda(), row_seq.cuda(), ctx.cuda())
    assert torch.equal(cq, cq2)


@pytest.mark.parametrize("dk, dv", [(64, 64), (64, 128), (128, 64),
                                    (128, 128), (256, 64), (128, 256),
                                    (256, 256)])
def test_attn_window(device, dk, dv):
    """Prompt continuations: queries are the last of their keys."""
    H = 3
    nq, nk = [130, 33, 1, 300], [130, 170, 65, 411]
    cu_q = torch.tensor([0] + nq).cumsum(0).int()
    cu_k = torch.tensor([0] + nk).cumsum(0).int()
    q = _rand(sum(nq), H, dk, dtype=BF16)
    kv = _rand(sum(nk), H * (dk + dv), seed=1, dtype=BF16)
    bm = tuple(t.cuda() for t in ops.varlen_block_map(cu_q))
    scale = 2.0 / dk ** 0.5
    for window in (1, 2, 64, 97, 128, 10 ** 12):
        out = torch.full((sum(nq), H, dv), 7.0, dtype=BF16, device="cuda")
        ops.attn_window(q, kv, out, cu_q.cuda(), cu_k.cuda(), bm, window,
                        scale)
        want = torch_ref.attn_window(q.cpu().float(), kv.cpu().float(), dv,
                                     cu_q, cu_k, window, scale)
        _close(out, want, BF16)


def test_attn_window_far_key(device):
    """One matching key, at every place around the window's edge."""
    H, d, W, Tk, Tq = 2, 64, 130, 400, 333
    cu_q = torch.tensor([0, Tq], dtype=torch.int32)
    cu_k = torch.tensor([0, Tk], dtype=torch.int32)
    bm = tuple(t.cuda() for t in ops.varlen_block_map(cu_q))
    base = _rand(Tk, 2 * H * d, dtype=BF16) * 0.05
    for pos in (0, 63, 64, 127, 200, 255, 269):
        kv = base.clone()
        kv[pos] = 4.0
        out = torch.empty(Tq, H, d, dtype=BF16, device="cuda")
        ops.attn_window(
            torch.full((Tq, H, d), 4.0, dtype=BF16, device="cuda"), kv, out,
            cu_q.cuda(), cu_k.cuda(), bm, W, 1.0)
        i = torch.arange(Tq) + Tk - Tq
        seen = (i >= pos) & (i - pos < W)
        got = out.float().mean((1, 2)).cpu() > 3.9
        assert torch.equal(got, seen), pos


def test_trace_run_program(device, tmp_path):
    """bin/trace_run as a program, both dtypes."""
    import json

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
