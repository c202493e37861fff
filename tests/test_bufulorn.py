"""Bufulorn on the CPU: every mechanism and the engine path against the
plain implementation."""

import json

import pytest
import torch

import bufulorn_cases as cases
import bufulorn_oracle as oracle
from distllm_amd import ops
from distllm_amd.engine.step import PromptBlocks, Segments, StepBatch
from distllm_amd.models import build_model, dims_from_checkpoint, get_dims
from distllm_amd.models.config import CONFIG_READERS

F32 = torch.float32


@pytest.fixture(scope="module")
def case(tmp_path_factory):
    return cases.Case(tmp_path_factory.mktemp("b"), "cpu", F32)


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


@pytest.mark.parametrize("size", [1, 2, 16, 33])
def test_chunk_edges(tmp_path, size):
    cases.check_edges(cases.edge_case(tmp_path, "cpu", F32, size), 100)


def test_state_memory(tmp_path):
    cases.check_state_memory(tmp_path, "cpu", F32)


def test_other_sizes(tmp_path):
    cases.check_sizes(tmp_path, "cpu", F32)


def test_greedy_generation(case):
    cases.check_greedy(case)


def test_greedy_generation_loop(case):
    cases.check_greedy(case, use_loop=True)


def test_long_decode(case):
    cases.check_long_decode(case)


# ---- mechanisms alone ------------------------------------------------------

def _rand(*shape, seed=0):
    g = torch.Generator().manual_seed(seed)
    return torch.randn(*shape, generator=g)


def _i32(*v):
    return torch.tensor(v, dtype=torch.int32)


def test_embed_positions():
    table, pos = _rand(9, 64), _rand(5, 64, seed=1)
    h, x = ops.embed_positions(torch.tensor([3, 8, 3, 0]), _i32(1, 2, 5, 0),
                               table, pos)
    assert torch.equal(x[:3], table[[3, 8, 3]] + pos[[0, 1, 4]])
    assert torch.equal(h, x)


@pytest.mark.parametrize("top", [0, 3])
def test_layer_norm_add(top):
    """Padded columns stay out of the statistics; with weights, several
    rows are summed first and rows of weight 0 are not read."""
    W, n, eps, M = 64, 50, 0.1, 4
    v = [_rand(W, seed=i) for i in range(4)]
    for t in v:
        t[n:] = 0
    w, b, wf, bf = v
    x = _rand(M, W, seed=5)
    x[:, n:] = 0
    y = _rand(M * max(top, 1), W, seed=6)
    y[:, n:] = 0
    mix, total = None, y
    if top:
        mix = torch.rand(M, top) + 0.1
        mix[2] = 0
        y[2 * top: 3 * top] = float("nan")
        total = (torch.nan_to_num(y).view(M, top, W) * mix[..., None]).sum(1)
    want = x[:, :n] + oracle.layer_norm(total[:, :n], w[:n], b[:n], eps)
    for final in (None, (wf, bf)):
        xs = x.clone()
        h = ops.layer_norm_add(y, xs, w, b, n, eps, final, mix)
        assert torch.allclose(xs[:, :n], want, atol=1e-5)
        hw = want if final is None else oracle.layer_norm(
            want, wf[:n], bf[:n], eps)
        assert torch.allclose(h[:, :n], hw, atol=1e-5)
        assert not h[:, n:].any() and not xs[:, n:].any()


def test_xielu():
    x, w = _rand(7, 16) * 3, _rand(24, 16, seed=1)
    act = torch.tensor([-0.4, 1.3])
    got = ops.up_xielu(x, w, act)
    assert (x @ w.T < -3).any() and (x @ w.T > 3).any()
    want = oracle.xielu((x @ w.T).double(), *act.double())
    assert torch.allclose(got.double(), want, rtol=1e-5, atol=1e-5)


@pytest.mark.parametrize("E, top, count, keep", [
    (6, 2, 3, 2), (8, 3, 2, 1), (5, 5, 1, 1), (12, 4, 12, 4), (1, 1, 1, 1),
    (10, 4, 5, 3)])
def test_route_and_experts(E, top, count, keep):
    W, ff, M = 64, 64, 40
    h = _rand(M, W)
    t = {"router": _rand(E, W, seed=1) * 0.3}
    for e in range(E):
        for i, (n, s) in enumerate((("gate", (ff, W)), ("up", (ff, W)),
                                    ("down", (W, ff)))):
            t[f"e{e}.{n}"] = _rand(*s, seed=10 + 3 * e + i) * 0.1
    ctx = torch.arange(1, M + 1).int()
    ctx[5] = 0
    ids, w = ops.route(h, t["router"], ctx, top, count, keep)
    s = oracle.softmax(h.double() @ t["router"].double().T)
    for m in range(M):
        if m == 5:
            assert (ids[m] == -1).all() and not w[m].any()
            continue
        want = oracle.choose(s[m], top, count, keep)
        assert ids[m].tolist() == want
        assert torch.allclose(w[m].double(), s[m, want], atol=1e-6)
    # the group rule matters: without it the choice is another one
    free = s.topk(top, -1).indices
    if count > keep and E > 6:
        assert any(set(ids[m].tolist()) != set(free[m].tolist())
                   for m in range(M))

    def gup(e):
        return torch.stack([t[f"e{e}.gate"].view(-1, 16, W),
                            t[f"e{e}.up"].view(-1, 16, W)], 1).view(-1, W)

    y = ops.experts(h, ids, torch.stack([gup(e) for e in range(E)]),
                    torch.stack([t[f"e{e}.down"] for e in range(E)]))
    y = (y.view(M, top, W) * w[..., None]).sum(1)
    y[5] = 0
    r = {"experts": E, "top": top, "groups": {"count": count, "keep": keep}}
    d = {k: v.double() for k, v in t.items()}
    want = oracle.moe(h.double(), d, "", r)
    want[5] = 0
    assert torch.allclose(y.double(), want, atol=1e-5)


def test_far_key_stands_out():
    """One query and one key that match: the value comes back from any
    place of the chunk and not at all from outside, for decoded rows and
    prompt rows."""
    blk, D, size = 16, 64, 37
    bt = _i32(2, 0, 4, 1, 5, 3)[None]
    kp = _rand(6, 1, blk, D, seed=7) * 0.01
    vp = torch.zeros(6, 1, D, blk)
    ab = torch.full((96, D), 30.0)  # gates wide open
    dist = torch.tensor([[0.5], [0.2]])
    for pos in (0, 15, 16, 36, 37, 73, 74):
        k, v = kp.clone(), vp.clone()
        k[bt[0, pos // blk], :, pos % blk] = 4.0
        v[bt[0, pos // blk], :, :, pos % blk] = 5.0
        q = torch.full((96, 1, D), 4.0)
        ctx = torch.arange(1, 97).int()
        seq = torch.zeros(96, dtype=torch.int32)
        out = ops.paged_attn_rows(q, k, v, ab, 0, torch.zeros(96, 1, D), bt,
                                  seq, ctx, size, 1.0, 30.0, dist)
        i = torch.arange(96)
        seen = (i >= pos) & (i // size == pos // size)
        assert torch.equal(out.mean((1, 2)) > 4.9, seen), pos
        assert out[~seen].abs().max() < 1e-3
        p = PromptBlocks(_i32(0, 3, 3, 93)[None], _i32(0, 0)[None])
        got = ops.paged_attn_prompts(q, k, v, ab, 0, torch.zeros(96, 1, D),
                                     bt, p, size, 1.0, 30.0, dist)
        assert torch.equal(got[3:], out[3:])


def _delta_args(m, T, W=48, seed=3):
    cfg = oracle.make_config([{"type": "delta", "mixer": m, "mlp": None}],
                             width=W)
    t = oracle.make_tensors(cfg, seed)
    model = build_model(CONFIG_READERS["Bufulorn"](cfg), dtype=F32)
    own = dict(model.named_parameters())
    with torch.no_grad():
        for k, v in model.checkpoint(t).items():
            own[k].copy_(v)
    h = torch.zeros(T, 64)
    h[:, :W] = _rand(T, W, seed=seed)
    want = oracle.delta(h[:, :W].double(),
                        {k: v.double() for k, v in t.items()}, "l0.mix.", m,
                        1e-5)
    return model, h, want


@pytest.mark.parametrize("taps", [1, 2, 5])
@pytest.mark.parametrize("cut", [1, 2, 3, 17])
def test_delta_alone(taps, cut):
    """A delta layer against the plain one, its state carried over a cut;
    slots of other sequences are left alone."""
    m = {"heads": 6, "kv_heads": 2, "dim": 10, "vdim": 14, "conv": taps}
    model, h, want = _delta_args(m, 20)
    mix = model.layers[0].mixer
    state = mix.make_cache(1, 16, 3, F32, "cpu")
    state.s.fill_(7.0), state.conv.fill_(7.0)  # what a slot held before
    got = []
    with torch.no_grad():
        for a, b in ((0, cut), (cut, 20)):
            batch = StepBatch.build([(list(range(b - a)), a, [0, 1])], 16,
                                    "cpu", slots=[2])
            hp = torch.zeros(batch.tokens.shape[0], 64)
            hp[: b - a] = h[a:b]
            got.append(mix(hp, batch, state)[: b - a, :48])
    assert torch.allclose(torch.cat(got).double(), want, atol=2e-5)
    assert (state.s[:2] == 7).all() and (state.conv[:2] == 7).all()


def test_unit_eps_and_decay():
    """Tiny convolution outputs meet the unit norm's constant, and a slow
    decay is kept apart from none at all."""
    k = torch.full((1, 1, 4), 3e-4, dtype=torch.float64)
    assert abs(float(oracle.unit(k)[0, 0, 0]) - 3e-4 / 1.36e-6 ** .5) < 1e-3
    m = {"heads": 1, "kv_heads": 1, "dim": 4, "vdim": 4, "conv": 1}
    model, h, want = _delta_args(m, 16)
    mix = model.layers[0].mixer
    ab = ops.linear(h, mix.win).detach()
    seg = Segments(_i32(0), _i32(16), _i32(1), 16)

    def run(scale, a_log):
        x = ab.clone()
        x[:, : 2 * mix.dp] *= scale
        d = mix.decay.detach().clone()
        d[0] = a_log
        s = torch.zeros(2, 1, 64, 64)
        y = ops.gated_delta(x, 1, 1, 64, 64, 4, 4, mix.conv.detach(), d,
                            mix.o_norm.detach(), 1e-6, 1e-5, s,
                            torch.zeros(2, 0, mix.channels), seg,
                            torch.zeros(16, dtype=torch.int32),
                            torch.arange(1, 17).int())
        return y, s

    assert (run(1e-3, -2.)[1] - run(1., -2.)[1]).abs().max() > 1e-2
    assert (run(1., -5.)[0] - run(1., -20.)[0]).abs().max() > 1e-4


# ---- configuration and loading ---------------------------------------------

def test_config_and_registry(case):
    d = dims_from_checkpoint(case.path)
    assert d.arch == "bufulorn" and d.num_layers == 6
    assert d.max_position_embeddings == 512
    kinds = [x.mixer.type for x in d.layers]
    assert kinds == ["attention", "delta", "attention", "attention",
                     "delta", "attention"]
    assert [getattr(x.mixer, "chunk", None) for x in d.layers] == \
        [20, None, 33, 7, None, 64]
    assert d.layers[2].mlp is None
    assert d.layers[3].mlp.experts == 8 and d.layers[3].mlp.keep == 1
    # layers that share keys and values share their pages
    engine = case.engine()
    cache = engine.cache
    assert cache.layers[3] is cache.layers[0]
    assert cache.layers[5] is cache.layers[2]
    assert cache.layers[1].s.shape[0] == 5 == engine.max_batch_size + 1
    assert get_dims("bufulorn-tiny").arch == "bufulorn"
    assert get_dims("bufulorn-8b").num_layers == 32


@pytest.mark.parametrize("edit, match", [
    (lambda c: c["layers"][3]["mixer"].update(kv_from=3), "earlier layer"),
    (lambda c: c["layers"][3]["mixer"].update(kv_from=1), "of its own"),
    (lambda c: c["layers"][5]["mixer"].update(kv_from=3), "of its own"),
    (lambda c: c["layers"][3]["mixer"].update(vdim=31), "vdim"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=3), "kv_heads"),
    (lambda c: c["layers"][0].update(type="scan"), "unknown mixer"),
    (lambda c: c["layers"][0]["mixer"].update(rope=1), "rope"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(sinks=1), "mask"),
    (lambda c: c["layers"][1]["mixer"].update(mask={"size": 3}), "mask"),
    (lambda c: c["layers"][0]["mlp"].update(kind="glu"), "kind"),
    (lambda c: c["layers"][0]["mlp"].update(limit=1), "limit"),
    (lambda c: c["layers"][1]["mlp"].update(shared=1), "shared"),
    (lambda c: c["layers"][1]["mlp"]["router"].update(bias=1), "bias"),
    (lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(count=4),
     "equal groups"),
    (lambda c: c["layers"][1]["mlp"]["router"].update(top=5), "top"),
])
def test_config_rejects(edit, match):
    cfg = oracle.make_config(cases.mixed_layers())
    edit(cfg)
    with pytest.raises(ValueError, match=match):
        CONFIG_READERS["Bufulorn"](cfg)


def test_loader_rejects(case, tmp_path):
    from safetensors.torch import save_file

    from distllm_amd.models import load_pretrained

    (tmp_path / "config.json").write_text(json.dumps(case.config))
    for edit, match in (
            (lambda t: t.pop("l1.mix.dt_bias"), "lacks"),
            (lambda t: t.update({"l3.mix.k": torch.ones(2)}), "unknown"),
            (lambda t: t.update({"l0.mix.o": torch.ones(3, 3)}), "shape"),
            (lambda t: t.update(pos=torch.ones(3, 48)), "shape")):
        t = dict(case.tensors)
        edit(t)
        save_file(t, str(tmp_path / "model.safetensors"))
        with pytest.raises(ValueError, match=match):
            load_pretrained(tmp_path, dtype=F32)


def test_random_init_keeps_padding_zero():
    m = build_model("bufulorn-tiny", dtype=F32)
    mix = m.layers[0].mixer
    q = mix.wqkvg[: mix.d.heads * mix.dp].view(mix.d.heads, mix.dp, -1)
    assert q[:, : mix.d.dim].any() and not q[:, mix.d.dim:].any()
    assert m.layers[1].mixer.d.kv_from == 0
    assert not mix.bias.any()


def test_padded_forward_matches_engine(case):
    """The batch forward that beam search and the embedders use."""
    t1, t2 = case.tokens(40, 91), case.tokens(13, 92)
    ids = torch.zeros(2, 40, dtype=torch.long)
    mask = torch.zeros(2, 40, dtype=torch.int32)
    ids[0], mask[0] = torch.tensor(t1), 1
    ids[1, :13], mask[1, :13] = torch.tensor(t2), 1
    h = case.model(ids, mask)
    assert h.shape == (2, 40, case.config["width"])
    assert not h[1, 13:].any()
    for row, t in ((0, t1), (1, t2)):
        got = case.model.logits(h[row, : len(t)])
        assert cases.rel(got, case.want(t)) < cases.TOL[F32]


def test_beam_search(case):
    from distllm_amd.engine.beam import beam_generate

    prompt = case.tokens(9, 93)
    out = beam_generate(case.model, prompt, num_beams=1, max_tokens=6)
    gaps, scale = cases.oracle_greedy(case, prompt, out)
    assert max(gaps) < 1e-4 * scale


def test_step_limits(case):
    """Growth past the position table, the pool or the slots is an error
    before anything is written or taken."""
    from distllm_amd.engine.engine import _Seq

    assert case.engine(tokens=4096).max_model_len == 512
    e = case.engine(tokens=64, num_blocks=3, max_batch_size=1)
    s = _Seq(0, [])
    with pytest.raises(RuntimeError, match="max_model_len"):
        cases.feed(e, s, case.tokens(65, 94))
    with pytest.raises(RuntimeError, match="exhausted"):
        cases.feed(e, s, case.tokens(60, 94))
    assert len(e.blockman.free) == 3 and s.cached == 0 and s.slot is None
    cases.feed(e, s, case.tokens(5, 94))
    assert s.slot == 1
    with pytest.raises(RuntimeError, match="slots"):
        cases.feed(e, _Seq(1, []), case.tokens(5, 94))
    assert len(e.blockman.free) == 2
    e.release(s)
    assert len(e.blockman.free) == 3 and e.slotman.free == [1]


def test_unsupported_options(case):
    with pytest.raises(ValueError, match="dtype"):
        case.model.make_cache(4, 16, "fp8_e4m3")
    with pytest.raises(ValueError, match="tensor_parallel"):
        build_model("bufulorn-tiny", tp_group=object())


def test_trace_replay(case, tmp_path):
    import numpy as np

    from distllm_amd.engine.trace import TraceReplay

    rp = TraceReplay(case.engine(), tmp_path)
    t1, t2 = case.tokens(37, 95), case.tokens(5, 96)
    rp.run({"step": 0, "entries": [
        {"id": "x", "tokens": t1[:35], "want": [34, 2]},
        {"id": "y", "tokens": t2, "want": [4]}], "end": ["y"]})
    rp.run({"step": 1, "entries": [
        {"id": "x", "tokens": t1[35:36], "want": []}], "end": []})
    rp.run({"step": 2, "entries": [
        {"id": "x", "tokens": t1[36:], "want": [0]}], "end": ["x"]})
    V = case.config["vocab"]
    got = np.fromfile(tmp_path / "0.f32", "<f4").reshape(3, V)
    want = torch.stack([case.want(t1)[34], case.want(t1)[2],
                        case.want(t2)[4]])
    assert cases.rel(torch.from_numpy(got), want) < cases.TOL[F32]
    assert not (tmp_path / "1.f32").exists()
    got = np.fromfile(tmp_path / "2.f32", "<f4").reshape(1, V)
    assert cases.rel(torch.from_numpy(got), case.want(t1)[36:]) \
        < cases.TOL[F32]
    assert not rp.live and len(rp.engine.slotman.free) == 4


def test_needed_extensions(case, tmp_path):
    """A replay compiles what the model's steps use and no more."""
    from distllm_amd.build_ext import NEEDED, needed_for
    from distllm_amd.ops.native import EXTENSIONS

    assert "_hip_hybrid" in needed_for(str(case.path))
    assert "_hip_ops" not in needed_for(str(case.path))
    assert needed_for(str(tmp_path / "nothing")) == ()
    assert set(NEEDED) == set(CONFIG_READERS)
    assert all(set(v) <= set(EXTENSIONS) for v in NEEDED.values())


def test_native_generator_from_folder(tmp_path):
    """generate's entry point picks the model class by config.json."""
    from distllm_amd.generate import get_generator

    cfg = oracle.make_config(cases.mixed_layers(), vocab=1200)
    c = cases.Case(tmp_path, "cpu", F32, cfg, seed=8)
    gen = get_generator({"name": "native", "model": str(c.path),
                         "temperature": 0.0, "min_p": 0.0, "max_tokens": 5,
                         "max_model_len": 128, "max_batch_size": 2})
    assert type(gen.model).__name__ == "BufulornModel"
    out = gen.generate(["hello there world", "a second, longer prompt"])
    assert len(out) == 2
    ids = gen._tokenize(["hello there world"])[0]
    toks = gen.engine.generate([ids], gen.params)[0]
    gaps, scale = cases.oracle_greedy(c, ids, toks)
    assert max(gaps) < 1e-4 * scale


def test_cli_generate_from_folder(tmp_path):
    """`distllm generate --llm-name FOLDER` over a jsonl input."""
    from datasets import load_from_disk
    from typer.testing import CliRunner

    from distllm_amd.cli import app

    cfg = oracle.make_config(cases.mixed_layers(), vocab=1200)
    c = cases.Case(tmp_path, "cpu", F32, cfg, seed=8)
    data = tmp_path / "in"
    data.mkdir()
    with open(data / "a.jsonl", "w") as fh:
        for i in range(3):
            fh.write(json.dumps({"text": f"document {i} " * (i + 1),
                                 "path": f"d{i}"}) + "\n")
    out = tmp_path / "out"
    r = CliRunner().invoke(app, [
        "generate", "--input-dir", str(data), "--output-dir", str(out),
        "--llm-name", str(c.path), "--generator-name", "native",
        "--reader-name", "jsonl", "--prompt-name", "identity",
        "--max-tokens", "4", "--temperature", "0.0", "--batch-size", "2"])
    assert r.exit_code == 0, r.output
    shard = next(p for p in out.iterdir() if p.is_dir())
    assert len(load_from_disk(str(shard))) == 3
