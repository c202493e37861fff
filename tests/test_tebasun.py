"""Tebasun on the CPU: every mechanism and the engine path against the
plain implementation."""

import json
import math

import pytest
import torch

import tebasun_cases as cases
import tebasun_oracle as oracle
from distllm_amd import ops
from distllm_amd.engine.step import PromptBlocks, Segments, StepBatch
from distllm_amd.models import build_model, dims_from_checkpoint, get_dims
from distllm_amd.models.config import CONFIG_READERS, RotaryDims

F32 = torch.float32


@pytest.fixture(scope="module")
def case(tmp_path_factory):
    return cases.Case(tmp_path_factory.mktemp("t"), "cpu", F32)


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


def test_far_key(tmp_path):
    cases.check_far_key(tmp_path, "cpu", F32)


def test_sink(tmp_path):
    cases.check_sink(tmp_path, "cpu", F32)


@pytest.mark.parametrize("kind", ["rglru", "delta"])
def test_state_memory(tmp_path, kind):
    cases.check_state_memory(tmp_path, "cpu", F32, kind)


def test_strong_decay(tmp_path):
    cases.check_strong_decay(tmp_path, "cpu", F32)


def test_loop(tmp_path):
    cases.check_loop(tmp_path, "cpu", F32)


def test_other_sizes(tmp_path):
    cases.check_sizes(tmp_path, "cpu", F32)


def test_greedy_generation(case):
    cases.check_greedy(case)


def test_greedy_generation_loop(case):
    cases.check_greedy(case, use_loop=True)


def test_long_decode(case):
    cases.check_long_decode(case)


def test_bf16_on_cpu(tmp_path):
    """The 16-bit mode, whose boundaries keep the stream in 32 bits."""
    c = cases.Case(tmp_path, "cpu", torch.bfloat16, seed=2)
    cases.check_whole(c, 40)
    cases.check_residuals(c, 20)


# ---- mechanisms alone ------------------------------------------------------

def _rand(*shape, seed=0):
    g = torch.Generator().manual_seed(seed)
    return torch.randn(*shape, generator=g)


def _i32(*v):
    return torch.tensor(v, dtype=torch.int32)


def test_residual_step():
    """Every piece of a boundary, alone and together; padded columns stay
    out of the norm's statistics."""
    W, n, M, eps = 64, 50, 4, 0.1
    y, x0 = _rand(M, W), _rand(M, W, seed=1)
    table, tok = _rand(9, W, seed=2), torch.tensor([3, 8, 3, 0])
    bias, w, vec, aw, ab = (_rand(W, seed=3 + i) for i in range(5))
    for t in (y, x0, table, bias, w, vec, aw, ab):
        t[..., n:] = 0
    alpha = torch.tensor([0.7])
    t = {"n": aw, "n.b": ab, "n.alpha": alpha[0]}
    for use_rms in (False, True):
        for extra in (False, True):
            for fresh in (False, True):
                x = x0.clone()
                h = ops.residual_step(
                    x, y, bias=None if use_rms else bias,
                    rms=(w, n, eps) if use_rms else None,
                    embed=(tok, table, 1.7) if extra else None,
                    vec=vec if extra else None, act=(aw, ab, alpha),
                    fresh=fresh)
                want = torch.zeros(M, n) if fresh else x0[:, :n].clone()
                want += (oracle.rms(y[:, :n], w[:n], eps) if use_rms
                         else (y + bias)[:, :n])
                if extra:
                    want += table[tok][:, :n] * 1.7 + vec[:n]
                assert torch.allclose(x[:, :n], want, atol=1e-5)
                hw = oracle.dyt(x, t, "n")
                assert torch.allclose(h, hw, atol=1e-5)
                assert not x[:, n:].any() and not h[:, n:].any()
    x = x0.clone()
    assert torch.equal(ops.residual_step(x, dtype=F32), x0)


def test_gated_rows():
    x, w, table = _rand(5, 64), _rand(64, 64, seed=1), _rand(7, 40, seed=2)
    tok = torch.tensor([0, 6, 2, 2, 5])
    got = ops.gated_rows(x, w, tok, table, 13, 9)
    want = oracle.gelu_tanh(x @ w.T)[:, :9] * table[tok][:, 13:22]
    assert torch.allclose(got[:, :9], want, atol=1e-5)
    assert not got[:, 9:].any()


@pytest.mark.parametrize("rot", [
    {"base": 10000.0, "dims": 8}, oracle.rotation(),
    oracle.rotation(64, 1e4, 16.0, 4096, 32.0, 1.0),
    oracle.rotation(64, 5e5, 1.0, 8192, 32.0, 1.0),
    oracle.rotation(2, 10.0, 4.0, 8, 1.0, 1.0)])
def test_frequencies(rot):
    freq, mult = RotaryDims(**rot).frequencies()
    want, m = oracle.frequencies(rot)
    assert torch.allclose(torch.tensor(freq, dtype=torch.float64), want,
                          rtol=1e-12)
    assert mult == pytest.approx(m)
    if "scaling" in rot and rot["dims"] == 64 and mult > 1:
        plain, _ = oracle.frequencies({"base": rot["base"], "dims": 64})
        assert want[0] == plain[0] and want[-1] < 0.1 * plain[-1]


@pytest.mark.parametrize("dim, half", [(16, 4), (20, 10), (7, 3), (64, 32)])
def test_rotary_prep(dim, half):
    """Norm, rotation by position, pages of both: keys turned, values as
    projected."""
    H, G, dp, blk = 3, 2, 64, 16
    rot = oracle.rotation(2 * half, 30.0)
    bt = _i32(2, 0, 4, 1)[None]
    ctx = _i32(18, 19, 20, 0, 21)
    seq = torch.zeros(5, dtype=torch.int32)
    ab = _rand(5, (H + G) * dp)
    ab.view(5, -1, dp)[..., dim:] = 0
    wq, wk = _rand(dp, seed=1), _rand(dp, seed=2)
    f, mult = oracle.frequencies(rot)
    table = ops.rotation_table(ctx, f, mult)
    kp, vp = torch.full((5, G, blk, dp), 3.), torch.full((5, G, dp, blk), 3.)
    q = ops.rotary_prep(ab, H, G, dp, dim, wq, wk, 1e-3, table, (kp, vp), bt,
                        seq, ctx)
    heads = ab.view(5, -1, dp)[..., :dim].double()
    pos = ctx - 1
    want = oracle.rotate(oracle.rms(heads[:, :H], wq[:dim], 1e-3), pos, rot)
    live = [0, 1, 2, 4]
    assert torch.allclose(q[live][..., :dim].double(), want[live], atol=1e-5)
    want = oracle.rotate(oracle.rms(heads[:, H:], wk[:dim], 1e-3), pos, rot)
    for r in live:
        p = int(pos[r])
        page = bt[0, p // blk]
        assert torch.allclose(kp[page, :, p % blk, :dim].double(), want[r],
                              atol=1e-5)
        assert torch.equal(vp[page, :, :dim, p % blk],
                           heads[r, H:].float())
    assert (kp == 3).sum() == (5 * blk - 4) * G * dp


def test_sink_attention_far_key():
    """One query and one key that match: the value comes back from any
    place before it, for decoded rows and prompt rows; a large sink takes
    everything, a small one nothing."""
    blk, D = 16, 64
    bt = _i32(2, 0, 4, 1, 5, 3)[None]
    kp = _rand(6, 1, blk, D, seed=7) * 0.01
    vp = torch.zeros(6, 1, D, blk)
    i = torch.arange(96)
    ctx, seq = (i + 1).int(), torch.zeros(96, dtype=torch.int32)
    q = torch.full((96, 2, D), 4.0)
    sink = torch.tensor([-20.0, 4000.0])
    for pos in (0, 15, 16, 36, 95):
        k, v = kp.clone(), vp.clone()
        k[bt[0, pos // blk], :, pos % blk] = 4.0
        v[bt[0, pos // blk], :, :, pos % blk] = 5.0
        out = ops.sink_attn_rows(q, k, v, torch.zeros(96, 2 * D), bt, seq,
                                 ctx, 1.0, sink, 2.0).view(96, 2, D)
        assert torch.equal(out[:, 0].mean(1) > 9.8, i >= pos), pos
        assert out[i < pos].abs().max() < 1e-3 if pos else True
        assert not out[:, 1].any()
        p = PromptBlocks(_i32(0, 3, 3, 93)[None], _i32(0, 0)[None])
        got = ops.sink_attn_prompts(q, k, v, torch.zeros(96, 2 * D), bt, p,
                                    1.0, sink, 2.0)
        assert torch.equal(got[3:], out.view(96, -1)[3:])


def _mixer(entry, T, W=48, seed=3):
    """A model of one layer, inputs of its mixer, and what comes out."""
    cfg = oracle.make_config([entry], width=W)
    t = oracle.make_tensors(cfg, seed)
    model = build_model(CONFIG_READERS["Tebasun"](
        cfg, lambda: {k: tuple(v.shape) for k, v in t.items()}), dtype=F32)
    own = dict(model.named_parameters())
    with torch.no_grad():
        for k, v in model.checkpoint(t).items():
            own[k].copy_(v)
    h = torch.zeros(T, 64)
    h[:, :W] = _rand(T, W, seed=seed)
    d = {k: v.double() for k, v in t.items()}
    want = oracle.MIXERS[entry["type"]](h[:, :W].double(), d, "l0.mix.",
                                        entry["mixer"], 1e-5)
    return model.layers[0].mixer, h, want


@pytest.mark.parametrize("cut", [1, 2, 3, 17, 33])
@pytest.mark.parametrize("entry", [
    oracle.parallel_layer(None),
    oracle.parallel_layer(None, right={"heads": 6, "kv_heads": 2, "dim": 10,
                                       "vdim": 14, "conv": 1}),
    oracle.parallel_layer(None, heads=1, kv_heads=1,
                          right={"heads": 1, "kv_heads": 1, "conv": 5}),
    oracle.rglru_layer(None), oracle.rglru_layer(None, 33, 3, 1),
    oracle.rglru_layer(None, 12, 12, 6)])
def test_mixer_alone(entry, cut):
    """A mixer against the plain one, its state and cache carried over a
    cut; slots of other sequences are left alone."""
    mix, h, want = _mixer(entry, 40)
    cache = mix.make_cache(4, 16, 3, F32, "cpu")
    state = cache if entry["type"] == "rglru" else cache[1]
    state.s.fill_(7.0), state.conv.fill_(7.0)  # what a slot held before
    got = []
    with torch.no_grad():
        for a, b in ((0, cut), (cut, 40)):
            batch = StepBatch.build([(list(range(b - a)), a, [3, 1, 2])], 16,
                                    "cpu", slots=[2])
            hp = torch.zeros(batch.tokens.shape[0], 64)
            hp[: b - a] = h[a:b]
            y = mix(hp, batch, cache)[: b - a, :48]
            bias = getattr(mix, "out_bias", None)
            got.append(y if bias is None else y + bias[:48])
    assert torch.allclose(torch.cat(got).double(), want, atol=3e-5)
    assert (state.s[:2] == 7).all() and (state.conv[:2] == 7).all()


def test_no_special_first_token():
    """The first token's input passes the same factor as any other."""
    entry = oracle.rglru_layer(None, 8, 2, 1)
    mix, h, want = _mixer(entry, 3)
    batch = StepBatch.build([([1], 0, [1])], 16, "cpu", slots=[1])
    hp = torch.zeros(batch.tokens.shape[0], 64)
    hp[:1] = h[:1]
    with torch.no_grad():
        y = mix(hp, batch, mix.make_cache(2, 16, 2, F32, "cpu"))
    assert torch.allclose(y[:1, :48].double(), want[:1], atol=1e-5)


def test_chunk_lists():
    seg = Segments.build([0, 3, 20, 90], [3, 17, 70, 1], [1, 2, 3, 4], "cpu")
    longs, chunks = seg.chunk_lists(64)
    assert longs.tolist() == [[1, 0], [2, 1]]
    assert chunks.tolist() == [[1, 0], [2, 0], [2, 1]]
    assert seg.longs.tolist() == [[1, 0], [2, 1]]
    assert seg.chunks.tolist() == [[1, 0], [2, 0], [2, 1], [2, 2]]
    assert Segments.build([0], [16], [1], "cpu").chunk_lists(64) == \
        (None, None)


# ---- configuration and loading ---------------------------------------------

def test_config_and_registry(case):
    d = dims_from_checkpoint(case.path)
    assert d.arch == "tebasun" and d.num_layers == 5
    assert [x.mixer.type for x in d.layers] == \
        ["rglru", "parallel", "rglru", "parallel", "parallel"]
    right = d.layers[1].mixer.right
    assert (right.decay_rank, right.gate_rank) == (5, 7)
    assert d.layers[4].mixer.left.rot.scaling is None
    assert d.layers[2].mlp is None and d.side_dim == 6
    runs = d.layer_runs()
    assert runs == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (1, 2),
                    (2, None), (3, None), (4, None)]
    # every run has a cache of its own, passes of a loop too
    engine = case.engine()
    layers = engine.cache.layers
    assert len({id(x) for x in layers}) == len(runs)
    assert layers[0].s.shape[0] == 5 == engine.max_batch_size + 1
    m = case.model
    per_token = sum(m.layers[i].mixer.cache_numel() for i, _ in runs)
    assert m.cache_bytes_per_block(16, "bf16") == per_token * 16 * 4
    assert not hasattr(m, "lm_head")
    assert get_dims("tebasun-tiny").arch == "tebasun"
    assert len(get_dims("tebasun-8b").layer_runs()) == 32


@pytest.mark.parametrize("edit, match", [
    (lambda c: c["layers"][1]["mixer"]["left"].update(vdim=9), "vdim"),
    (lambda c: c["layers"][1]["mixer"]["left"].update(kv_heads=3),
     "kv_heads"),
    (lambda c: c["layers"][3]["mixer"]["right"].update(kv_heads=3),
     "kv_heads"),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=7),
     "pairs"),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=18),
     "rotated"),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"]["scaling"].update(
        ramp=1), "ramp"),
    (lambda c: c["layers"][0]["mixer"].update(blocks=3), "blocks"),
    (lambda c: c["layers"][0]["mixer"].update(window=3), "window"),
    (lambda c: c["layers"][0].update(type="scan"), "unknown mixer"),
    (lambda c: c["layers"][0]["mlp"].update(kind="moe"), "kind"),
    (lambda c: c["layers"][0]["mlp"].update(limit=1), "limit"),
    (lambda c: c["loop"].update(stop=6), "loop over"),
    (lambda c: c["loop"].update(start=3), "loop over"),
    (lambda c: c["loop"].update(skip=1), "skip"),
])
def test_config_rejects(case, edit, match):
    cfg = json.loads(json.dumps(case.config))
    edit(cfg)
    with pytest.raises(ValueError, match=match):
        CONFIG_READERS["Tebasun"](cfg, lambda: {
            k: tuple(v.shape) for k, v in case.tensors.items()})


def test_loader_rejects(case, tmp_path):
    from safetensors.torch import save_file

    from distllm_amd.models import load_pretrained

    (tmp_path / "config.json").write_text(json.dumps(case.config))
    for edit, match in (
            (lambda t: t.pop("l1.mix.right.dt_bias"), "lacks"),
            (lambda t: t.update({"l1.mix.left.v": torch.ones(2)}),
             "unknown"),
            (lambda t: t.update({"l0.mix.ra": torch.ones(2, 3, 3)}),
             "shape"),
            (lambda t: t.update({"l0.norm1.alpha": torch.ones(1)}),
             "shape"),
            (lambda t: t.update({"loop.step": torch.ones(2, 48)}), "shape")):
        t = dict(case.tensors)
        edit(t)
        save_file(t, str(tmp_path / "model.safetensors"))
        with pytest.raises(ValueError, match=match):
            load_pretrained(tmp_path, dtype=F32)


def test_random_init_keeps_padding_zero():
    m = build_model("tebasun-tiny", dtype=F32)
    mix = m.layers[0].mixer
    left, right = mix.branches
    q = mix.win[: left.d.heads * left.dp].view(left.d.heads, left.dp, -1)
    assert q[:, : left.d.dim].any() and not q[:, left.d.dim:].any()
    r = right.d.decay_rank
    n = right.d.heads * right.dp
    assert right.w2[:n, :r].any() and not right.w2[:n, r:].any()
    assert not right.w2[n:, :r].any()
    toks = list(range(20))
    batch = StepBatch.build([(toks, 0, [1, 2])], 16, "cpu", slots=[1])
    h = m.forward_step(batch, m.make_cache(3, 16, "bf16", 2))
    assert torch.isfinite(m.logits(h)[:20]).all()


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
        case.passes(case.model.logits(h[row, : len(t)]), t)


def test_beam_search(case):
    from distllm_amd.engine.beam import beam_generate

    prompt = case.tokens(9, 93)
    out = beam_generate(case.model, prompt, num_beams=1, max_tokens=6)
    gaps, scale = cases.oracle_greedy(case, prompt, out)
    assert max(gaps) < 1e-4 * scale


def test_step_limits(case):
    """Growth past the pool or the slots is an error before anything is
    written or taken."""
    e = case.engine(tokens=64, num_blocks=3, max_batch_size=1)
    s = cases._Seq(0, [])
    with pytest.raises(RuntimeError, match="exhausted"):
        cases.feed(e, s, case.tokens(60, 94))
    assert len(e.blockman.free) == 3 and s.cached == 0 and s.slot is None
    cases.feed(e, s, case.tokens(5, 94))
    with pytest.raises(RuntimeError, match="slots"):
        cases.feed(e, cases._Seq(1, []), case.tokens(5, 94))
    e.release(s)
    assert len(e.blockman.free) == 3 and e.slotman.free == [1]


def test_unsupported_options(case):
    with pytest.raises(ValueError, match="dtype"):
        case.model.make_cache(4, 16, "fp8_e4m3")
    with pytest.raises(ValueError, match="tensor_parallel"):
        build_model("tebasun-tiny", tp_group=object())


def test_trace_replay(case, tmp_path):
    import numpy as np

    from distllm_amd.engine.trace import TraceReplay

    rp = TraceReplay(case.engine(), tmp_path)
    t1, t2 = case.tokens(37, 95), case.tokens(5, 96)
    rp.run({"step": 0, "entries": [
        {"id": "x", "tokens": t1[:35], "want": [34, 2]},
        {"id": "y", "tokens": t2, "want": [4]}], "end": ["y"]})
    rp.run({"step": 1, "entries": [
        {"id": "x", "tokens": t1[35:], "want": [1]}], "end": ["x"]})
    V = case.config["vocab"]
    got = torch.from_numpy(np.concatenate([
        np.fromfile(tmp_path / f"{i}.f32", "<f4") for i in range(2)]))
    want = torch.cat([case.want(t1)[[34, 2]], case.want(t2)[4:],
                      case.want(t1)[36:]])
    assert cases.rel(got.view(4, V), want) < cases.TOL[F32]
    assert not rp.live and len(rp.engine.slotman.free) == 4


def test_needed_extensions(case):
    """A replay compiles what the model's steps use and no more."""
    from distllm_amd.build_ext import needed_for

    need = needed_for(str(case.path))
    assert "_hip_lru" in need and "_hip_hybrid" in need
    assert not {"_hip_ops", "_hip_latent", "_hip_chunked",
                "_hip_experts"} & set(need)


def test_cli_generate_from_folder(tmp_path):
    """`distllm generate --llm-name FOLDER` over a jsonl input."""
    from datasets import load_from_disk
    from typer.testing import CliRunner

    from distllm_amd.cli import app

    def edit(t):  # no end-of-text token wins
        t["embed"][:4] = 0

    c = cases.Case(tmp_path, "cpu", F32, cases.mixed_config(vocab=1200),
                   seed=8, edit=edit)
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


def test_decay_scale_is_eight(case):
    assert case.model.layers[0].mixer.d.decay_scale == 8.0
    lam = case.tensors["l0.mix.lam"].double()
    got = case.model.layers[0].mixer.decay[:20].double()
    assert torch.allclose(got, -8 * oracle.softplus(lam)[:20], rtol=1e-6)
    assert math.isclose(float(oracle.softplus(torch.tensor(0.0))),
                        math.log(2), rel_tol=1e-6)
