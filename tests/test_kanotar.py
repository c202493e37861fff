"""Kanotar on the CPU: every mechanism and the engine path against the
plain implementation."""

import json

import pytest
import torch

import kanotar_cases as cases
import kanotar_oracle as oracle
from distllm_amd import ops
from distllm_amd.models import build_model, dims_from_checkpoint, get_dims
from distllm_amd.models.config import CONFIG_READERS

F32 = torch.float32


@pytest.fixture(scope="module")
def case(tmp_path_factory):
    return cases.Case(tmp_path_factory.mktemp("k"), "cpu", F32)


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


@pytest.mark.parametrize("size", [1, 2, 16, 33])
def test_window_edges(tmp_path, size):
    cases.check_edges(cases.edge_case(tmp_path, "cpu", F32, size), 100)


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


def test_embed_and_sandwich_norm():
    W, n, eps = 64, 50, 0.1
    table, w, wp = _rand(9, W), _rand(W, seed=1), _rand(W, seed=2)
    for t in (table, w, wp):
        t[..., n:] = 0
    tok = torch.tensor([3, 8, 3])
    h, x = ops.embed_norm(tok, table, w, n, eps)
    assert torch.equal(x, table[tok])
    assert torch.allclose(h[:, :n], oracle.rms(x[:, :n], w[:n], eps),
                          atol=1e-6)
    y = _rand(3, W, seed=3)
    y[:, n:] = 0
    want_x = x[:, :n] + oracle.rms(y[:, :n], wp[:n], eps)
    h = ops.post_norm_add(y, x, wp, w, n, eps)
    assert torch.allclose(x[:, :n], want_x, atol=1e-6)
    assert torch.allclose(h[:, :n], oracle.rms(want_x, w[:n], eps),
                          atol=1e-6)
    assert not h[:, n:].any() and not x[:, n:].any()


@pytest.mark.parametrize("limit", [0.3, 1.0, 7.0])
def test_clamped_glu(limit):
    """Both clamps at work: the gate only from above, the up-projection
    on both sides."""
    x = _rand(5, 16) * 4
    t = {"gate": _rand(24, 16, seed=1), "up": _rand(24, 16, seed=2),
         "down": torch.eye(24)}
    assert (x @ t["gate"].T).min() < -2 * limit or limit > 1
    got = ops.gateup_clamped_glu(x, torch.cat([t["gate"], t["up"]]), limit,
                                 1.702, 1.0)
    assert torch.allclose(got, oracle.clamped_glu(x, t, "", limit),
                          atol=1e-5)


def test_latent_attention_forms():
    """Folded and expanded attention against the plain one, for one
    layer with an own latent."""
    m = oracle.make_layer(heads=3, dim=10, vdim=14, q_rank=12, kv_rank=20,
                          size=6)["mixer"]
    cfg = oracle.make_config([{"type": "latent_attention", "mixer": m,
                               "mlp": None}])
    t = {k: v.double() for k, v in oracle.make_tensors(cfg, 5).items()}
    h = _rand(40, cfg["width"], seed=6).double()
    c = oracle.latent(h, t, "l0.mix.", 1e-5)
    want = oracle.latent_attention(h, c, t, "l0.mix.", m, 1e-5)
    from distllm_amd.engine.step import StepBatch
    from distllm_amd.models.layered import LayeredCache

    model = build_model(CONFIG_READERS["Kanotar"](cfg), dtype=F32)
    own = dict(model.named_parameters())
    with torch.no_grad():
        for k, v in model.checkpoint(
                {k: v.float() for k, v in t.items()}).items():
            own[k].copy_(v)
        hp = torch.zeros(64, 64)
        hp[:40, :48] = h
        for expand_min in (1000, 2):
            cache = LayeredCache(model, 4, 16)
            b = StepBatch.build([(list(range(40)), 0, [3, 1, 2])], 16,
                                "cpu", expand_min)
            assert bool(b.portions) == (expand_min == 2)
            y = model.layers[0].mixer(hp, b, cache.layers[0])
            assert torch.allclose(y[:40, :48].double(), want, atol=1e-5)


def test_far_key_stands_out():
    """One query and one key that match: the key's latent comes back just
    inside the window and not at all just outside."""
    blk, R, W = 16, 64, 37
    bt = torch.tensor([[2, 0, 4, 1]], dtype=torch.int32)
    cache = _rand(5, blk, R, seed=7) * 0.1
    pos = 13
    cache[bt[0, pos // blk], pos % blk] = 5.0
    for ctx in range(pos + 1, 64):
        out = ops.latent_attn(
            torch.full((1, 1, R), 5.0), cache, bt,
            torch.zeros(1, dtype=torch.int32),
            torch.tensor([ctx], dtype=torch.int32), W, 1.0)
        seen = ctx - 1 - pos < W
        assert (out.mean() > 4.9) == seen, ctx
        if not seen:
            assert out.abs().mean() < 0.5


# ---- configuration and loading ---------------------------------------------

def test_config_and_registry(case):
    d = dims_from_checkpoint(case.path)
    assert d.arch == "kanotar" and d.num_layers == 4
    assert [x.mixer.window for x in d.layers] == [8, 21, 64, 5]
    assert [x.mixer.kv_from for x in d.layers] == [None, None, 0, 1]
    assert d.layers[1].mlp is None and d.layers[2].mlp.limit == 0.6
    assert d.norm_eps == 1e-5 and d.logit_scale == 0.7
    # layers that share a latent share its pages
    cache = case.engine().cache
    assert cache.layers[2] is cache.layers[0]
    assert cache.layers[3] is cache.layers[1]
    assert get_dims("kanotar-tiny").arch == "kanotar"


@pytest.mark.parametrize("edit, match", [
    (lambda c: c["layers"][2]["mixer"].update(kv_from=3), "earlier layer"),
    (lambda c: c["layers"][3]["mixer"].update(kv_from=2), "own"),
    (lambda c: c["layers"][2]["mixer"].update(kv_rank=31), "kv_rank"),
    (lambda c: c["layers"][0].update(type="scan"), "unknown mixer"),
    (lambda c: c["layers"][0]["mixer"].update(rope=1), "rope"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(sinks=1), "mask"),
    (lambda c: c["layers"][0]["mlp"].update(kind="moe"), "kind"),
])
def test_config_rejects(edit, match):
    cfg = oracle.make_config(cases.mixed_layers())
    edit(cfg)
    with pytest.raises(ValueError, match=match):
        CONFIG_READERS["Kanotar"](cfg)


def test_loader_rejects(case, tmp_path):
    from safetensors.torch import save_file

    from distllm_amd.models import load_pretrained

    (tmp_path / "config.json").write_text(json.dumps(case.config))
    for edit, match in (
            (lambda t: t.pop("l1.mix.uk"), "lacks"),
            (lambda t: t.update(extra=torch.ones(2)), "unknown"),
            (lambda t: t.update({"l0.mix.o": torch.ones(3, 3)}), "shape")):
        t = dict(case.tensors)
        edit(t)
        save_file(t, str(tmp_path / "model.safetensors"))
        with pytest.raises(ValueError, match=match):
            load_pretrained(tmp_path, dtype=F32)


def test_random_init_keeps_padding_zero():
    m = build_model("kanotar-tiny", dtype=F32)
    mix = m.layers[0].mixer
    uq = mix.wuq.view(mix.d.heads, mix.dp, mix.qp)
    assert uq[:, : mix.d.dim, : mix.d.q_rank].any()
    assert not uq[:, mix.d.dim:].any()
    assert m.layers[2].mixer.d.kv_from == 1


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
    """Growth past the model length or the pool is an error before
    anything is written."""
    from distllm_amd.engine.engine import _Seq

    e = case.engine(tokens=64, num_blocks=3)
    s = _Seq(0, [])
    with pytest.raises(RuntimeError, match="max_model_len"):
        cases.feed(e, s, case.tokens(65, 94))
    with pytest.raises(RuntimeError, match="exhausted"):
        cases.feed(e, s, case.tokens(60, 94))
    assert len(e.blockman.free) == 3 and s.cached == 0


def test_unsupported_options(case):
    with pytest.raises(ValueError, match="dtype"):
        case.model.make_cache(4, 16, "fp8_e4m3")
    with pytest.raises(ValueError, match="tensor_parallel"):
        build_model("kanotar-tiny", tp_group=object())


def test_trace_replay(case, tmp_path):
    """The replay tool's reader and writer around engine steps."""
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
    assert not rp.live


def test_trace_run_needs_gpu(case, tmp_path, monkeypatch, capsys):
    from distllm_amd.engine import trace

    monkeypatch.setattr(torch.cuda, "is_available", lambda: False)
    assert trace.main(["--model", str(case.path), "--out", str(tmp_path),
                       "--max-tokens", "64"]) == 1
    assert "GPU" in capsys.readouterr().err


def test_native_generator_from_folder(tmp_path):
    """generate's entry point picks the model class by config.json."""
    from distllm_amd.generate import get_generator

    cfg = oracle.make_config(cases.mixed_layers(), vocab=1200)
    c = cases.Case(tmp_path, "cpu", F32, cfg, seed=8)
    gen = get_generator({"name": "native", "model": str(c.path),
                         "temperature": 0.0, "min_p": 0.0, "max_tokens": 5,
                         "max_model_len": 128, "max_batch_size": 2})
    assert type(gen.model).__name__ == "KanotarModel"
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
