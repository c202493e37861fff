"""Kedelorn on the CPU: every mechanism and the engine path against the
plain implementation."""

import json

import pytest
import torch

import kedelorn_cases as cases
import kedelorn_oracle as oracle
from distllm_amd import ops
from distllm_amd.engine.step import Segments, StepBatch
from distllm_amd.models import build_model, dims_from_checkpoint, get_dims
from distllm_amd.models.config import CONFIG_READERS, RotaryDims

F32 = torch.float32


@pytest.fixture(scope="module")
def case(tmp_path_factory):
    return cases.Case(tmp_path_factory.mktemp("k"), "cpu", F32)


def test_whole_prompt(case):
    cases.check_whole(case)


def test_residual_stream(case):
    cases.check_residuals(case)


def test_first_tokens(case):
    cases.check_first_tokens(case)


def test_portions(case):
    cases.check_portions(case, 110)


def test_mixed_batches(case):
    cases.check_batches(case)


def test_page_and_slot_reuse(case):
    cases.check_reuse(case)


@pytest.mark.parametrize("rotated", [False, True])
def test_far_key(tmp_path, rotated):
    cases.check_far_key(tmp_path, "cpu", F32, rotated=rotated)


def test_sink_and_gate(tmp_path):
    cases.check_sink_and_gate(tmp_path, "cpu", F32)


def test_shared_latents(tmp_path):
    cases.check_shared_latents(tmp_path, "cpu", F32)


def test_state_memory(tmp_path):
    cases.check_state_memory(tmp_path, "cpu", F32)


def test_streams(tmp_path):
    cases.check_streams(tmp_path, "cpu", F32)


def test_router(tmp_path):
    cases.check_router(tmp_path, "cpu", F32)


def test_other_sizes(tmp_path):
    cases.check_sizes(tmp_path, "cpu", F32)


def test_greedy_generation(case):
    cases.check_greedy(case)


def test_greedy_generation_loop(case):
    cases.check_greedy(case, use_loop=True)


def test_long_decode(case):
    cases.check_long_decode(case)


def test_bf16_on_cpu(tmp_path):
    """The 16-bit mode, whose boundaries keep the streams in 32 bits."""
    c = cases.Case(tmp_path, "cpu", torch.bfloat16, seed=2)
    cases.check_whole(c, 40)
    cases.check_residuals(c, 20)


# ---- mechanisms alone ------------------------------------------------------

def _rand(*shape, seed=0):
    g = torch.Generator().manual_seed(seed)
    return torch.randn(*shape, generator=g)


def _i32(*v):
    return torch.tensor(v, dtype=torch.int32)


@pytest.mark.parametrize("S", [1, 2, 3, 5])
def test_stream_step(S):
    """Every piece of a boundary, alone and together; padded columns stay
    out of the norm's statistics."""
    W, n, M, eps = 64, 50, 4, 0.1
    x0, y = _rand(M, S, W), _rand(M * 2, W, seed=1)
    shared, mix = _rand(M, W, seed=2), torch.rand(M, 3)
    table, tok = _rand(9, W, seed=3), torch.tensor([3, 8, 3, 0])
    w, coef = _rand(W, seed=4), _rand(S * (S + 2), seed=5)
    for t in (x0, y, shared, table, w):
        t[..., n:] = 0
    mix[1, 0], y[2] = 0, float("nan")  # no expert: its row is not looked at
    t = {"h.in": coef[:S], "h.out": coef[S: 2 * S],
         "h.mix": coef[2 * S:].view(S, S)}
    t = {k: v.double() for k, v in t.items()}
    weighted = (y.view(M, 2, W).nan_to_num() * mix[:, :2, None]).sum(1) \
        + shared * mix[:, 2:]
    for embed in (None, (tok, table)):
        for out, kw in ((None, {}), (shared, {"y": shared}),
                        (weighted, {"y": y, "mix": mix, "shared": shared})):
            for read in (coef[:S], None):
                for store in (True, False):
                    x = x0.clone()
                    if kw:
                        kw["writes"] = coef[S:]
                    h = ops.stream_step(x, embed=embed, read=read,
                                        norm=(w, n, eps), store=store,
                                        dtype=F32, **kw)
                    X = (x0.transpose(0, 1) if embed is None else
                         table[tok].expand(S, -1, -1)).double()
                    if out is not None:
                        X = oracle.write(X, out.double(), t, "h.")
                    u = X.sum(0) if read is None else oracle.read(X, t, "h.")
                    want = oracle.norm(u[:, :n], w[:n] - 1, eps)
                    assert torch.allclose(h[:, :n].double(), want, atol=1e-4)
                    assert not h[:, n:].any()
                    kept = X if store and out is not None else \
                        x0.transpose(0, 1).double()
                    assert torch.allclose(x.transpose(0, 1).double(), kept,
                                          atol=1e-5)


@pytest.mark.parametrize("E, top, gates", [(1, 1, 0), (5, 2, 1), (70, 7, 1),
                                           (9, 9, 0)])
def test_route_sigmoid(E, top, gates):
    h, W = _rand(6, 32), _rand(E + gates, 32, seed=1)
    corr = _rand(E, seed=2) - 3.0  # choices below zero, too
    ctx = _i32(4, 1, 0, 9, 2, 7)
    ids, w = ops.route_sigmoid(h, W, corr, ctx, top, 1.6)
    t = {"router": W[:E].double(), "correction": corr.double()}
    want_ids, want_w = oracle.route(h.double(), t, "", {"top": top,
                                                        "scale": 1.6})
    live = ctx > 0
    assert torch.equal(ids[live].long(), want_ids[live])
    assert torch.allclose(w[live, :top].double(), want_w[live], atol=1e-6)
    if gates:
        assert torch.allclose(w[live, top:].double(), oracle.sigmoid(
            h.double() @ W[E:].double().T)[live], atol=1e-6)
    assert (ids[2] == -1).all() and not w[2].any()
    if gates:  # the shared expert as three more choices
        ids3, w3 = ops.route_sigmoid(h, W, corr, ctx, top, 1.6, 3)
        assert torch.equal(ids3[:, :top], ids)
        assert torch.equal(ids3[live, top:],
                           (E + torch.arange(3)).expand(5, 3).int())
        assert torch.equal(w3, torch.cat([w[:, :top], w[:, top:].expand(
            -1, 3)], 1))
        assert (ids3[2] == -1).all()


@pytest.mark.parametrize("shared, shards", [(None, 0), (9, 1), (64, 1),
                                            (65, 2), (150, 3)])
def test_shared_expert_in_shards(shared, shards):
    """With few rows the shared expert runs among the others, with many
    beside them."""
    cfg = oracle.make_config([oracle.retention_layer(oracle.moe_mlp(
        ff=40, shared=shared))])
    t = oracle.make_tensors(cfg, 4)
    model = build_model(CONFIG_READERS["Kedelorn"](cfg), dtype=F32)
    own = dict(model.named_parameters())
    with torch.no_grad():
        for k, v in model.checkpoint(t).items():
            own[k].copy_(v)
    mlp = model.layers[0].mlp
    assert mlp.shards == shards and len(mlp.wup) == 6 + shards
    h = torch.zeros(20, 64)
    h[:, :48] = _rand(20, 48, seed=5)
    d = {k: v.double() for k, v in t.items()}
    want = oracle.moe(h[:, :48].double(), d, "l0.mlp.",
                      cfg["layers"][0]["mlp"])
    for few in (256, 8):
        mlp.FEW = few
        y, beside, w = mlp(h, torch.ones(20, dtype=torch.int32))
        assert (beside is None) == (few == 256 or shared is None)
        n = w.shape[1] - (beside is not None)
        got = (y.view(20, n, -1) * w[:, :n, None]).sum(1)
        if beside is not None:
            got = got + beside * w[:, n:]
        assert torch.allclose(got[:, :48].double(), want, atol=1e-4)


@pytest.mark.parametrize("rot_dim, tp", [(8, 64), (6, 64), (2, 64),
                                         (64, 64), (70, 128)])
@pytest.mark.parametrize("n", [0, 2, 5])
def test_rotary_latent_prep(rot_dim, tp, n):
    """Query parts turned in place or to the folded queries; latents normed
    and key parts turned, to the cache."""
    H, dp, rank, R, blk = 3, 64, 40, 64, 16
    rot = oracle.yarn(rot_dim, 30.0)
    bt = _i32(2, 0, 4, 1)[None]
    ctx, seq = _i32(18, 19, 20, 0, 21), torch.zeros(5, dtype=torch.int32)
    ab = _rand(5, H * (dp + tp) + R + tp + 64)
    q = ab[:, : H * (dp + tp)].view(5, H, dp + tp)
    kv = ab[:, H * (dp + tp):]
    q[..., dp + rot_dim:] = 0
    kv[:, rank: R], kv[:, R + rot_dim: R + tp] = 0, 0
    before = ab.clone()
    wc = torch.zeros(R)
    wc[:rank] = _rand(rank, seed=1)
    f, mult = RotaryDims(**rot).frequencies()
    table = ops.rotation_table(ctx, torch.tensor(f, dtype=torch.float64),
                               mult)
    cache = torch.full((5, blk, R + tp), 3.0)
    ql = torch.full((n, H, R + tp), 7.0)
    ops.rotary_latent_prep(ab, H, dp, tp, rank, wc, 1e-3, table, cache, bt,
                           seq, ctx, ql)
    pos = (ctx - 1).clamp(min=0)
    want = oracle.rotate(before[:, : H * (dp + tp)].view(
        5, H, dp + tp)[..., dp: dp + rot_dim].double(), pos, rot)
    got = torch.cat([ql[..., R: R + rot_dim], q[n:, :, dp: dp + rot_dim]])
    live = [0, 1, 2, 4]
    assert torch.allclose(got[live].double(), want[live], atol=1e-5)
    assert not ql[..., R + rot_dim:].any() and (ql[..., :R] == 7).all()
    same = before.clone()
    same[n:, : H * (dp + tp)] = ab[n:, : H * (dp + tp)]
    assert torch.equal(ab, same)
    assert torch.equal(q[..., :dp], before[:, : H * (dp + tp)].view(
        5, H, -1)[..., :dp])
    z = before[:, H * (dp + tp): H * (dp + tp) + R + tp].double()
    c = oracle.rms(z[:, :rank], 1e-3) * wc[:rank]
    kr = oracle.rotate(z[:, None, R: R + rot_dim], pos, rot)[:, 0]
    for r in live:
        row = cache[bt[0, pos[r] // blk], pos[r] % blk].double()
        assert torch.allclose(row[:rank], c[r], atol=1e-5)
        assert torch.allclose(row[R: R + rot_dim], kr[r], atol=1e-5)
        assert not row[rank: R].any() and not row[R + rot_dim:].any()
    assert (cache == 3).sum() == (5 * blk - 4) * (R + tp)


def test_squared_relu_experts():
    h, E, F, W = _rand(5, 32), 3, 64, 32
    up, down = _rand(E, F, W, seed=1), _rand(E, W, F, seed=2)
    ids = _i32(0, 2, 1, 0, -1, -1, 2, 1, 1, 2).view(5, 2)
    y = ops.experts(h, ids, up, down, gated=False).view(5, 2, W)
    for m in range(5):
        for k, e in enumerate(ids[m].tolist()):
            if e >= 0:
                t = {"up": up[e].double(), "down": down[e].double()}
                want = oracle.expert(h[m].double(), t, "")
                assert torch.allclose(y[m, k].double(), want, rtol=1e-4,
                                      atol=1e-3)
    z = ops.up_relu2(h, up[0])
    assert torch.allclose(z, torch.relu(h @ up[0].T) ** 2, rtol=1e-5)


def _mixer(entry, T, W=48, seed=3):
    """A model of one layer, inputs of its mixer, and what comes out."""
    cfg = oracle.make_config([entry], width=W)
    t = oracle.make_tensors(cfg, seed)
    model = build_model(CONFIG_READERS["Kedelorn"](cfg), dtype=F32)
    own = dict(model.named_parameters())
    with torch.no_grad():
        for k, v in model.checkpoint(t).items():
            own[k].copy_(v)
    h = torch.zeros(T, 64)
    h[:, :W] = _rand(T, W, seed=seed)
    d = {k: v.double() for k, v in t.items()}
    want = oracle.MIXERS[entry["type"]](h[:, :W].double(), d, "l0.mix.",
                                        entry["mixer"], 2e-5, [])
    return model.layers[0].mixer, h, want


@pytest.mark.parametrize("cut", [1, 2, 3, 17, 33])
@pytest.mark.parametrize("entry", [
    oracle.retention_layer(None),
    oracle.retention_layer(None, heads=1, dim=70, vdim=3, decay=[1.0],
                           rot={"base": 9.0, "dims": 70}),
    oracle.latent_layer(None), oracle.latent_layer(
        None, heads=5, dim=70, rot_dim=2, vdim=65, kv_rank=33,
        rot={"base": 20.0, "dims": 2}),
    oracle.latent_layer(None, heads=1, dim=3, rot_dim=66, vdim=5,
                        kv_rank=9, scale=0.1)])
def test_mixer_alone(entry, cut):
    """A mixer against the plain one, its state and cache carried over a
    cut; slots of other sequences are left alone."""
    mix, h, want = _mixer(entry, 40)
    cache = mix.make_cache(4, 16, 3, F32, "cpu")
    cache.fill_(7.0)  # what slots and pages held before
    got = []
    with torch.no_grad():
        for a, b in ((0, cut), (cut, 40)):
            batch = StepBatch.build([(list(range(b - a)), a, [3, 1, 2])], 16,
                                    "cpu", slots=[2])
            hp = torch.zeros(batch.tokens.shape[0], 64)
            hp[: b - a] = h[a:b]
            got.append(mix(hp, batch, cache)[: b - a, :48])
    assert torch.allclose(torch.cat(got).double(), want, atol=3e-5)
    if entry["type"] == "retention":
        assert (cache[:2] == 7).all()
    else:
        assert (cache[0] == 7).all() and (cache[2, 8:] == 7).all()


def test_pieces():
    """Long segments in pieces that fill the GPU, whole chunks each."""
    seg = Segments.build([0, 3, 20, 90], [3, 17, 70, 1], [1, 2, 3, 4], "cpu")
    longs, pieces, several = seg.pieces(4)
    assert longs.tolist() == [[1, 0], [2, 1]] and not several
    assert pieces.tolist() == [[1, 0, 17, 0, 1], [2, 0, 70, 0, 1]]
    seg = Segments.build([0, 3000], [3000, 513], [1, 2], "cpu")
    longs, pieces, several = seg.pieces(4)
    assert several
    for i, n in ((0, 3000), (1, 513)):
        own = [p for p in pieces.tolist() if p[0] == i]
        first = longs.tolist()[i][1]
        assert pieces.tolist()[first] == own[0]
        assert [p[3] for p in own] == list(range(len(own)))
        assert all(p[4] == len(own) for p in own)
        at = 0
        for p in own:
            assert p[1] == at and p[1] % 32 == 0 and 0 < p[2] <= 256 + 32
            at += p[2]
        assert at == n
    assert Segments.build([0], [16], [1], "cpu").pieces(4) == \
        (None, None, False)


# ---- configuration and loading ---------------------------------------------

def test_config_and_registry(case):
    d = dims_from_checkpoint(case.path)
    assert d.arch == "kedelorn" and d.num_layers == 7 and d.streams == 3
    assert [x.mixer.type for x in d.layers] == [
        "retention", "rotary_latent", "rotary_latent", "retention",
        "rotary_latent", "retention", "rotary_latent"]
    assert d.layers[0].mlp.shared == 28 and d.layers[1].mlp.shared is None
    assert d.layers[2].mlp is None and d.layers[4].mixer.kv_from == 1
    assert d.layers[2].mixer.rot.scaling is None
    engine = case.engine()
    layers = engine.cache.layers
    assert layers[4] is layers[1] and layers[6] is layers[2]
    assert layers[0].shape[0] == 5 == engine.max_batch_size + 1
    m = case.model
    per_token = sum(x.mixer.cache_numel() for x in m.layers)
    assert per_token == 2 * 128  # two layers own latents
    assert m.cache_bytes_per_block(16, "bf16") == per_token * 16 * 4
    assert m.state_bytes_per_slot() == (3 + 2 + 5) * 64 * 64 * 4
    assert m.layers[2].hc2 is None and m.layers[2].hc1 is not None
    assert get_dims("kedelorn-tiny").arch == "kedelorn"
    assert len(get_dims("kedelorn-8b").layers) == 32


@pytest.mark.parametrize("edit, match", [
    (lambda c: c["layers"][0]["mixer"].update(heads=4), "decays"),
    (lambda c: c["layers"][0]["mixer"].update(decay=[0.5, 0.0, 1.0]),
     "decays"),
    (lambda c: c["layers"][0]["mixer"].update(window=3), "window"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=14), "rotated"),
    (lambda c: c["layers"][1]["mixer"].update(rot_dim=6), "rot_dim"),
    (lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].update(ramp=1),
     "ramp"),
    (lambda c: c["layers"][4]["mixer"].update(kv_from=4), "earlier layer"),
    (lambda c: c["layers"][4]["mixer"].update(kv_from=0), "of its own"),
    (lambda c: c["layers"][6]["mixer"].update(kv_from=4), "of its own"),
    (lambda c: c["layers"][4]["mixer"].update(kv_rank=25), "kv_rank"),
    (lambda c: c["layers"][4]["mixer"]["rot"].update(base=2.0), "rot"),
    (lambda c: c["layers"][0].update(type="scan"), "unknown mixer"),
    (lambda c: c["layers"][0]["mlp"].update(kind="dense"), "kind"),
    (lambda c: c["layers"][0]["mlp"].update(limit=1), "limit"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(groups=1), "groups"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=7), "top"),
    (lambda c: c["layers"][0]["mlp"]["shared"].update(gate=1), "shared"),
    (lambda c: c.update(streams=0), "streams"),
])
def test_config_rejects(case, edit, match):
    cfg = json.loads(json.dumps(case.config))
    edit(cfg)
    with pytest.raises(ValueError, match=match):
        CONFIG_READERS["Kedelorn"](cfg)


def test_loader_rejects(case, tmp_path):
    from safetensors.torch import save_file

    from distllm_amd.models import load_pretrained

    (tmp_path / "config.json").write_text(json.dumps(case.config))
    for edit, match in (
            (lambda t: t.pop("l0.hc2.mix"), "lacks"),
            (lambda t: t.update({"l4.mix.dkv": torch.ones(2)}), "unknown"),
            (lambda t: t.update({"l2.hc2.in": torch.ones(3)}), "unknown"),
            (lambda t: t.update({"l0.mlp.shared.sg": torch.ones(48)}),
             "shape"),
            (lambda t: t.update({"l0.hc1.mix": torch.ones(3, 2)}),
             "shape")):
        t = dict(case.tensors)
        edit(t)
        save_file(t, str(tmp_path / "model.safetensors"))
        with pytest.raises(ValueError, match=match):
            load_pretrained(tmp_path, dtype=F32)


def test_norms_are_stored_around_zero(case):
    got = case.model.layers[0].norm1
    want = 1 + case.tensors["l0.norm1"].float()
    assert torch.equal(got[:48], want) and not got[48:].any()
    # but not the latent's, which is a plain one
    got = case.model.layers[1].mixer.kv_norm
    assert torch.equal(got[:24], case.tensors["l1.mix.dkv.norm"].float())


def test_random_init():
    """Padding stays zero, norms and streams start as the identity."""
    m = build_model("kedelorn-tiny", dtype=F32)
    mix = m.layers[1].mixer
    q = mix.win[: mix.q_cols].view(mix.d.heads, mix.dp + mix.tp, -1)
    assert q[:, : mix.d.dim].any() and not q[:, mix.d.dim: mix.dp].any()
    assert not q[:, mix.dp + mix.d.rot_dim:].any()
    assert (m.layers[0].norm1 == 1).all() and (m.final_norm == 1).all()
    assert m.layers[0].hc1.coef.tolist() == [.5, .5, 1, 1, 1, 0, 0, 1]
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


def test_unsupported_options(case):
    with pytest.raises(ValueError, match="dtype"):
        case.model.make_cache(4, 16, "fp8_e4m3")
    with pytest.raises(ValueError, match="tensor_parallel"):
        build_model("kedelorn-tiny", tp_group=object())


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
    assert {"_hip_retention", "_hip_latent", "_hip_experts"} < set(need)
    assert not {"_hip_ops", "_hip_hybrid", "_hip_chunked", "_hip_lru"} \
        & set(need)


def test_cli_generate_from_folder(tmp_path):
    """`distllm generate --llm-name FOLDER` over a jsonl input."""
    from datasets import load_from_disk
    from typer.testing import CliRunner

    from distllm_amd.cli import app

    def edit(t):  # no end-of-text token wins
        t["head"][:4] = 0

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
