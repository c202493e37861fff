"""Checks of the Kedelorn model and engine path, run on the CPU by
test_kedelorn.py and on the GPU by test_kedelorn_gpu.py.

Every check compares with the plain implementation in kedelorn_oracle.py;
those that hold for any design are tebasun_cases'. In 16 bits rounding
swaps experts of nearly equal scores, which is no fault: there, corrections
far apart decide the choice (choices by scores are tested on given inputs
and in 32 bits).
"""

import torch

import kedelorn_oracle as oracle
import tebasun_cases as common
from kanotar_cases import feed, run_cut  # noqa: F401
from tebasun_cases import (check_batches, check_first_tokens,  # noqa: F401
                           check_greedy, check_long_decode, check_portions,
                           check_reuse, check_whole, oracle_greedy, rel)

F32, BF16 = torch.float32, torch.bfloat16
TOL = {F32: 6e-5, BF16: 8e-2}


def mixed_layers():
    """Unequal layers: both mixers with and without a feed-forward, own and
    shared latents, rotations of a part and of all of a head, with and
    without scaling, experts with and without a shared one."""
    o = oracle
    whole = {"base": 50.0, "dims": 12}
    plain = {"base": 200.0, "dims": 6}
    return [
        o.retention_layer(o.moe_mlp()),
        o.latent_layer(o.moe_mlp(experts=9, top=4, scale=0.6, shared=None)),
        o.latent_layer(None, heads=6, dim=12, vdim=20, kv_rank=40,
                       rot_dim=6, rot=plain, scale=0.3),
        o.retention_layer(None, heads=2, dim=12, vdim=16, rot=whole,
                          decay=[0.5, 1.0]),
        o.latent_layer(o.moe_mlp(ff=70, top=1, shared=9), heads=2, dim=24,
                       vdim=8, kv_from=1, scale=0.4),
        o.retention_layer(o.moe_mlp(experts=3, top=3), heads=5, dim=9,
                          vdim=7, rot={"base": 30.0, "dims": 2}),
        o.latent_layer(o.moe_mlp(), heads=3, dim=8, vdim=16, kv_rank=40,
                       rot_dim=6, rot=plain, kv_from=2),
    ]


def mixed_config(**kw):
    return oracle.make_config(mixed_layers(), **kw)


def decide(tensors, seed):
    """Corrections so far apart that scores do not matter for the choice."""
    g = torch.Generator().manual_seed(seed)
    for k, v in tensors.items():
        if k.endswith(".correction"):
            v.copy_(2.0 * torch.randperm(len(v), generator=g))


class Case(common.Case):
    oracle = oracle
    TOL = TOL

    @staticmethod
    def default_config():
        return mixed_config()

    def __init__(self, tmp, device, dtype, config=None, seed=0, gain=None,
                 edit=None):
        def edit_all(t):
            if dtype == BF16:
                decide(t, seed)
            if edit is not None:
                edit(t)

        super().__init__(tmp, device, dtype, config, seed, gain, edit_all)


def check_residuals(c: Case, n=40):
    """The sum of the streams after every layer."""
    from distllm_amd.engine.step import StepBatch

    toks = c.tokens(n, 2)
    want, got = [], []
    oracle.forward(c.config, c.tensors, toks, want)
    cache = c.model.make_cache(n // 16 + 2, 16, "bf16", 2)
    batch = StepBatch.build([(toks, 0, list(range(1, n // 16 + 2)))], 16,
                            c.model.device, slots=[1])
    hidden = c.model.forward_step(batch, cache, trace=got)
    assert len(got) == len(want) == len(c.config["layers"])
    assert all(g.dtype == F32 for g in got)
    for g, w in zip(got, want):
        assert rel(g[:n], w) < TOL[c.dtype]
    c.passes(c.model.logits(hidden)[:n], toks)


def check_sizes(tmp, device, dtype):
    """Sizes of 1, sizes that are no multiple of anything, equal sizes
    that usually differ, all constants away from their usual values."""
    o = oracle
    M, R, L, X = o.make_config, o.retention_layer, o.latent_layer, o.moe_mlp
    configs = [
        M([R(X(1, 1, 1, 1.0, 1), heads=1, dim=2, vdim=1,
             rot={"base": 10.0, "dims": 2}, decay=[0.9]),
           L(None, heads=1, dim=1, rot_dim=2, vdim=1, kv_rank=1,
             rot=o.yarn(2))], width=2, vocab=3, streams=1),
        M([L(X(33, 5, 2, 0.3, 130), heads=7, dim=9, rot_dim=4, vdim=33,
             kv_rank=70, rot=o.yarn(4, 20.0, 8.0, 100, 9.0, 0.1),
             scale=0.2),
           R(X(70, 17, 5, 3.0, None), heads=7, dim=33, vdim=65,
             rot={"base": 1e4, "dims": 14}),
           L(X(8, 2, 1), heads=3, dim=20, rot_dim=4, vdim=9, kv_rank=70,
             rot=o.yarn(4, 20.0, 8.0, 100, 9.0, 0.1), kv_from=0)],
          width=29, vocab=31, eps=0.3, streams=6),
        M([R(X(64), heads=2, dim=130, vdim=70, decay=[0.99, 0.7],
             rot={"base": 1e4, "dims": 128}),
           L(X(64), heads=2, dim=100, rot_dim=64, vdim=130, kv_rank=130,
             rot=o.yarn(64, 1e4, 2.0, 32, 2.0, 1.0), scale=0.1)],
          width=130, vocab=64, streams=2),
        M([R(None, heads=4, dim=64, vdim=64, rot={"base": 1e4, "dims": 64}),
           R(None, heads=1, dim=70, vdim=200, decay=[0.95],
             rot={"base": 1e4, "dims": 48})], width=64, vocab=64, streams=4),
        M([L(None, heads=34, dim=129, rot_dim=64, vdim=129, kv_rank=200,
             rot={"base": 100.0, "dims": 64}, scale=0.1),
           L(None, heads=17, dim=60, rot_dim=64, vdim=70, kv_rank=200,
             rot={"base": 100.0, "dims": 64}, scale=0.1, kv_from=0)],
          width=200, vocab=300, streams=3),
        M([L(X(20, 40, 3), heads=2, dim=30, rot_dim=72, vdim=260,
             kv_rank=600, rot=o.yarn(72), scale=0.1),
           R(X(20, 70, 2), heads=2, dim=200, vdim=64, decay=[0.8, 0.999],
             rot={"base": 1e3, "dims": 200}),
           R(None, heads=1, dim=20, vdim=290, decay=[0.99])], width=80,
          vocab=50, streams=9),
    ]
    for i, cfg in enumerate(configs):
        c = Case(tmp, device, dtype, cfg, seed=60 + i)
        toks = c.tokens(80, 60 + i)
        for cuts in ([80], [41, 1, 2, 34, 1]):
            err = c.error(run_cut(c.engine(), toks, cuts), toks)
            assert err < TOL[dtype], (i, cuts, err)


# ---- weights that make one fault show ---------------------------------------

def differs(c: Case, other, toks, factor=4):
    """The yardstick with something left out or changed is far away."""
    far = rel(other, c.want(toks))
    assert far > factor * TOL[c.dtype], far


def without(c: Case, toks, **names):
    """The yardstick's logits with tensors replaced."""
    return oracle.forward(c.config, {**c.tensors, **names}, toks)


def check_far_key(tmp, device, dtype, n=150, rotated=False):
    """An attention layer that finds one token by its content: queries and
    keys are constant but for a rare token's key, so that the logits depend
    on where that token is, from any distance and at page borders. The key
    is found through the latent or through the rotated part (a rotation so
    slow that it hardly turns)."""
    o = oracle
    rot = {"base": 1e12, "dims": 4}
    cfg = o.make_config([o.latent_layer(
        None, heads=2, dim=8, rot_dim=4, vdim=8, kv_rank=16, rot=rot,
        scale=1.0)], width=32, vocab=40, streams=2)

    def edit(t):
        q = "l0.mix."
        t["l0.norm1"][:] = 0
        t["embed"][:, 0] = 0
        t["embed"][:, 1] = 1.0
        t["embed"][1] = 0
        t["embed"][1, 0] = 4.0
        t["embed"][1, 1] = 1.0
        for nm in ("q", "dkv", "uk"):
            t[q + nm] *= 0.02
        t[q + "dkv.norm"][:] = 1.0
        t[q + "sink"][:] = -20.0
        t[q + "o"] *= 3
        if rotated:
            # the second pair hardly turns: numbers 1 and 3 of four
            t[q + "q"].view(2, 12, 32)[:, 9, 1] = 12.0
            t[q + "dkv"][17, 0] = 6.0
        else:
            t[q + "q"].view(2, 12, 32)[:, 3, 1] = 12.0
            t[q + "dkv"][5, 0] = 6.0       # number 5 of the latent
            t[q + "uk"].view(2, 8, 16)[:, 3, 5] = 6.0

    c = Case(tmp, device, dtype, cfg, seed=76 + rotated, edit=edit)
    base = [t if t != 1 else 2 for t in c.tokens(n, 4)]
    for pos in (0, 1, 15, 16, 31, 32, 63, 64, 100):
        toks = list(base)
        toks[pos] = 1
        want = c.want(toks)
        assert rel(c.want(base)[-20:], want[-20:]) > 4 * TOL[dtype], pos
        for cuts in ([n], [pos + 1, 1], [40, 2, 33]):
            c.passes(run_cut(c.engine(), toks, cuts), toks)


def check_sink_and_gate(tmp, device, dtype):
    """Sinks far above and far below the scores, gates that open and shut
    heads; without either the logits would be others."""
    o = oracle
    cfg = o.make_config([o.latent_layer(None, heads=3)], width=32, vocab=40)

    def edit(t):
        t["l0.mix.sink"] = torch.tensor([6.0, -30.0, 60.0]).to(BF16)
        t["l0.mix.g"] *= 8

    c = Case(tmp, device, dtype, cfg, seed=75, edit=edit)
    toks = c.tokens(80, 5)
    differs(c, without(c, toks, **{"l0.mix.sink": torch.full((3,), -99.)}),
            toks)
    differs(c, without(c, toks, **{"l0.mix.g": torch.zeros(3, 32)}), toks)
    for cuts in ([80], [1], [2], [40, 1, 33, 2]):
        c.passes(run_cut(c.engine(), toks, cuts), toks)


def check_shared_latents(tmp, device, dtype):
    """A layer that reads another layer's latents as the cache holds them,
    with scores, values, sinks and gates of its own, other layers between."""
    o = oracle
    cfg = o.make_config([
        o.latent_layer(None), o.retention_layer(None),
        o.latent_layer(None, kv_rank=40),
        o.latent_layer(None, heads=2, dim=30, vdim=18, kv_from=0)],
        width=32, vocab=40)
    c = Case(tmp, device, dtype, cfg, seed=79)
    toks = c.tokens(70, 7)
    other = {**cfg, "layers": [*cfg["layers"][:3], o.latent_layer(
        None, heads=2, dim=30, vdim=18)]}
    fake = {**c.tensors, "l3.mix.dkv": c.tensors["l0.mix.dkv"],
            "l3.mix.dkv.norm": c.tensors["l0.mix.dkv.norm"]}
    differs(c, o.forward(other, fake, toks), toks)  # latents of its own
    engine = c.engine()
    assert engine.cache.layers[3] is engine.cache.layers[0]
    for cuts in ([70], [1], [33, 1, 2]):
        c.passes(run_cut(c.engine(), toks, cuts), toks)


def check_state_memory(tmp, device, dtype):
    """A retention layer that never forgets beside heads that do: the
    logits of the last token depend on the first one, through prompts,
    portions and decoded tokens."""
    o = oracle
    cfg = o.make_config([o.retention_layer(
        None, heads=3, dim=16, vdim=16, decay=[1.0, 0.998046875, 0.25],
        rot={"base": 1e4, "dims": 16})], width=32, vocab=40)

    def edit(t):
        t["l0.mix.o"] *= 3
        t["embed"][1] *= 6  # normed, but its keys and values are aligned
        t["l0.mix.k"] *= 2

    c = Case(tmp, device, dtype, cfg, seed=77, edit=edit)
    toks = [1, 2] + c.tokens(13, 5) * 6
    other = [3] + toks[1:]
    if dtype == F32:
        assert rel(c.want(other)[-20:], c.want(toks)[-20:]) > 20 * TOL[dtype]
    for cuts in ([80], [2], [1], [40, 1], [33, 47], [17, 30, 33]):
        c.passes(run_cut(c.engine(), toks, cuts), toks)


def check_streams(tmp, device, dtype):
    """Mixing matrices far from symmetric, streams that are read and written
    unequally: the yardstick with transposed ones, or with streams that are
    not mixed, is far away."""
    o = oracle
    cfg = o.make_config([o.retention_layer(o.moe_mlp()),
                         o.latent_layer(o.moe_mlp())], width=32, vocab=40,
                        streams=4)

    def edit(t):
        g = torch.Generator().manual_seed(3)
        for k in t:
            if ".hc" in k:
                t[k] = (torch.randn(t[k].shape, generator=g) * 0.6).to(BF16)

    c = Case(tmp, device, dtype, cfg, seed=80, edit=edit)
    toks = c.tokens(50, 8)
    mixes = [k for k in c.tensors if k.endswith(".mix")]
    assert len(mixes) == 4
    for k in mixes[1:]:  # the streams are equal before the first
        differs(c, without(c, toks, **{k: c.tensors[k].T}), toks, 2)
        differs(c, without(c, toks, **{k: torch.eye(4)}), toks, 2)
    for cuts in ([50], [1], [33, 1, 2]):
        c.passes(run_cut(c.engine(), toks, cuts), toks)


def check_router(tmp, device, dtype):
    """The correction takes part in the choice and not in the weights, the
    weights are scaled and not renormalized, the shared expert has a gate of
    its own."""
    o = oracle
    cfg = o.make_config([o.retention_layer(o.moe_mlp(top=3, scale=2.2))],
                        width=32, vocab=40)
    c = Case(tmp, device, dtype, cfg, seed=81)
    toks = c.tokens(50, 9)
    E = cfg["layers"][0]["mlp"]["router"]["experts"]
    differs(c, without(c, toks, **{"l0.mlp.correction": torch.zeros(E)}),
            toks)
    differs(c, without(c, toks, **{"l0.mlp.shared.sg": torch.zeros(1, 32)}),
            toks)
    plain = {**cfg, "layers": [o.retention_layer(o.moe_mlp(top=3,
                                                           scale=1.0))]}
    differs(c, c.want(toks, plain), toks)
    for cuts in ([50], [1], [33, 1, 2]):
        c.passes(run_cut(c.engine(), toks, cuts), toks)
