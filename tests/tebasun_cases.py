"""Checks of the Tebasun model and engine path, run on the CPU by
test_tebasun.py and on the GPU by test_tebasun_gpu.py.

Every check compares with the plain implementation in tebasun_oracle.py.
Errors are root mean squares over the vocabulary relative to the logits'
own; `TOL` holds what rounding may cause per dtype.
"""

import json

import torch
from safetensors.torch import save_file

import tebasun_oracle as oracle
from distllm_amd.engine import LLMEngine, SamplingParams
from distllm_amd.engine.engine import _Seq
from distllm_amd.models import load_pretrained
from kanotar_cases import feed, run_cut

F32, BF16 = torch.float32, torch.bfloat16
TOL = {F32: 6e-5, BF16: 8e-2}


def rel(got, want, spare=0):
    """Rms difference per row over the rms of all wanted logits: the worst
    row, or of many rows three times the mean where that is more. `spare`
    rows count a third."""
    d = got.double().cpu() - want
    d = d - d.mean(-1, keepdim=True)
    scale = (want - want.mean(-1, keepdim=True)).pow(2).mean().sqrt()
    rows = (d.pow(2).mean(-1).sqrt() / scale).sort().values
    rows[len(rows) - spare:] /= 3
    return float(max(rows.max(), 3 * rows.mean() if len(rows) > 8 else 0))


def mixed_layers():
    """Unequal layers: both mixers with and without a feed-forward, shared
    queries and keys on either side, rotations of a part and of all of a
    head, with and without scaling, several tap and block counts."""
    o = oracle
    whole = o.rotation(dims=12, base=50.0, factor=3.0, original=40)
    plain = {"base": 300.0, "dims": 6}
    return [
        o.rglru_layer(o.dense_mlp(40)),
        o.parallel_layer(o.dense_mlp()),
        o.rglru_layer(None, width=36, blocks=3, conv=2),
        o.parallel_layer(None, heads=6, kv_heads=3, dim=12, rot=whole,
                         right={"heads": 4, "kv_heads": 2, "dim": 10,
                                "vdim": 14, "conv": 3}),
        o.parallel_layer(o.dense_mlp(72), heads=2, kv_heads=1, dim=10,
                         rot=plain, left_scale=1.3, right_scale=0.4,
                         right={"heads": 2, "kv_heads": 1, "conv": 1}),
    ]


def mixed_config(**kw):
    kw.setdefault("loop", (1, 3, 3))
    return oracle.make_config(mixed_layers(), **kw)


class Case:
    """gain: in 16 bits smaller by default, as a norm of numbers that
    happen to be small magnifies rounding. Models of other designs have
    their own `oracle` and `default_config`."""

    oracle = oracle
    TOL = TOL

    @staticmethod
    def default_config():
        return mixed_config()

    def __init__(self, tmp, device, dtype, config=None, seed=0, gain=None,
                 edit=None):
        self.config = config or self.default_config()
        gain = gain or (1.0 if dtype == F32 else 0.7)
        self.tensors = self.oracle.make_tensors(self.config, seed, gain)
        if edit is not None:
            edit(self.tensors)
        self.device, self.dtype = device, dtype
        d = tmp / f"ckpt{seed}"
        d.mkdir(exist_ok=True)
        (d / "config.json").write_text(json.dumps(self.config))
        save_file(self.tensors, str(d / "model.safetensors"))
        self.path = d
        self.model = load_pretrained(d, device=device, dtype=dtype)
        self._want: dict = {}

    def engine(self, tokens=512, **kw):
        kw.setdefault("max_batch_size", 4)
        kw.setdefault("num_blocks", (tokens + 15) // 16)
        return LLMEngine(self.model, max_model_len=tokens, **kw)

    def tokens(self, n, seed):
        g = torch.Generator().manual_seed(3000 + seed)
        return torch.randint(0, self.config["vocab"], (n,),
                             generator=g).tolist()

    def want(self, toks, config=None):
        key = (tuple(toks), json.dumps(config))
        if key not in self._want:
            self._want[key] = self.oracle.forward(config or self.config,
                                                  self.tensors, toks)
        return self._want[key]

    def error(self, got, toks):
        """rel() of the logits of all of toks. In 16 bits a norm of numbers
        that happen to be small magnifies rounding in a row now and then."""
        spare = 0 if self.dtype == F32 else (len(toks) + 24) // 40
        return rel(got, self.want(toks), spare)

    def passes(self, got, toks):
        err = self.error(got, toks)
        assert err < self.TOL[self.dtype], (len(toks), err)


def check_whole(c: Case, n=90):
    toks = c.tokens(n, 1)
    c.passes(feed(c.engine(), _Seq(0, []), toks), toks)


def check_residuals(c: Case, n=40):
    """The residual stream after every layer run, looped layers each time."""
    from distllm_amd.engine.step import StepBatch

    toks = c.tokens(n, 2)
    want, got = [], []
    oracle.forward(c.config, c.tensors, toks, want)
    cache = c.model.make_cache(n // 16 + 2, 16, "bf16", 2)
    batch = StepBatch.build([(toks, 0, list(range(1, n // 16 + 2)))], 16,
                            c.model.device, slots=[1])
    hidden = c.model.forward_step(batch, cache, trace=got)
    loop = c.config["loop"]
    assert len(got) == len(want) == len(c.config["layers"]) + \
        (loop["times"] - 1) * (loop["stop"] - loop["start"])
    assert all(g.dtype == F32 for g in got)
    for g, w in zip(got, want):
        assert rel(g[:n], w) < TOL[c.dtype]
    c.passes(c.model.logits(hidden)[:n], toks)


def check_first_tokens(c: Case):
    """Sequences of one token, two and a few more: nothing before the
    start enters the convolutions, the states or the attention."""
    for n in (1, 2, 3, 4, 5):
        toks = c.tokens(n, 20 + n)
        for cuts in ([n], [1], [2, 1]):
            c.passes(run_cut(c.engine(), toks, cuts), toks)


def check_portions(c: Case, n=150):
    """Cut anywhere: single tokens, two tokens, in and across pages,
    chunks and the sizes at which the form of a mixer changes."""
    toks = c.tokens(n, 3)
    for cuts in ([1], [2], [31, 1], [32, 2, 33], [70, 1], [15, 1, 16, 17],
                 [3, 64, 3, 47, 2], [65, 63, 1], [n - 1, 1]):
        c.passes(run_cut(c.engine(), toks, cuts), toks)


def check_batches(c: Case):
    """Unequal requests together, each against itself alone: prompt
    portions of several sizes beside single decoded tokens, a request
    that pauses, requests that end and others that take their pages and
    state slots."""
    lens = {"a": 130, "b": 47, "c": 3, "d": 75, "e": 61, "f": 1}
    toks = {k: c.tokens(n, 10 + i) for i, (k, n) in enumerate(lens.items())}
    # name -> portion sizes, one per step from `start` on (0 = pause)
    plan = {
        "a": (0, [40, 1, 1, 0, 2, 50, 1, 33, 1, 1]),
        "b": (0, [2, 44, 1]),
        "c": (1, [1, 1, 1]),
        "f": (2, [1]),
        "d": (3, [72, 1, 1, 1]),
        "e": (4, [31, 0, 30]),
    }
    # room for what is live at once, not for the sum of all requests
    engine = c.engine(tokens=272, num_blocks=17)
    assert sum((n + 15) // 16 for n in lens.values()) > 17
    pages, slots = len(engine.blockman.free), len(engine.slotman.free)
    assert slots == 4 < len(lens)
    seqs, at = {}, dict.fromkeys(lens, 0)
    got = {k: [] for k in lens}
    for step in range(10):
        work, want, names = [], [], []
        for k, (start, sizes) in plan.items():
            i = step - start
            if 0 <= i < len(sizes) and sizes[i]:
                n = sizes[i]
                seqs.setdefault(k, _Seq(len(seqs), []))
                work.append((seqs[k], toks[k][at[k]: at[k] + n]))
                want.append(list(range(n)))
                names.append((k, n))
                at[k] += n
        logits = engine.step(work, want)
        o = 0
        for k, n in names:
            got[k].append(logits[o: o + n])
            o += n
            if at[k] == lens[k]:
                engine.release(seqs[k])
    assert at == lens
    assert len(engine.blockman.free) == pages
    assert sorted(engine.slotman.free) == [1, 2, 3, 4]
    for k in lens:
        c.passes(torch.cat(got[k]), toks[k])


def check_reuse(c: Case):
    """Pages and slots that earlier requests filled are used again, in
    another order, without a trace of what they held."""
    engine = c.engine(tokens=112, num_blocks=7, max_batch_size=1)
    for i, n in enumerate((100, 33, 112, 1, 17, 65)):
        toks = c.tokens(n, 30 + i)
        got = run_cut(engine, toks, [max(1, n // 2), 1, 2, 40])
        c.passes(got, toks)
        engine.blockman.free.reverse()
        assert engine.slotman.free == [1]


def check_sizes(tmp, device, dtype):
    """Sizes of 1, sizes that are no multiple of anything, equal sizes
    that usually differ, all constants away from their usual values, loops
    over everything, over the last layer and over none twice."""
    o = oracle
    M, P, R = o.make_config, o.parallel_layer, o.rglru_layer
    rot = o.rotation
    configs = [
        M([P(o.dense_mlp(1), heads=1, kv_heads=1, dim=2, rot=rot(2),
             right={"heads": 1, "kv_heads": 1, "dim": 1, "vdim": 1,
                    "conv": 1}),
           R(None, width=1, blocks=1, conv=1)], width=2, vocab=3, side=1,
          loop=(0, 2, 2)),
        M([R(o.dense_mlp(33), width=66, blocks=6, conv=7),
           P(None, heads=7, kv_heads=1, dim=9,
             rot=rot(4, 20.0, 8.0, 100, 9.0, 0.1), scale=0.05,
             right={"heads": 6, "kv_heads": 3, "dim": 33, "vdim": 65,
                    "conv": 7})], width=29, vocab=31, eps=0.3, side=70,
          loop=(1, 2, 4), scale=0.2),
        M([P(o.dense_mlp(130), heads=3, kv_heads=3, dim=70,
             rot=rot(64, 1e4, 2.0, 32, 2.0, 1.0),
             right={"heads": 2, "kv_heads": 2, "dim": 130, "vdim": 70,
                    "conv": 3})] * 2, width=130, vocab=64, side=64),
        M([R(None, width=96, blocks=1, conv=2),
           R(None, width=160, blocks=5, conv=4)], width=64, vocab=64),
        M([P(None, heads=34, kv_heads=2, dim=129, rot=rot(128, 100.0),
             right={"heads": 2, "kv_heads": 1, "dim": 64, "vdim": 64,
                    "conv": 4})], width=200, vocab=300, loop=(0, 1, 1)),
        M([P(o.dense_mlp(64), heads=2, kv_heads=1, dim=260, rot=rot(40),
             right={"heads": 2, "kv_heads": 1, "dim": 130, "vdim": 200,
                    "conv": 4})], width=80, vocab=50),
    ]
    for i, cfg in enumerate(configs):
        c = Case(tmp, device, dtype, cfg, seed=60 + i)
        toks = c.tokens(80, 60 + i)
        for cuts in ([80], [41, 1, 2, 34, 1]):
            err = c.error(run_cut(c.engine(), toks, cuts), toks)
            assert err < TOL[dtype], (i, cuts, err)


def oracle_greedy(c: Case, prompt, follow):
    """Per generated token, how far its logit is below the best one."""
    want = c.want(prompt + follow)
    gaps = []
    for j, t in enumerate(follow):
        row = want[len(prompt) - 1 + j]
        gaps.append(float(row.max() - row[t]))
    return gaps, float(want.pow(2).mean().sqrt())


def check_greedy(c: Case, use_loop=False):
    """Greedy generation through the engine's scheduler: more prompts
    than fit at once, unequal lengths."""
    prompts = [c.tokens(n, 70 + n) for n in (5, 61, 1, 33, 90)]
    params = SamplingParams(temperature=0.0, min_p=0.0, max_tokens=24)
    engine = c.engine(tokens=160, num_blocks=24, max_batch_size=3)
    engine.STEP_TOKENS = 40  # prompts take several steps
    pages = len(engine.blockman.free)
    if use_loop:
        from distllm_amd.engine.loop import EngineLoop

        loop = EngineLoop(engine, params)
        try:
            outs = loop.generate(prompts, 24)
        finally:
            loop.close()
    else:
        outs = engine.generate(prompts, params)
    assert len(engine.blockman.free) == pages
    assert sorted(engine.slotman.free) == [1, 2, 3]
    for p, o in zip(prompts, outs):
        assert len(o) == 24
        gaps, scale = oracle_greedy(c, p, o)
        assert max(gaps) < 3 * c.TOL[c.dtype] * scale, (len(p), gaps)


def check_long_decode(c: Case, prompt=20, new=200):
    toks = c.tokens(prompt + new, 90)
    c.passes(run_cut(c.engine(), toks, [prompt, 1]), toks)


# ---- weights that make one fault show ---------------------------------------

def check_far_key(tmp, device, dtype, n=150):
    """An attention layer that finds one token by its content: queries and
    keys are constant but for a rare token's key, so that the logits depend
    on where that token is, from any distance and at page borders. The other
    branch is silent."""
    o = oracle
    plain = {"base": 1e6, "dims": 2}
    cfg = o.make_config([o.parallel_layer(
        None, heads=2, kv_heads=1, dim=8, rot=plain, scale=2.0)],
        width=32, vocab=40, side=2)

    def edit(t):
        q = "l0.mix.left."
        t["l0.norm1.alpha"] = torch.tensor(1.0).to(BF16)
        t["embed"][1] = 0
        t["embed"][1, 0] = 4.0
        t["embed"][torch.arange(40) != 1, 0] = 0
        for nm in "qk":
            t[q + nm] *= 0.02
            t[q + nm + ".b"] *= 0
            t[q + nm + ".norm"][:] = 1.0
        t[q + "q.b"][3::8] = 6.0          # all queries look at number 3
        t[q + "k.b"][4] = 6.0             # where keys have nothing
        t[q + "k"][3, 0] = 30.0           # but for the rare token's
        t[q + "o"] *= 3
        t["l0.mix.right.o"] *= 0

    c = Case(tmp, device, dtype, cfg, seed=76, edit=edit)
    base = [t if t != 1 else 2 for t in c.tokens(n, 4)]
    for pos in (0, 1, 15, 16, 31, 32, 63, 64, 100):
        toks = list(base)
        toks[pos] = 1
        want = c.want(toks)
        assert rel(c.want(base)[-20:], want[-20:]) > 4 * TOL[dtype], pos
        for cuts in ([n], [pos + 1, 1], [40, 2, 33]):
            c.passes(run_cut(c.engine(), toks, cuts), toks)


def check_sink(tmp, device, dtype):
    """Sinks far above and far below the scores; without them the logits
    would be others."""
    o = oracle
    cfg = o.make_config([o.parallel_layer(None, heads=3, kv_heads=1)],
                        width=32, vocab=40)

    def edit(t):
        t["l0.mix.left.sink"] = torch.tensor([6.0, -30.0, 60.0]).to(BF16)

    c = Case(tmp, device, dtype, cfg, seed=75, edit=edit)
    toks = c.tokens(80, 5)
    off = dict(c.tensors)
    off["l0.mix.left.sink"] = torch.full((3,), -100.0).to(BF16)
    assert rel(oracle.forward(cfg, off, toks), c.want(toks)) > 4 * TOL[dtype]
    for cuts in ([80], [1], [2], [40, 1, 33, 2]):
        c.passes(run_cut(c.engine(), toks, cuts), toks)


def check_state_memory(tmp, device, dtype, kind):
    """A recurrent layer that hardly forgets: the logits of the last token
    depend on the first one, through prompts, portions and decoded
    tokens."""
    o = oracle
    cfg = o.make_config([o.rglru_layer(None, width=32, blocks=2)
                         if kind == "rglru" else o.parallel_layer(
                             None, right={"heads": 2, "kv_heads": 1,
                                          "dim": 16, "vdim": 16})],
                        width=32, vocab=40)

    def edit(t):
        if kind == "rglru":
            t["l0.mix.lam"] = torch.full((32,), -9.0).to(BF16)
            t["l0.mix.ri.b"][:] = 2.0
            t["l0.mix.conv"] *= 8
            t["l0.mix.o"] *= 20
        else:
            t["l0.mix.right.A_log"] = torch.full((2,), -9.0).to(BF16)
            t["l0.mix.left.o"] *= 0
            t["l0.mix.right.o"] *= 3

    c = Case(tmp, device, dtype, cfg, seed=77, edit=edit)
    toks = [1, 2] + c.tokens(13, 5) * 6
    other = [3] + toks[1:]
    if dtype == F32:
        assert rel(c.want(other)[-20:], c.want(toks)[-20:]) > 20 * TOL[dtype]
    for cuts in ([80], [2], [1], [40, 1], [33, 47]):
        c.passes(run_cut(c.engine(), toks, cuts), toks)


def check_strong_decay(tmp, device, dtype):
    """Decays from next to none to a state that is gone in one token, side
    by side in the channels of a head: nothing overflows, nothing that
    should stay is lost."""
    o = oracle
    cfg = o.make_config([o.parallel_layer(None, right={
        "heads": 2, "kv_heads": 1, "dim": 16, "vdim": 16})], width=32,
        vocab=40)

    def edit(t):
        t["l0.mix.right.A_log"] = torch.tensor([3.0, 0.0]).to(BF16)
        t["l0.mix.right.dt_bias"] = torch.linspace(-12, 6, 32).to(BF16)

    c = Case(tmp, device, dtype, cfg, seed=78, edit=edit)
    toks = c.tokens(110, 6)
    for cuts in ([110], [1], [50, 2, 58]):
        c.passes(run_cut(c.engine(), toks, cuts), toks)


def check_loop(tmp, device, dtype):
    """Every pass of a loop has a state and a cache of its own, starts from
    its own vector and, but for the first, from the embedding output once
    more: the yardstick without any of them is far away."""
    o = oracle
    cfg = o.make_config([o.rglru_layer(None), o.parallel_layer(None),
                         o.rglru_layer(o.dense_mlp())], loop=(0, 2, 3))
    c = Case(tmp, device, dtype, cfg, seed=79)
    toks = c.tokens(70, 7)
    want = c.want(toks)
    fewer = json.loads(json.dumps(cfg))
    fewer["loop"]["times"] = 2
    assert rel(c.want(toks, fewer), want) > 4 * TOL[dtype]
    for k in range(3):
        t = dict(c.tensors)
        t["loop.step"] = t["loop.step"].clone()
        t["loop.step"][k] = 0
        assert rel(o.forward(cfg, t, toks), want) > 2 * TOL[dtype]
    mixers = [x for x, _ in c.model.runs]
    assert mixers == [0, 1, 0, 1, 0, 1, 2]
    for cuts in ([70], [1], [33, 1, 2]):
        c.passes(run_cut(c.engine(), toks, cuts), toks)
