"""Checks of the Bufulorn model and engine path, run on the CPU by
test_bufulorn.py and on the GPU by test_bufulorn_gpu.py.

Every check compares with the plain implementation in bufulorn_oracle.py.
Errors are root mean squares over the vocabulary relative to the logits'
own; `TOL` holds what rounding may cause per dtype.
"""

import json

import torch
from safetensors.torch import save_file

import bufulorn_oracle as oracle
from distllm_amd.engine import LLMEngine, SamplingParams
from distllm_amd.engine.engine import _Seq
from distllm_amd.models import load_pretrained
from kanotar_cases import feed, rel, run_cut

TOL = {torch.float32: 6e-5, torch.bfloat16: 8e-2}


def mixed_layers():
    """Unequal layers: own and shared keys (the sharing layer's chunk is
    another than the owner's), both mixers and feed-forwards, several
    tap and expert counts, one layer without a feed-forward."""
    o = oracle
    return [
        o.attention_layer(o.dense_mlp(), size=20),
        o.delta_layer(o.moe_mlp(), heads=4, kv_heads=2, conv=4),
        o.attention_layer(None, heads=6, kv_heads=3, dim=12, vdim=20,
                          size=33, scale=0.3, softcap=4.0),
        o.attention_layer(o.moe_mlp(experts=8, top=3, count=2, keep=1),
                          size=7, kv_from=0),
        o.delta_layer(o.dense_mlp(72), heads=3, kv_heads=1, dim=24, vdim=40,
                      conv=2),
        o.attention_layer(o.dense_mlp(), heads=6, kv_heads=3, dim=12,
                          vdim=20, size=64, kv_from=2),
    ]


def undecided(config):
    """The same config with every expert serving every token: in 16 bits
    rounding swaps experts of nearly equal scores, which is no fault (the
    choice itself is tested on given scores)."""
    config = json.loads(json.dumps(config))
    for layer in config["layers"]:
        if (layer["mlp"] or {}).get("kind") == "moe":
            r = layer["mlp"]["router"]
            r["top"], r["groups"]["keep"] = r["experts"], r["groups"]["count"]
    return config


class Case:
    def __init__(self, tmp, device, dtype, config=None, seed=0, gain=1.5):
        self.config = config or oracle.make_config(mixed_layers())
        router = 5.0
        if dtype == torch.bfloat16:
            self.config, router = undecided(self.config), 1.0
        self.tensors = oracle.make_tensors(self.config, seed, gain, router)
        self.device, self.dtype = device, dtype
        d = tmp / f"ckpt{seed}"
        d.mkdir(exist_ok=True)
        (d / "config.json").write_text(json.dumps(self.config))
        save_file(self.tensors, str(d / "model.safetensors"))
        self.path = d
        self.model = load_pretrained(d, device=device, dtype=dtype)
        self._want: dict = {}
        self._shaky: dict = {}

    def engine(self, tokens=512, **kw):
        kw.setdefault("max_batch_size", 4)
        kw.setdefault("num_blocks", (tokens + 15) // 16)
        return LLMEngine(self.model, max_model_len=tokens, **kw)

    def tokens(self, n, seed):
        g = torch.Generator().manual_seed(2000 + seed)
        return torch.randint(0, self.config["vocab"], (n,),
                             generator=g).tolist()

    def want(self, toks, config=None):
        key = (tuple(toks), json.dumps(config))
        if key not in self._want:
            self._want[key] = oracle.forward(config or self.config,
                                             self.tensors, toks)
        return self._want[key]


    def error(self, got, toks):
        """rel() of the logits of all of toks. In 16 bits a row counts by
        what rounding does to it where that is more than the tolerance:
        a norm of numbers that happen to be small magnifies it. It is
        measured by the yardstick with weights that differ in the last
        bit of 16."""
        want = self.want(toks)
        if self.dtype == torch.float32:
            return rel(got, want)
        key = tuple(toks)
        if key not in self._shaky:
            g = torch.Generator().manual_seed(1)
            off = []
            for _ in range(3):
                t = {k: v.double() * (1 + (2 * torch.rand(
                    v.shape, generator=g) - 1) / 512)
                    for k, v in self.tensors.items()}
                d = oracle.forward(self.config, t, toks) - want
                off.append((d - d.mean(-1, keepdim=True)).pow(2).mean(-1))
            scale = (want - want.mean(-1, keepdim=True)).pow(2).mean()
            self._shaky[key] = (torch.stack(off).amax(0) / scale).sqrt()
        allow = (4 * self._shaky[key] / TOL[self.dtype]).clamp(min=1)
        assert len(toks) < 30 or (allow > 1).double().mean() < 0.15
        return rel(want + (got.double().cpu() - want) / allow[:, None], want)


def check_whole(c: Case, n=90):
    toks = c.tokens(n, 1)
    got = feed(c.engine(), _Seq(0, []), toks)
    assert c.error(got, toks) < TOL[c.dtype]


def check_residuals(c: Case, n=40):
    """The residual stream after every layer."""
    from distllm_amd.engine.step import StepBatch

    toks = c.tokens(n, 2)
    want, got = [], []
    oracle.forward(c.config, c.tensors, toks, want)
    cache = c.model.make_cache(n // 16 + 2, 16, "bf16", 2)
    batch = StepBatch.build([(toks, 0, list(range(1, n // 16 + 2)))], 16,
                            c.model.device, slots=[1])
    c.model.forward_step(batch, cache, trace=got)
    assert len(got) == len(want) == len(c.config["layers"])
    assert all(g.dtype == torch.float32 for g in got)
    for g, w in zip(got, want):
        assert rel(g[:n], w) < TOL[c.dtype]


def check_first_tokens(c: Case):
    """Sequences of one token, two and a few more: nothing before the
    start enters the convolutions, the state or the attention."""
    for n in (1, 2, 3, 4, 5):
        toks = c.tokens(n, 20 + n)
        for cuts in ([n], [1], [2, 1]):
            assert c.error(run_cut(c.engine(), toks, cuts), toks) \
                < TOL[c.dtype], (n, cuts)


def check_portions(c: Case, n=150):
    """Cut anywhere: single tokens, two tokens, in and across pages,
    chunks and the sizes at which the form of a mixer changes."""
    toks = c.tokens(n, 3)
    for cuts in ([1], [2], [31, 1], [32, 2, 33], [70, 1], [15, 1, 16, 17],
                 [3, 64, 3, 47, 2], [n - 1, 1]):
        assert c.error(run_cut(c.engine(), toks, cuts), toks) \
            < TOL[c.dtype], cuts


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
        assert c.error(torch.cat(got[k]), toks[k]) < TOL[c.dtype], k


def check_reuse(c: Case):
    """Pages and slots that earlier requests filled are used again, in
    another order, without a trace of what they held."""
    engine = c.engine(tokens=112, num_blocks=7, max_batch_size=1)
    for i, n in enumerate((100, 33, 112, 1, 17, 65)):
        toks = c.tokens(n, 30 + i)
        got = run_cut(engine, toks, [max(1, n // 2), 1, 2, 40])
        assert c.error(got, toks) < TOL[c.dtype], n
        engine.blockman.free.reverse()
        assert engine.slotman.free == [1]


def edge_case(tmp, device, dtype, size):
    """One peaky attention layer, so that a key more or less shows."""
    o = oracle
    cfg = o.make_config([o.attention_layer(
        None, heads=4, kv_heads=2, dim=16, vdim=16, size=size, scale=1.0,
        softcap=30.0)], width=64)
    return Case(tmp, device, dtype, cfg, seed=size,
                gain=2.0 if dtype == torch.float32 else 1.0)


def check_edges(c: Case, n):
    """Chunk edges in prompts, in portions and in decoding. The yardstick
    with a chunk one off must be far outside the tolerance."""
    size = c.config["layers"][0]["mixer"]["mask"]["size"]
    toks = c.tokens(n, 50)
    want = c.want(toks)
    for off in (-1, 1):
        wrong = json.loads(json.dumps(c.config))
        wrong["layers"][0]["mixer"]["mask"]["size"] = size + off
        if size + off > 0:
            assert rel(c.want(toks, wrong), want) > 4 * TOL[c.dtype]
    for cuts in ([n], [1], [size + 1, 2], [max(1, size - 1), 3, 40],
                 [n - 40, 1]):
        got = run_cut(c.engine(), toks, cuts)
        assert c.error(got, toks) < TOL[c.dtype], (size, cuts)


def check_sizes(tmp, device, dtype):
    """Sizes of 1, sizes that are no multiple of anything, equal sizes
    that usually differ, all constants away from their usual values."""
    o = oracle
    M = o.make_config
    configs = [
        M([o.attention_layer(o.dense_mlp(1), heads=1, kv_heads=1, dim=1,
                             vdim=1, size=1),
           o.delta_layer(o.moe_mlp(1, 1, 1, 1, 1), heads=1, kv_heads=1,
                         dim=1, vdim=1, conv=1)], width=2, vocab=3),
        M([o.delta_layer(None, heads=6, kv_heads=3, dim=33, vdim=65,
                         conv=7),
           o.attention_layer(o.moe_mlp(23, 10, 4, 5, 3), heads=7,
                             kv_heads=1, dim=9, vdim=11, size=19,
                             scale=0.05, softcap=0.5)],
          width=29, vocab=31, eps=0.3),
        M([o.attention_layer(None, heads=3, kv_heads=3, dim=70, vdim=130,
                             size=1000),
           o.delta_layer(o.dense_mlp(130), heads=2, kv_heads=2, dim=130,
                         vdim=70, conv=3)], width=130, vocab=64,
          max_positions=80),
        M([o.delta_layer(o.dense_mlp(64), heads=2, kv_heads=1, dim=64,
                         vdim=64, conv=2)] * 2, width=64, vocab=64),
        M([o.attention_layer(o.moe_mlp(64, 70, 6, 7, 7), heads=34,
                             kv_heads=2, dim=129, vdim=65, size=50),
           o.attention_layer(None, heads=34, kv_heads=2, dim=129, vdim=65,
                             size=16, kv_from=0, softcap=50.0)],
          width=200, vocab=300),
        M([o.attention_layer(o.dense_mlp(33), heads=2, kv_heads=1, dim=260,
                             vdim=12, size=40),
           o.delta_layer(None, heads=2, kv_heads=1, dim=130, vdim=200,
                         conv=4)], width=80, vocab=50),
    ]
    if dtype == torch.bfloat16:  # a layer norm of two numbers is a sign
        configs = configs[1:]
    for i, cfg in enumerate(configs):
        c = Case(tmp, device, dtype, cfg, seed=60 + i, gain=1.0)
        toks = c.tokens(80, 60 + i)
        for cuts in ([80], [41, 1, 2, 34, 1]):
            assert c.error(run_cut(c.engine(), toks, cuts), toks) \
                < TOL[dtype], (i, cuts)


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
    than fit at once, unequal lengths, decoding past chunk edges."""
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
        assert max(gaps) < 3 * TOL[c.dtype] * scale, (len(p), gaps)


def check_long_decode(c: Case, prompt=20, new=200):
    toks = c.tokens(prompt + new, 90)
    got = run_cut(c.engine(), toks, [prompt, 1])
    assert c.error(got, toks) < TOL[c.dtype]


# ---- a far token that has to be remembered ---------------------------------

def check_state_memory(tmp, device, dtype):
    """A delta layer alone that hardly forgets: the logits of the last
    token depend on the first one, through prompts, portions and decoded
    tokens."""
    o = oracle
    cfg = o.make_config([o.delta_layer(None, heads=2, kv_heads=1, dim=16,
                                       vdim=16, conv=3)], width=32, vocab=40)
    c = Case(tmp, device, dtype, cfg, seed=77)
    c.tensors["l0.mix.A_log"] = torch.full((2,), -8.0).to(torch.bfloat16)
    save_file(c.tensors, str(c.path / "model.safetensors"))
    c.model = load_pretrained(c.path, device=device, dtype=dtype)
    toks = [1, 2] + c.tokens(13, 5) * 6
    other = [3] + toks[1:]
    want = c.want(toks)
    tol = TOL[dtype]
    if dtype == torch.float32:
        assert rel(c.want(other)[-20:], want[-20:]) > 20 * tol
    for cuts in ([80], [2], [1], [40, 1], [33, 47]):
        assert c.error(run_cut(c.engine(), toks, cuts), toks) < tol, cuts
