"""Checks of the Kanotar model and engine path, run on the CPU by
test_kanotar.py and on the GPU by test_kanotar_gpu.py.

Every check compares with the plain implementation in kanotar_oracle.py.
Errors are root mean squares over the vocabulary relative to the logits'
own; `TOL` holds what rounding may cause per dtype. Attention is made
peaky (`gain`) where a single wrong key has to show.
"""

import json

import torch
from safetensors.torch import save_file

import kanotar_oracle as oracle
from distllm_amd.engine import LLMEngine, SamplingParams
from distllm_amd.engine.engine import _Seq
from distllm_amd.models import load_pretrained

# (bf16: rounding alone gives a mean of 1e-2 and single rows of 4e-2)
TOL = {torch.float32: 2e-5, torch.bfloat16: 6e-2}


def mixed_layers():
    """Unequal layers: own and shared latents, several windows (the
    sharing layer's is larger than the owner's), one without mlp."""
    L = oracle.make_layer
    return [
        L(heads=3, dim=16, vdim=24, q_rank=20, kv_rank=32, size=8),
        L(heads=2, dim=24, vdim=8, q_rank=36, kv_rank=40, size=21, ff=None),
        L(heads=5, dim=8, vdim=16, q_rank=12, kv_rank=32, size=64,
          kv_from=0, ff=72, limit=0.6),
        L(heads=1, dim=40, vdim=32, q_rank=24, kv_rank=40, size=5,
          kv_from=1),
    ]


class Case:
    def __init__(self, tmp, device, dtype, config=None, seed=0, gain=2.0):
        self.config = config or oracle.make_config(mixed_layers())
        self.tensors = oracle.make_tensors(self.config, seed, gain)
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
        g = torch.Generator().manual_seed(1000 + seed)
        return torch.randint(0, self.config["vocab"], (n,),
                             generator=g).tolist()

    def want(self, toks, config=None):
        key = (tuple(toks), json.dumps(config))
        if key not in self._want:
            self._want[key] = oracle.forward(config or self.config,
                                             self.tensors, toks)
        return self._want[key]


def rel(got, want):
    """Rms difference per row over the rms of all wanted logits: the
    worst row, or three times the mean where that is more."""
    d = got.double().cpu() - want
    d = d - d.mean(-1, keepdim=True)
    scale = (want - want.mean(-1, keepdim=True)).pow(2).mean().sqrt()
    rows = d.pow(2).mean(-1).sqrt() / scale
    # a fault in a few rows shows in the worst, one in many in the mean
    return float(max(rows.max(), 3 * rows.mean()))


def feed(engine, seq, toks):
    """All logits of the next tokens of one sequence, as one step."""
    return engine.step([(seq, list(toks))], [list(range(len(toks)))])


def run_cut(engine, toks, cuts):
    """Logits of a sequence fed in portions of the given sizes; the last
    size repeats."""
    seq, out, at, i = _Seq(0, []), [], 0, 0
    while at < len(toks):
        n = cuts[min(i, len(cuts) - 1)]
        out.append(feed(engine, seq, toks[at: at + n]))
        at += n
        i += 1
    engine.release(seq)
    return torch.cat(out)


def check_whole(c: Case, n=90):
    toks = c.tokens(n, 1)
    got = feed(c.engine(), _Seq(0, []), toks)
    assert rel(got, c.want(toks)) < TOL[c.dtype]


def check_residuals(c: Case, n=40):
    """The residual stream after every layer."""
    from distllm_amd.engine.step import StepBatch
    from distllm_amd.models.layered import LayeredCache

    toks = c.tokens(n, 2)
    want, got = [], []
    oracle.forward(c.config, c.tensors, toks, want)
    cache = LayeredCache(c.model, n // 16 + 2, 16)
    batch = StepBatch.build([(toks, 0, list(range(1, n // 16 + 2)))], 16,
                            c.model.device)
    c.model.forward_step(batch, cache, trace=got)
    assert len(got) == len(want) == len(c.config["layers"])
    assert all(g.dtype == torch.float32 for g in got)
    for g, w in zip(got, want):
        assert rel(g[:n], w) < TOL[c.dtype]


def check_portions(c: Case, n=150):
    """Cut anywhere: single tokens, two tokens, in and across pages,
    windows and the sizes at which the attention form changes."""
    toks = c.tokens(n, 3)
    want = c.want(toks)
    for cuts in ([1], [2], [31, 1], [32, 2, 33], [70, 1], [15, 1, 16, 17],
                 [5, 64, 3, 47, 2], [n - 1, 1]):
        assert rel(run_cut(c.engine(), toks, cuts), want) < TOL[c.dtype], \
            cuts


def check_batches(c: Case):
    """Unequal requests together, each against itself alone: prompt
    portions of several sizes beside single decoded tokens, a request
    that pauses, requests that end and others that take their pages."""
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
    free = len(engine.blockman.free)
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
    assert at == lens and len(engine.blockman.free) == free
    for k in lens:
        assert rel(torch.cat(got[k]), c.want(toks[k])) < TOL[c.dtype], k


def check_reuse(c: Case):
    """Pages that earlier requests filled are used again, in another
    order, without a trace of what they held."""
    engine = c.engine(tokens=112, num_blocks=7)
    for i, n in enumerate((100, 33, 112, 17, 65)):
        toks = c.tokens(n, 30 + i)
        got = run_cut(engine, toks, [n // 2, 1, 2, 40])
        assert rel(got, c.want(toks)) < TOL[c.dtype], n
        engine.blockman.free.reverse()


def check_wanted(c: Case):
    """Only the places asked for, in the order of entries and places."""
    e = c.engine()
    t1, t2 = c.tokens(50, 40), c.tokens(9, 41)
    got = e.step([(_Seq(0, []), t1), (_Seq(1, []), t2)],
                 [[49, 0, 7], [3]])
    want = torch.stack([c.want(t1)[49], c.want(t1)[0], c.want(t1)[7],
                        c.want(t2)[3]])
    assert rel(got, want) < TOL[c.dtype]
    assert e.step([(_Seq(2, []), t2)], [[]]) is None


def edge_case(tmp, device, dtype, size):
    """One peaky layer, so that a key more or less shows at once."""
    cfg = oracle.make_config(
        [oracle.make_layer(heads=4, dim=16, vdim=16, q_rank=24, kv_rank=48,
                           size=size, scale=1.0)], width=64)
    return Case(tmp, device, dtype, cfg, seed=size,
                gain=3.0 if dtype == torch.float32 else 1.0)


def check_edges(c: Case, n):
    """Window edges in prompts, in portions and in decoding. The yardstick
    with a window one off must be far outside the tolerance."""
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
        assert rel(got, want) < TOL[c.dtype], (size, cuts)


def check_sizes(tmp, device, dtype):
    """Sizes of 1, sizes that are no multiple of anything, equal sizes
    that usually differ, all constants away from their usual values."""
    L, M = oracle.make_layer, oracle.make_config
    configs = [
        M([L(heads=1, dim=1, vdim=1, q_rank=1, kv_rank=1, size=1, ff=1)],
          width=1, vocab=3),
        M([L(heads=7, dim=9, vdim=11, q_rank=13, kv_rank=17, size=19,
             ff=23, limit=0.2, scale=0.05)] * 2,
          width=29, vocab=31, eps=0.3, logit_scale=3.5),
        M([L(heads=2, dim=70, vdim=130, q_rank=66, kv_rank=129, size=1000,
             ff=None)] * 3, width=130, vocab=64, logit_scale=1.0),
        M([L(heads=17, dim=64, vdim=64, q_rank=64, kv_rank=64, size=64,
             ff=64, scale=0.125)], width=64, vocab=64),
        M([L(heads=33, dim=129, vdim=65, q_rank=96, kv_rank=300, size=50),
           L(heads=70, dim=12, vdim=20, q_rank=96, kv_rank=300, size=45,
             kv_from=0)], width=200, vocab=300),
        M([L(heads=2, dim=260, vdim=12, q_rank=16, kv_rank=513, size=40)],
          width=80, vocab=50),
    ]
    for i, cfg in enumerate(configs):
        c = Case(tmp, device, dtype, cfg, seed=60 + i, gain=1.0)
        toks = c.tokens(80, 60 + i)
        want = c.want(toks)
        for cuts in ([80], [41, 1, 2, 34, 1]):
            assert rel(run_cut(c.engine(), toks, cuts), want) \
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
    than fit at once, unequal lengths, long decoding past every window."""
    prompts = [c.tokens(n, 70 + n) for n in (5, 61, 1, 33, 90)]
    params = SamplingParams(temperature=0.0, min_p=0.0, max_tokens=24)
    engine = c.engine(tokens=160, num_blocks=24, max_batch_size=3)
    engine.STEP_TOKENS = 40  # prompts take several steps
    free = len(engine.blockman.free)
    if use_loop:
        from distllm_amd.engine.loop import EngineLoop

        loop = EngineLoop(engine, params)
        try:
            outs = loop.generate(prompts, 24)
        finally:
            loop.close()
    else:
        outs = engine.generate(prompts, params)
    assert len(engine.blockman.free) == free
    for p, o in zip(prompts, outs):
        assert len(o) == 24
        gaps, scale = oracle_greedy(c, p, o)
        assert max(gaps) < 3 * TOL[c.dtype] * scale, (len(p), gaps)


def check_long_decode(c: Case, prompt=20, new=200):
    toks = c.tokens(prompt + new, 90)
    got = run_cut(c.engine(), toks, [prompt, 1])
    assert rel(got, c.want(toks)) < TOL[c.dtype]
