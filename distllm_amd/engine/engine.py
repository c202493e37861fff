"""Native generation engine: paged KV cache + continuous batching +
fused HIP sampling. Replaces the reference's vLLM dependency
(reference generate/generators/vllm_backend.py).

Architecture (MI355X-first):
  - a paged cache sized for the 288 GB HBM budget, in the model's own
    layout (per-layer K/V pages, or pages of latents), and state slots,
    one per running sequence, for models with recurrent layers;
  - prefill: batched padded forward through the flash-attention prefill
    kernel, K/V scattered into the paged cache; models that run ragged
    step batches (engine/step.py) take prompts in portions instead, in
    the same step as the decoded tokens of other sequences;
  - decode: one fused paged-attention kernel call per layer for the
    whole running batch (batch grows/shrinks every step =
    token-granularity continuous batching);
  - sampling: fused temperature+min-p kernel (top-p via torch sort path
    when requested).
"""

from __future__ import annotations

import gc
import math
from dataclasses import dataclass, field

import torch

from .. import ops
from ..models.mistral import DecoderModel
from .step import StepBatch


@dataclass
class SamplingParams:
    """Defaults follow the reference's vLLM call
    (vllm_backend.py:46-60): temperature .5, min_p .1, max_tokens 2000."""

    temperature: float = 0.5
    min_p: float = 0.1
    top_p: float = 1.0
    max_tokens: int = 2000
    stop_token_ids: tuple[int, ...] = ()


@dataclass
class _Seq:
    seq_id: int
    prompt_ids: list[int]
    out_ids: list[int] = field(default_factory=list)
    blocks: list[int] = field(default_factory=list)
    done: bool = False
    # per-sequence token budget; None -> the batch SamplingParams cap
    max_tokens: int | None = None
    cached: int = 0  # leading tokens whose cache entries are written
    slot: int | None = None  # recurrent state, where the model has one

    @property
    def length(self) -> int:
        return len(self.prompt_ids) + len(self.out_ids)

    def pending(self, n: int | None = None) -> list[int]:
        """The next n (default: all) tokens that are not cached yet."""
        end = self.length if n is None else self.cached + n
        p = len(self.prompt_ids)
        if self.cached >= p:
            return self.out_ids[self.cached - p: end - p]
        return (self.prompt_ids[self.cached: end]
                + self.out_ids[: max(0, end - p)])


class BlockManager:
    """Fixed-pool paged KV block allocator (BLK tokens per block).
    Block 0 is reserved as the dummy target for padded graph slots."""

    def __init__(self, num_blocks: int, blk: int = 16):
        self.blk = blk
        self.free: list[int] = list(range(1, num_blocks))

    def can_alloc(self, n: int) -> bool:
        return len(self.free) >= n

    def alloc(self, n: int) -> list[int]:
        if n > len(self.free):
            raise RuntimeError("KV blocks exhausted")
        out = self.free[:n]
        del self.free[:n]
        return out

    def release(self, blocks: list[int]) -> None:
        self.free.extend(blocks)

    def blocks_for(self, n_tokens: int) -> int:
        return (n_tokens + self.blk - 1) // self.blk


class SlotManager:
    """State slots of the running sequences. Slot 0 is reserved as the
    target of padded graph rows."""

    def __init__(self, num_slots: int):
        self.free: list[int] = list(range(1, num_slots))

    def alloc(self) -> int:
        if not self.free:
            raise RuntimeError("state slots exhausted")
        return self.free.pop(0)

    def release(self, slot: int) -> None:
        self.free.append(slot)


class LLMEngine:
    BLK = 16
    # prompt tokens that a ragged step takes on at most
    STEP_TOKENS = 16384

    def __init__(self, model: DecoderModel, max_batch_size: int = 64,
                 max_model_len: int = 4096,
                 kv_memory_fraction: float = 0.6,
                 num_blocks: int | None = None,
                 use_graphs: bool | None = None,
                 kv_cache_dtype: str = "bf16",
                 weight_dtype: str = "bf16"):
        self.model = model
        d = model.dims
        # optional W8A16 decode weights (OCP fp8-e4m3, per-channel
        # scales): the B<=8 decode step is weight-stream bound, so fp8
        # halves its HBM bytes (models/mistral.py enable_fp8_decode;
        # prefill and larger batches keep bf16)
        if weight_dtype not in ("bf16", "fp8_e4m3"):
            raise ValueError(f"weight_dtype {weight_dtype!r}")
        self.weight_dtype = weight_dtype
        if weight_dtype == "fp8_e4m3":
            if not str(model.device).startswith("cuda"):
                raise ValueError("fp8_e4m3 weights require a GPU")
            if not hasattr(model, "enable_fp8_decode"):
                raise ValueError(f"{type(model).__name__} has no "
                                 "fp8_e4m3 weight path")
            model.enable_fp8_decode()
        self.device = model.device
        self.max_batch_size = max_batch_size
        self.max_model_len = min(max_model_len, d.max_position_embeddings)
        dev = self.device
        # optional OCP fp8-e4m3 KV cache (CDNA4-native): halves KV
        # bandwidth/footprint; off by default (bf16 = reference dtype)
        if kv_cache_dtype not in ("bf16", "fp8_e4m3"):
            raise ValueError(f"kv_cache_dtype {kv_cache_dtype!r}")
        self.kv_cache_dtype = kv_cache_dtype
        # recurrent state: a slot per running sequence and the reserved one
        slot_bytes = model.state_bytes_per_slot()
        self.slotman = (SlotManager(max_batch_size + 1) if slot_bytes
                        else None)
        num_slots = max_batch_size + 1 if slot_bytes else 0
        if num_blocks is None:
            if str(dev).startswith("cuda"):
                free, _total = torch.cuda.mem_get_info(dev)
                budget = int(free * kv_memory_fraction)
            else:
                budget = 64 << 20  # CPU tests: 64 MiB
            budget = max(budget - num_slots * slot_bytes, 0)
            per_block = model.cache_bytes_per_block(self.BLK, kv_cache_dtype)
            num_blocks = max(budget // max(per_block, 1), 16)
            # cap: enough for max_batch_size * max_model_len
            need = (self.max_model_len // self.BLK + 1) * max_batch_size
            num_blocks = min(num_blocks, need)
        num_blocks += 1  # block 0 is reserved (graph-padding dummy)
        self.num_blocks = num_blocks
        if kv_cache_dtype == "fp8_e4m3" and not str(dev).startswith("cuda"):
            raise ValueError("fp8_e4m3 KV cache requires a GPU")
        self.cache = model.make_cache(num_blocks, self.BLK, kv_cache_dtype,
                                      num_slots)
        self.ragged = model.ragged
        self.blockman = BlockManager(num_blocks, self.BLK)
        self._next_id = 0
        # hipGraph-captured decode (one graph per pow2 batch bucket):
        # the decode step is ~300 small launches per step for a 32-layer
        # model — graph replay removes the launch overhead. ROCm 7
        # supports RCCL collectives inside graph capture, so tp>1
        # captures the per-layer all-reduces too; if
        # capture fails on a given stack, _graph_for falls back to
        # eager decode with a warning.
        self.use_graphs = (use_graphs if use_graphs is not None
                           else str(dev).startswith("cuda"))
        # deterministic sampling RNG shared across TP ranks
        self._rng = torch.Generator(device=dev)
        self._rng.manual_seed(0x5EED)
        self.max_blocks_per_seq = (self.max_model_len // self.BLK) + 1
        self._graphs: dict[int, "_GraphRunner"] = {}

    @property
    def kcaches(self):
        return self.cache.k

    @property
    def vcaches(self):
        return self.cache.v

    # ---- public --------------------------------------------------------
    @torch.no_grad()
    def generate(self, prompts_ids: list[list[int]],
                 params: SamplingParams) -> list[list[int]]:
        """Generate completions for all prompts (continuous batching);
        returns generated token ids per prompt (prompt excluded)."""
        dev = self.device
        waiting = [
            _Seq(seq_id=i,
                 prompt_ids=list(p[-(self.max_model_len - 1):]))
            for i, p in enumerate(prompts_ids)
        ]
        results: dict[int, list[int]] = {}
        running: list[_Seq] = []

        while waiting or running:
            # admit as many waiting seqs as fit (batch + blocks)
            admitted: list[_Seq] = []
            while waiting and len(running) + len(admitted) < \
                    self.max_batch_size:
                s = waiting[0]
                need = self.blockman.blocks_for(
                    min(s.length + params.max_tokens, self.max_model_len)
                )
                if not self.blockman.can_alloc(need):
                    break
                s.blocks = self.blockman.alloc(need)
                admitted.append(waiting.pop(0))
            if admitted:
                self._start(admitted, params, results)
                running.extend(s for s in admitted if not s.done)
            if not running:
                if admitted or not waiting:
                    if not waiting:
                        break
                    continue
                raise RuntimeError(
                    "cannot admit any sequence: KV pool too small"
                )
            # one step for the whole running batch
            self._advance(running, params, results)
            running = [s for s in running if not s.done]

        return [results.get(i, []) for i in range(len(prompts_ids))]

    def _start(self, seqs: list[_Seq], params: SamplingParams,
               results: dict[int, list[int]]) -> None:
        """Take up admitted sequences. Ragged models need nothing here:
        the following steps bring the prompts in."""
        if not self.ragged:
            self._run_prefill(seqs, params, results)

    def _advance(self, seqs: list[_Seq], params: SamplingParams,
                 results: dict[int, list[int]]) -> None:
        """One step of the running batch: every sequence that has been
        sampled decodes its token; prompts advance by what is left of
        the step's token budget."""
        if not self.ragged or all(s.length - s.cached == 1 and s.cached
                                  for s in seqs):
            self._run_decode(seqs, params, results)
            return
        budget = self.STEP_TOKENS
        work, ready = [], []
        for s in sorted(seqs, key=lambda s: s.length - s.cached > 1):
            left = s.length - s.cached
            if left == 0:
                raise ValueError("a sequence needs at least one token")
            n = min(left, budget)
            if n == 0:
                continue
            budget -= n
            work.append((s, s.pending(n)))
            if n == left:
                ready.append((s, len(work) - 1, n - 1))
        want: list[list[int]] = [[] for _ in work]
        for _, w, last in ready:
            want[w] = [last]
        logits = self.step(work, want)
        if ready:
            self._sample_and_append([s for s, _, _ in ready], logits,
                                    params, results)

    @torch.no_grad()
    def step(self, work: list[tuple[_Seq, list[int]]],
             want: list[list[int]]) -> torch.Tensor | None:
        """Run one ragged step: for each (sequence, its next tokens).
        Returns the f32 logits [wanted, vocab] at the places `want` names
        among each entry's tokens, in entry order; None if there are
        none. Cache blocks are allotted as sequences grow."""
        if not self.ragged:
            raise RuntimeError("this model does not run ragged steps")
        self._grow(work)
        if (all(len(t) == 1 and s.cached for s, t in work)
                and len(work) <= self.max_batch_size):
            tokens = torch.tensor([t[0] for _, t in work],
                                  device=self.device)
            ctx = torch.tensor([s.cached + 1 for s, _ in work],
                               dtype=torch.int32, device=self.device)
            logits = self._decode_logits([s for s, _ in work], tokens, ctx)
            pick = [i for i, w in enumerate(want) for _ in w]
            out = None
            if pick:
                # a copy: the next replay overwrites the graph's output
                out = logits[torch.tensor(pick, device=self.device)]
        else:
            batch = StepBatch.build(
                [(t, s.cached, s.blocks) for s, t in work], self.BLK,
                self.device, self.model.expand_min,
                self._slots([s for s, _ in work]))
            hidden = self.model.forward_step(batch, self.cache)
            pick = [int(batch.rows[i][k]) for i, w in enumerate(want)
                    for k in w]
            out = None
            if pick:
                rows = torch.tensor(pick, device=self.device)
                out = self.model.logits(hidden[rows])
        for s, t in work:
            s.cached += len(t)
        return out

    def _grow(self, work) -> None:
        need = []
        for s, t in work:
            end = s.cached + len(t)
            if end > self.max_model_len:
                raise RuntimeError(
                    f"sequence {s.seq_id} exceeds max_model_len "
                    f"{self.max_model_len}")
            need.append(max(0, self.blockman.blocks_for(end)
                            - len(s.blocks)))
        if not self.blockman.can_alloc(sum(need)):
            raise RuntimeError("KV blocks exhausted")
        if self.slotman is not None:
            new = [s for s, _ in work if s.slot is None]
            if len(new) > len(self.slotman.free):
                raise RuntimeError("state slots exhausted")
            for s in new:
                s.slot = self.slotman.alloc()
        for (s, _), n in zip(work, need):
            if n:
                s.blocks = s.blocks + self.blockman.alloc(n)

    def _slots(self, seqs: list[_Seq]) -> list[int] | None:
        if self.slotman is None:
            return None
        return [s.slot for s in seqs]

    def release(self, s: _Seq) -> None:
        """Give back everything a finished sequence holds."""
        self.blockman.release(s.blocks)
        if s.slot is not None:
            self.slotman.release(s.slot)
            s.slot = None
        s.blocks = []
        s.cached = 0

    def _block_table(self, seqs: list[_Seq],
                     width: int | None = None) -> torch.Tensor:
        # build on the host, upload in ONE copy (a per-row device
        # tensor-from-list costs one tiny H2D copy per sequence/step)
        maxb = width or max(len(s.blocks) for s in seqs)
        bt = torch.zeros(len(seqs), maxb, dtype=torch.int32)
        for i, s in enumerate(seqs):
            bt[i, : len(s.blocks)] = torch.tensor(s.blocks,
                                                  dtype=torch.int32)
        return bt.to(self.device, non_blocking=True)

    @torch.no_grad()
    def _run_prefill(self, seqs: list[_Seq], params: SamplingParams,
                     results: dict[int, list[int]]) -> None:
        if self.ragged:
            todo = list(seqs)
            while todo:
                self._advance(todo, params, results)
                todo = [s for s in todo if not s.out_ids]
            return
        dev = self.device
        B = len(seqs)
        maxlen = max(s.length for s in seqs)
        ids = torch.zeros(B, maxlen, dtype=torch.long, device=dev)
        mask = torch.zeros(B, maxlen, dtype=torch.int32, device=dev)
        for i, s in enumerate(seqs):
            ids[i, : s.length] = torch.tensor(s.prompt_ids, device=dev)
            mask[i, : s.length] = 1
        kv: list = []
        hidden = self.model.forward(ids, mask, kv_out=kv)
        # scatter prefill K/V into the paged caches
        bt = self._block_table(seqs)
        lens = torch.tensor([s.length for s in seqs], device=dev)
        pos = torch.arange(maxlen, device=dev)[None, :].expand(B, -1)
        valid = pos < lens[:, None]                       # [B, maxlen]
        blk_idx = bt.long().gather(
            1, (pos // self.BLK).clamp(max=bt.shape[1] - 1)
        )                                                  # [B, maxlen]
        slot = pos % self.BLK
        bsel, tsel = valid.nonzero(as_tuple=True)
        flat_blk = blk_idx[bsel, tsel]
        flat_slot = slot[bsel, tsel]
        fp8 = self.kv_cache_dtype == "fp8_e4m3"
        for li, (k, v) in enumerate(kv):
            # k/v: [B, maxlen, HKV, D]
            ksel, vsel = k[bsel, tsel], v[bsel, tsel]
            if fp8:  # OCP e4m3fn bit pattern == the kernel's fp8 type
                ksel = ksel.to(torch.float8_e4m3fn).view(torch.uint8)
                vsel = vsel.to(torch.float8_e4m3fn).view(torch.uint8)
            self.kcaches[li][flat_blk, :, flat_slot] = ksel
            self.vcaches[li][flat_blk, :, flat_slot] = vsel
        for s in seqs:
            s.cached = s.length
        # last-token logits -> first sampled token
        last = (lens - 1).long()
        hlast = hidden[torch.arange(B, device=dev), last]
        logits = self.model.logits(hlast)
        self._sample_and_append(seqs, logits, params, results)

    @torch.no_grad()
    def _graph_for_or_eager(self, n: int):
        """Graph for the bucket, or None after a failed capture (e.g. a
        ROCm stack without RCCL-in-graph support for tp>1)."""
        try:
            return self._graph_for(n)
        except RuntimeError as e:
            import warnings

            warnings.warn(
                f"[engine] hipGraph decode capture failed ({e}); "
                "falling back to eager decode", RuntimeWarning)
            self.use_graphs = False
            self._graphs.clear()
            return None

    def _graph_for(self, n: int) -> "_GraphRunner":
        bucket = 1
        while bucket < n:
            bucket <<= 1
        bucket = min(max(bucket, n), max(self.max_batch_size, n))
        if bucket not in self._graphs:
            self._graphs[bucket] = _GraphRunner(self, bucket)
        return self._graphs[bucket]

    def _run_decode(self, seqs: list[_Seq], params: SamplingParams,
                    results: dict[int, list[int]]) -> None:
        dev = self.device
        # (a prompt that a step's budget cut one short has no output yet)
        tokens = torch.tensor([(s.out_ids or s.prompt_ids)[-1]
                               for s in seqs], device=dev)
        ctx = torch.tensor([s.length for s in seqs], dtype=torch.int32,
                           device=dev)
        logits = self._decode_logits(seqs, tokens, ctx)
        for s in seqs:
            s.cached = s.length
        self._sample_and_append(seqs, logits, params, results)

    def _decode_logits(self, seqs: list[_Seq], tokens: torch.Tensor,
                       ctx: torch.Tensor) -> torch.Tensor:
        """Logits of one token per sequence, from the captured graph of
        the batch bucket where graphs are in use."""
        runner = None
        if self.use_graphs:
            runner = self._graph_for_or_eager(len(seqs))
        state = ()
        if self.slotman is not None:
            state = (torch.tensor(self._slots(seqs), dtype=torch.int32,
                                  device=self.device),)
        if runner is not None:
            bt = self._block_table(seqs, width=self.max_blocks_per_seq)
            return runner.run(tokens, bt, ctx, *state)[: len(seqs)]
        return self.model.decode_step(tokens, self.cache,
                                      self._block_table(seqs), ctx, *state)

    def _sample_and_append(self, seqs, logits, params, results):
        dev = self.device
        if params.top_p < 1.0:
            next_ids = self._sample_top_p(logits, params)
        elif len(seqs) <= 16 and params.temperature > 0 \
                and str(dev).startswith("cuda"):
            next_ids = self._gumbel_sample(logits, params, self._rng)
        else:
            rand = torch.rand(len(seqs), device=dev,
                              generator=self._rng)
            next_ids = ops.sample_tokens(logits, rand, params.temperature,
                                         params.min_p)
        next_list = next_ids.tolist()
        for s, tok in zip(seqs, next_list):
            s.out_ids.append(int(tok))
            stop = (
                tok in params.stop_token_ids
                or len(s.out_ids) >= (s.max_tokens or params.max_tokens)
                or s.length >= self.max_model_len
            )
            if stop:
                s.done = True
                out = s.out_ids
                if tok in params.stop_token_ids:
                    out = out[:-1]
                results[s.seq_id] = out
                self.release(s)

    def warm_graphs(self, batch_sizes: list[int] | None = None) -> None:
        """Pre-capture decode graphs for the given batch buckets."""
        if not self.use_graphs:
            return
        for b in batch_sizes or [self.max_batch_size]:
            if self._graph_for_or_eager(b) is None:
                return

    @staticmethod
    def _gumbel_sample(logits: torch.Tensor, params: SamplingParams,
                       rng: torch.Generator) -> torch.Tensor:
        """Small-batch Gumbel-max draw: the CDF-walk kernel is one
        block per row (latency-bound, ~170us at B=1 over a 128k
        vocab); argmax over logits/T + Gumbel noise is exact for
        categorical sampling and fully parallel. Seeded engine RNG
        keeps TP ranks identical."""
        lf = logits.float() / max(params.temperature, 1e-5)
        if params.min_p > 0:
            floor = (lf.max(dim=-1, keepdim=True).values
                     + math.log(params.min_p))
            lf = lf.masked_fill(lf < floor, float("-inf"))
        u = torch.rand(lf.shape, device=lf.device, generator=rng)
        gumbel = -torch.log((-torch.log(u.clamp_min(1e-20)))
                            .clamp_min(1e-20))
        return (lf + gumbel).argmax(dim=-1).int()

    def _sample_top_p(self, logits: torch.Tensor,
                      params: SamplingParams) -> torch.Tensor:
        t = max(params.temperature, 1e-5)
        probs = torch.softmax(logits.float() / t, dim=-1)
        if params.min_p > 0.0:
            floor = params.min_p * probs.max(dim=-1, keepdim=True).values
            probs = probs.masked_fill(probs < floor, 0.0)
        sorted_p, sorted_i = probs.sort(dim=-1, descending=True)
        cum = sorted_p.cumsum(-1)
        cut = cum - sorted_p > params.top_p
        sorted_p = sorted_p.masked_fill(cut, 0.0)
        sorted_p = sorted_p / sorted_p.sum(-1, keepdim=True)
        # seeded engine RNG: keeps sampling identical across TP ranks
        choice = torch.multinomial(sorted_p, 1, generator=self._rng)
        return sorted_i.gather(1, choice).squeeze(1).int()


class _GraphRunner:
    """One hipGraph-captured decode step at a fixed batch size.

    Static input/output tensors; padded rows point at the reserved
    dummy KV block 0 (and state slot 0) with ctx_len=1, so their cache
    writes and reads are harmless. Capture follows the torch.cuda.graph protocol (side-stream
    warmup, then capture); replay removes the ~10 launches/layer CPU
    overhead that dominates small-batch decode.
    """

    def __del__(self):
        # Drain the device before torch destroys the captured hipGraph:
        # GC can collect a dead engine's graphs from any thread at any
        # time, and hipGraphExecDestroy racing in-flight kernels was
        # the best candidate for intermittent full-test-suite aborts.
        try:
            import torch as _t

            if _t.cuda.is_available():
                _t.cuda.synchronize()
        except Exception:
            pass

    def __init__(self, engine: LLMEngine, batch: int):
        dev = engine.device
        # no reference to the engine is kept: the pair would be a cycle,
        # freed only by a garbage collection at some arbitrary moment
        self.batch = batch
        self.tokens = torch.zeros(batch, dtype=torch.long, device=dev)
        self.bt = torch.zeros(batch, engine.max_blocks_per_seq,
                              dtype=torch.int32, device=dev)
        self.ctx = torch.ones(batch, dtype=torch.int32, device=dev)
        self.state = ()
        if engine.slotman is not None:
            self.state = (torch.zeros(batch, dtype=torch.int32, device=dev),)
        torch.cuda.synchronize()
        side = torch.cuda.Stream()
        side.wait_stream(torch.cuda.current_stream())
        with torch.cuda.stream(side):
            for _ in range(2):  # warmup allocations/paths
                engine.model.decode_step(self.tokens, engine.cache,
                                         self.bt, self.ctx, *self.state)
        torch.cuda.current_stream().wait_stream(side)
        torch.cuda.synchronize()
        self.graph = torch.cuda.CUDAGraph()
        # A collection during capture may destroy graphs of a dead engine
        # or synchronize (see __del__); neither is allowed while a stream
        # is capturing, and the failed destructor ends the process.
        gc.collect()
        enabled = gc.isenabled()
        gc.disable()
        try:
            with torch.cuda.graph(self.graph):
                self.logits = engine.model.decode_step(
                    self.tokens, engine.cache, self.bt, self.ctx,
                    *self.state)
        finally:
            if enabled:
                gc.enable()

    def run(self, tokens: torch.Tensor, bt: torch.Tensor,
            ctx: torch.Tensor, *state: torch.Tensor) -> torch.Tensor:
        n = tokens.shape[0]
        self.tokens[:n] = tokens
        if n < self.batch:
            self.tokens[n:] = 0
        self.bt[:n] = bt
        if n < self.batch:
            self.bt[n:] = 0
        self.ctx[:n] = ctx
        if n < self.batch:
            self.ctx[n:] = 1
        for own, new in zip(self.state, state):
            own[:n] = new
            own[n:] = 0
        self.graph.replay()
        return self.logits
