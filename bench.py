"""Flagship benchmark: PubMedBERT bs512 embedding throughput (seqs/sec).

Driver contract: `python bench.py --gpus N --steps K --warmup W`.
For N>1 the driver launches this under torch.distributed.run with one
rank per GPU (RCCL over xGMI). One timed step = embed one batch of
`--batch-size` synthetic sequences of length `--seq-len` through the
native HIP-kernel encoder forward + fused mean-pool + L2 normalize +
async D2H into a pinned host buffer — the hot loop of the reference's
headline config (examples/embed/AMP.nougat.pubmedbert.yaml:
batch_size=512, maxlen 512, mean pool).

Rank 0 prints ONE JSON line with the whole-job aggregate.
"""

from __future__ import annotations

import argparse
import json
import os
import time

import torch

# Synthetic benchmark: the hash tokenizer is the sanctioned stand-in.
os.environ.setdefault("DISTLLM_ALLOW_HASH_TOKENIZER", "1")


def main() -> None:
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=30)
    ap.add_argument("--warmup", type=int, default=5)
    ap.add_argument("--batch-size", type=int, default=512)
    ap.add_argument("--seq-len", type=int, default=512)
    ap.add_argument("--model", type=str, default="pubmedbert-base")
    ap.add_argument("--mode", type=str, default="embed",
                    choices=["embed", "generate", "pipeline", "decoders"],
                    help="embed = flagship seqs/s; generate = decode "
                         "tokens/s (Llama-class, paged KV); pipeline = "
                         "full jsonl_chunk -> semantic_chunk embed -> "
                         "write (tokenizer + staging included); "
                         "decoders = prefill and decode of Kanotar "
                         "and Bufulorn layers beside llama layers of equal "
                         "size, and of Tebasun and Kedelorn beside "
                         "layers of the closest of these")
    ap.add_argument("--docs-per-file", type=int, default=128)
    ap.add_argument("--pooler", type=str, default="mean",
                    choices=["mean", "last_token"])
    ap.add_argument("--prompt-len", type=int, default=128)
    ap.add_argument("--weight-dtype", type=str, default="bf16",
                    choices=["bf16", "fp8_e4m3"],
                    help="generate mode: W8A16 fp8 decode weights")
    ap.add_argument("--layers", type=int, default=8,
                    help="decoders mode: layers per model")
    ap.add_argument("--only", type=str, default="",
                    help="decoders mode: sizes to run, with commas")
    args = ap.parse_args()

    if args.mode == "decoders":
        bench_decoders(args)
        return
    if args.mode == "generate":
        bench_generate(args)
        return
    if args.mode == "pipeline":
        bench_pipeline(args)
        return

    from distllm_amd.models import build_model
    from distllm_amd.parallel import (barrier, get_rank, get_world_size,
                                      init_distributed)
    from distllm_amd import ops

    rank, world = init_distributed()
    have_gpu = torch.cuda.is_available()
    if have_gpu:
        local_rank = int(os.environ.get("LOCAL_RANK", "0"))
        torch.cuda.set_device(local_rank)
        device = f"cuda:{local_rank}"
        dtype = torch.bfloat16
    else:
        device, dtype = "cpu", torch.float32

    torch.manual_seed(1234 + rank)
    model = build_model(args.model, device=device, dtype=dtype)
    dims = model.dims

    B, S = args.batch_size, args.seq_len
    ids = torch.randint(4, dims.vocab_size, (B, S), device=device)
    mask = torch.ones(B, S, device=device, dtype=torch.int32)
    host = torch.empty(B, dims.hidden_size, dtype=torch.float32,
                       pin_memory=have_gpu)
    # pinned-host staged inputs: each step re-uploads (H2D in the loop,
    # like the real dataloader path)
    ids_host = ids.to("cpu").pin_memory() if have_gpu else ids
    mask_host = mask.to("cpu").pin_memory() if have_gpu else mask

    @torch.no_grad()
    def step() -> None:
        d_ids = ids_host.to(device, non_blocking=True)
        d_mask = mask_host.to(device, non_blocking=True)
        hidden = model(d_ids, d_mask)
        if args.pooler == "last_token":
            pooled = ops.last_token_pool(hidden, d_mask, normalize=True)
        else:
            pooled = ops.mean_pool(hidden, d_mask, normalize=True)
        host.copy_(pooled, non_blocking=True)

    for _ in range(args.warmup):
        step()
    barrier()
    if have_gpu:
        torch.cuda.synchronize()
    t0 = time.perf_counter()
    for _ in range(args.steps):
        step()
    if have_gpu:
        torch.cuda.synchronize()
    barrier()
    elapsed = time.perf_counter() - t0

    # MAX elapsed over ranks -> whole-job throughput
    if world > 1:
        import torch.distributed as dist

        t = torch.tensor([elapsed], dtype=torch.float64,
                         device=device if have_gpu else "cpu")
        dist.all_reduce(t, op=dist.ReduceOp.MAX)
        elapsed = float(t.item())

    ms_per_step = elapsed / args.steps * 1000.0
    value = world * B * args.steps / elapsed

    metric = ("seqs/sec embedded (PubMedBERT bs512)"
              if args.model == "pubmedbert-base"
              else f"seqs/sec embedded ({args.model} bs{B})")
    if rank == 0:
        print(json.dumps({
            "metric": metric,
            "value": round(value, 2),
            "unit": "seqs/s",
            "n_gpus": world,
            "steps": args.steps,
            "warmup": args.warmup,
            "ms_per_step": round(ms_per_step, 3),
            "higher_is_better": True,
            "scaling": "weak",
            "vs_baseline": None,
            "dtype": "bf16" if have_gpu else "fp32",
            "data": "synthetic",
            "config": {
                "model": args.model,
                "global_batch": world * B,
                "seq_len": S,
                "parallelism": f"dp{world}",
            },
        }))


def bench_generate(args) -> None:
    """Decode throughput: one step = one continuous-batching decode step
    for the whole batch (paged-KV attention + sampling)."""
    import torch

    from distllm_amd import ops
    from distllm_amd.engine import LLMEngine, SamplingParams
    from distllm_amd.models import build_model
    from distllm_amd.parallel import barrier, init_distributed

    rank, world = init_distributed()
    have_gpu = torch.cuda.is_available()
    if have_gpu:
        local_rank = int(os.environ.get("LOCAL_RANK", "0"))
        torch.cuda.set_device(local_rank)
        device, dtype = f"cuda:{local_rank}", torch.bfloat16
    else:
        device, dtype = "cpu", torch.float32

    model_name = args.model if args.model != "pubmedbert-base" \
        else "llama3-8b"
    torch.manual_seed(99 + rank)
    model = build_model(model_name, device=device, dtype=dtype)
    B, P = args.batch_size, args.prompt_len
    engine = LLMEngine(model, max_batch_size=B,
                       max_model_len=P + args.steps + args.warmup + 8,
                       weight_dtype=args.weight_dtype)
    params = SamplingParams(temperature=0.5, min_p=0.1,
                            max_tokens=args.steps + args.warmup + 4,
                            stop_token_ids=())

    # set up B running sequences via one prefill
    prompts = torch.randint(4, model.dims.vocab_size, (B, P)).tolist()
    from distllm_amd.engine.engine import _Seq

    seqs = [_Seq(seq_id=i, prompt_ids=p) for i, p in enumerate(prompts)]
    for s in seqs:
        s.blocks = engine.blockman.alloc(
            engine.blockman.blocks_for(P + params.max_tokens + 1))
    results: dict = {}
    engine._run_prefill(seqs, params, results)

    def step():
        engine._run_decode(seqs, params, results)

    for _ in range(args.warmup):
        step()
    barrier()
    if have_gpu:
        torch.cuda.synchronize()
    t0 = time.perf_counter()
    for _ in range(args.steps):
        step()
    if have_gpu:
        torch.cuda.synchronize()
    barrier()
    elapsed = time.perf_counter() - t0
    if world > 1:
        import torch.distributed as dist

        t = torch.tensor([elapsed], dtype=torch.float64,
                         device=device if have_gpu else "cpu")
        dist.all_reduce(t, op=dist.ReduceOp.MAX)
        elapsed = float(t.item())
    value = world * B * args.steps / elapsed
    if rank == 0:
        print(json.dumps({
            "metric": f"generate tokens/sec ({model_name} decode)",
            "value": round(value, 2),
            "unit": "tokens/s",
            "n_gpus": world,
            "steps": args.steps,
            "warmup": args.warmup,
            "ms_per_step": round(elapsed / args.steps * 1000.0, 3),
            "higher_is_better": True,
            "scaling": "weak",
            "vs_baseline": None,
            "dtype": ("bf16" if args.weight_dtype == "bf16"
                      else "bf16+fp8w") if have_gpu else "fp32",
            "data": "synthetic",
            "config": {
                "model": model_name,
                "global_batch": world * B,
                "seq_len": P,
                "parallelism": f"dp{world}",
            },
        }))


def bench_decoders(args) -> None:
    """Kanotar and Bufulorn layers beside llama layers of the same width,
    heads and (active) feed-forward weights, Tebasun layers beside Bufulorn
    layers, and Kedelorn layers beside Bufulorn and Kanotar layers, through
    the same engine: tokens/s of prefilling a batch of prompts and of
    decoding at a given context, both models in turn.
    Random weights, synthetic tokens, one GPU."""
    from distllm_amd.engine import LLMEngine, SamplingParams
    from distllm_amd.engine.engine import _Seq
    from distllm_amd.models import ModelDims, build_model
    from distllm_amd.models.config import (ExpertsDims, GatedExpertsDims,
                                           hybrid_preset, layered_preset,
                                           looped_preset, streamed_preset)

    dev = "cuda:0"
    torch.manual_seed(5)
    V = 32768

    def llama(hidden, heads, kv, ff):
        return ModelDims(arch="llama", vocab_size=V, hidden_size=hidden,
                         num_layers=args.layers, num_heads=heads,
                         num_kv_heads=kv, intermediate_size=ff,
                         max_position_embeddings=16384)

    def kanotar(hidden, heads, q_rank, kv_rank, ff, window, share=None):
        return layered_preset(args.layers, hidden, V, heads, 128, 128,
                              q_rank, kv_rank, ff, [window], share)

    def bufulorn(hidden, heads, kv, ff, chunk, order="A", **kw):
        # two matrices per dense feed-forward where llama has three
        routed = kw.pop("routed", False)
        d = hybrid_preset(args.layers, hidden, V, heads, kv, 128,
                          max(ff * 3 // 2, 1), chunk, order=order, **kw)
        for layer in d.layers if routed else ():
            layer.mlp = kw["experts"]
        return d

    def tebasun(hidden, heads, kv, ff, order, **kw):
        # half of the heads in each of two mixers side by side
        return looped_preset(kw.pop("layers", args.layers), hidden, V, heads,
                             kv, 128, ff, order, **kw)

    def kedelorn(hidden, heads, kv_rank, order, mlp=None, **kw):
        return streamed_preset(args.layers, hidden, V, heads, 128, kv_rank,
                               mlp, order, **kw)

    def mixers(dims):
        for layer in dims.layers:
            layer.mlp = None
        return dims

    # name: (model, the other one, [(prompts, prompt len)],
    #        [(batch, context)])
    some = [(16, 2048)], [(1, 2048), (32, 2048), (128, 2048)]
    sizes = {
        "4096x32h full": (
            kanotar(4096, 32, 1536, 512, 14336, 8192),
            llama(4096, 32, 8, 14336),
            [(16, 2048), (2, 8000)], [(1, 2048), (32, 2048), (128, 2048),
                                      (32, 8000)]),
        "4096x32h window 1024": (
            kanotar(4096, 32, 1536, 512, 14336, 1024),
            llama(4096, 32, 8, 14336), [(2, 8000)], [(32, 8000)]),
        "2048x16h full": (
            kanotar(2048, 16, 768, 256, 8192, 8192),
            llama(2048, 16, 4, 8192),
            [(16, 2048)], [(1, 2048), (128, 2048)]),
        "7168x64h shared latents": (
            kanotar(7168, 64, 1536, 512, 18432, 8192, args.layers // 2),
            llama(7168, 56, 8, 18432), [(8, 2048)], [(32, 2048)]),
        "4096x32h attention": (
            bufulorn(4096, 32, 8, 14336, 8192), llama(4096, 32, 8, 14336),
            [(16, 2048), (2, 8000)], [(1, 2048), (32, 2048), (128, 2048),
                                      (32, 8000)]),
        "4096x32h attention and delta": (
            bufulorn(4096, 32, 8, 14336, 1024, "AD"),
            llama(4096, 32, 8, 14336), some[0] + [(2, 8000)], some[1]),
        # 8 of 64 experts of 1024: the active weights of one of 8192
        "2048x16h experts": (
            bufulorn(2048, 16, 4, 8192, 4096, "AAD", share=True,
                     experts=ExpertsDims(ff=1024, experts=64, top=8,
                                         groups=8, keep=4)),
            llama(2048, 16, 4, 8192), *some),
        "4096x32h parallel": (
            tebasun(4096, 32, 16, 14336, "P"),
            bufulorn(4096, 32, 8, 14336, 8192, "AD"),
            some[0] + [(2, 8000)], some[1] + [(32, 8000)]),
        "4096x32h recurrent": (
            tebasun(4096, 32, 16, 14336, "R"),
            bufulorn(4096, 32, 8, 14336, 8192, "D"),
            some[0] + [(2, 8000)], some[1]),
        # two thirds of the layers, the first half of them twice
        "2048x16h looped": (
            tebasun(2048, 16, 8, 8192, "PPR", layers=args.layers * 2 // 3,
                    loop=(0, args.layers - args.layers * 2 // 3, 2)),
            bufulorn(2048, 16, 4, 8192, 8192, "AD"), *some),
        "4096x32h retention": (
            kedelorn(4096, 32, 512, "R"),
            mixers(bufulorn(4096, 32, 32, 0, 8192, "D")),
            some[0] + [(2, 8000)], some[1]),
        "4096x32h rotary latent": (
            kedelorn(4096, 32, 512, "L"),
            mixers(kanotar(4096, 32, 1536, 512, 14336, 8192)),
            some[0] + [(2, 8000)], some[1] + [(32, 8000)]),
        # two matrices per expert where Bufulorn has three: the same active
        # weights, and as many in all
        "2048x16h streams": (
            kedelorn(2048, 16, 256, "RL", GatedExpertsDims(
                ff=1280, experts=76, top=8, shared=2048)),
            bufulorn(2048, 16, 4, 8192, 8192, "DA", routed=True,
                     experts=ExpertsDims(ff=1024, experts=64, top=8,
                                         groups=8, keep=4)), *some),
    }
    params = SamplingParams(temperature=0.0, min_p=0.0, max_tokens=10 ** 6)
    rows = []
    for name, (md, ld, prefills, decodes) in sizes.items():
        if args.only and name.split()[0] not in args.only.split(",") \
                and name not in args.only.split(","):
            continue
        models = {d.arch: build_model(d, device=dev) for d in (md, ld)}

        def run(kind, model, batch, ctx):
            eng = LLMEngine(model, max_batch_size=batch,
                            max_model_len=ctx + 64,
                            num_blocks=batch * ((ctx + 64) // 16 + 2))
            ids = torch.randint(4, V, (batch, ctx)).tolist()

            def start():
                seqs = [_Seq(seq_id=i, prompt_ids=p)
                        for i, p in enumerate(ids)]
                for s in seqs:
                    s.blocks = eng.blockman.alloc((ctx + 64) // 16 + 1)
                return seqs

            times = []
            if kind == "prefill":
                for i in range(args.warmup + args.steps):
                    seqs = start()
                    torch.cuda.synchronize()
                    t0 = time.perf_counter()
                    eng._run_prefill(seqs, params, {})
                    torch.cuda.synchronize()
                    times.append(time.perf_counter() - t0)
                    for s in seqs:
                        eng.release(s)
                n = batch * ctx
            else:
                seqs = start()
                eng._run_prefill(seqs, params, {})
                for i in range(args.warmup + args.steps):
                    torch.cuda.synchronize()
                    t0 = time.perf_counter()
                    eng._run_decode(seqs, params, {})
                    torch.cuda.synchronize()
                    times.append(time.perf_counter() - t0)
                n = batch
            times = sorted(times[args.warmup:])
            return n, times[len(times) // 2]

        for kind, todo in (("prefill", prefills), ("decode", decodes)):
            for batch, ctx in todo:
                row = {"size": name, "kind": kind, "batch": batch,
                       "context": ctx}
                for which, model in models.items():
                    n, t = run(kind, model, batch, ctx)
                    row[which + "_ms"] = round(t * 1e3, 3)
                    row[which + "_tok_s"] = round(n / t, 1)
                rows.append(row)
                print(json.dumps(row), flush=True)
        del models
        torch.cuda.empty_cache()
    print(json.dumps({"metric": "decoder layers, tokens/s",
                      "layers": args.layers, "steps": args.steps,
                      "warmup": args.warmup, "dtype": "bf16",
                      "data": "synthetic", "rows": rows}))


def bench_pipeline(args) -> None:
    """End-to-end semantic-chunk pipeline throughput:
    one step = one synthetic jsonl file through
    tokenize/split/buffer -> embed buffers -> GPU distance ->
    percentile chunking -> re-embed chunks -> write shard — the
    reference's wording ("semantic_chunk embedder") measured as
    a whole, host staging included. Reports docs/s and seqs/s plus a
    tokenize-vs-GPU breakdown. Single-rank (the DP story is covered by
    --mode embed)."""
    import random
    import shutil
    import tempfile
    from pathlib import Path

    from distllm_amd.distributed_embedding import embedding_worker

    have_gpu = torch.cuda.is_available()
    torch.manual_seed(1234)
    rng = random.Random(7)
    words = [f"w{i:03d}" for i in range(400)] + [
        "protein", "cell", "model", "study", "effect", "binding",
        "analysis", "method", "result", "treatment",
    ]

    def synth_doc() -> str:
        sents = []
        for _ in range(rng.randint(25, 60)):
            n = rng.randint(12, 24)
            s = " ".join(rng.choice(words) for _ in range(n))
            sents.append(s.capitalize() + ".")
        return " ".join(sents)

    root = Path(tempfile.mkdtemp(prefix="bench_pipeline_"))
    nfiles = args.warmup + args.steps
    files = []
    for f in range(nfiles):
        p = root / f"part_{f:03d}.jsonl"
        with open(p, "w") as fh:
            for _ in range(args.docs_per_file):
                fh.write(json.dumps({"text": synth_doc(), "path": f"{p.name}#{_}"}) + "\n")
        files.append(p)

    dataset_kwargs = {"name": "jsonl_chunk", "text_field": "text",
                      "batch_size": args.batch_size,
                      "num_data_workers": 4, "buffer_size": 4}
    encoder_kwargs = {"name": "auto",
                      "pretrained_model_name_or_path": args.model}
    pooler_kwargs = {"name": "mean"}
    embedder_kwargs = {"name": "semantic_chunk",
                       "chunk_batch_size": args.batch_size,
                       "normalize_embeddings": True}
    writer_kwargs = {"name": "numpy"}

    out = root / "out"
    out.mkdir()

    n_docs = n_bufs = n_chunks = 0
    t_total = 0.0
    for i, p in enumerate(files):
        timed = i >= args.warmup
        if have_gpu:
            torch.cuda.synchronize()
        t0 = time.perf_counter()
        embedding_worker(p, out, dataset_kwargs, encoder_kwargs,
                         pooler_kwargs, embedder_kwargs, writer_kwargs)
        if have_gpu:
            torch.cuda.synchronize()
        dt = time.perf_counter() - t0
        if timed:
            t_total += dt
            n_docs += args.docs_per_file

    # breakdown on one extra file: host (tokenize/split/buffer) vs rest
    from distllm_amd.embed import (get_dataset, get_embedder, get_encoder,
                                   get_pooler)

    enc = get_encoder(encoder_kwargs, register=True)
    ds = get_dataset(dataset_kwargs)
    t0 = time.perf_counter()
    dl = ds.get_dataloader(files[0], enc)
    t_host = time.perf_counter() - t0
    n_bufs = len(dl.dataset)
    emb = get_embedder(embedder_kwargs)
    t0 = time.perf_counter()
    res = emb.embed(dl, enc, get_pooler(pooler_kwargs))
    if have_gpu:
        torch.cuda.synchronize()
    t_embed = time.perf_counter() - t0
    n_chunks = len(res.text)

    value = n_docs / t_total
    print(json.dumps({
        "metric": f"docs/sec semantic-chunk embedded ({args.model})",
        "value": round(value, 2),
        "unit": "docs/s",
        "n_gpus": 1,
        "steps": args.steps,
        "warmup": args.warmup,
        "ms_per_step": round(t_total / args.steps * 1000.0, 3),
        "higher_is_better": True,
        "scaling": "weak",
        "vs_baseline": None,
        "dtype": "bf16" if have_gpu else "fp32",
        "data": "synthetic",
        "config": {
            "model": args.model,
            "docs_per_file": args.docs_per_file,
            "batch_size": args.batch_size,
            "embedder": "semantic_chunk",
            "parallelism": "dp1",
        },
        "breakdown": {
            "host_tokenize_split_s_per_file": round(t_host, 3),
            "embed_chunk_write_s_per_file": round(t_embed, 3),
            "buffers_per_file": n_bufs,
            "chunks_per_file": n_chunks,
            "buffers_per_s": round(n_bufs * args.steps / t_total, 1),
        },
    }))
    shutil.rmtree(root, ignore_errors=True)


if __name__ == "__main__":
    main()


