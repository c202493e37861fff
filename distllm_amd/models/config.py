"""Model architecture configs for the native MI355X model family.

Covers the reference's encoder zoo plus the
decoder family used for generation (K15):
  - BERT-class bidirectional encoders (S-PubMedBERT, pubmedbert,
    bert-base) and RoBERTa-class (offset position ids)
  - ESM2 protein encoders (rotary, no token types)
  - ESMC protein encoders
  - Mistral-class decoder embedders (SFR-Embedding-Mistral)
  - Llama-class causal LMs for generation
  - Qwen2-class causal LMs (llama family + qkv bias)
  - Kanotar and Bufulorn causal LMs: every layer has its own description
    (LayeredDims)
Dims are from the public model cards; weights are random-init here
(no network) or loadable from local safetensors.
"""

from __future__ import annotations

import json
from pathlib import Path
from typing import Literal

from pydantic import (BaseModel, ConfigDict, NonNegativeInt, PositiveFloat,
                      PositiveInt, model_validator)


class ModelDims(BaseModel):
    arch: Literal["bert", "esm2", "esmc", "mistral", "llama", "qwen2"]
    vocab_size: int
    hidden_size: int
    num_layers: int
    num_heads: int
    num_kv_heads: int | None = None  # None -> MHA
    intermediate_size: int
    max_position_embeddings: int = 512
    layer_norm_eps: float = 1e-12
    rms_norm_eps: float = 1e-5
    rope_theta: float = 10000.0
    type_vocab_size: int = 2          # BERT token types
    gelu: Literal["tanh", "erf"] = "erf"
    tie_word_embeddings: bool = False
    attention_bias: bool = False      # Qwen2: bias on q/k/v only
    # RoBERTa-family: positions = cumsum(ids != pad) + pad (HF
    # create_position_ids_from_input_ids), vs BERT's arange
    position_style: Literal["absolute", "roberta"] = "absolute"
    pad_token_id: int = 0

    @property
    def head_dim(self) -> int:
        return self.hidden_size // self.num_heads

    @property
    def kv_heads(self) -> int:
        return self.num_kv_heads or self.num_heads


class _Strict(BaseModel):
    model_config = ConfigDict(extra="forbid")


class LatentAttentionDims(_Strict):
    """Attention whose keys and values are linear in one cached latent of
    kv_rank numbers per token; queries come from a latent of q_rank."""

    type: Literal["latent_attention"] = "latent_attention"
    heads: PositiveInt
    dim: PositiveInt           # query/key size per head
    vdim: PositiveInt          # value size per head
    q_rank: PositiveInt
    kv_rank: PositiveInt
    scale: float
    window: PositiveInt        # a token sees itself and window - 1 before
    kv_from: int | None = None  # layer whose latents this one reads


    def shared_sizes(self) -> dict[str, int]:
        """What a layer and the layer whose cache it reads agree on."""
        return {"kv_rank": self.kv_rank}


class AttentionDims(_Strict):
    """Softmax attention on cached keys and values. Queries and keys are
    normed per head; scores are capped at softcap * tanh and lose
    r1 * ln(1 + r2 * distance), r1 and r2 being weights of the head; the
    heads' outputs are gated. A token sees the earlier tokens of its own
    chunk: positions are cut into chunks of `chunk` from position 0."""

    type: Literal["attention"] = "attention"
    heads: PositiveInt
    kv_heads: PositiveInt
    dim: PositiveInt           # query/key size per head
    vdim: PositiveInt          # value size per head
    scale: float
    softcap: PositiveFloat
    chunk: PositiveInt
    kv_from: NonNegativeInt | None = None  # layer whose keys and values

    def shared_sizes(self) -> dict[str, int]:
        return {k: getattr(self, k)
                for k in ("heads", "kv_heads", "dim", "vdim")}


class DeltaDims(_Strict):
    """Gated delta rule: a recurrent [dim, vdim] state per head, behind
    short causal convolutions of `conv` taps; kv_heads queries and keys,
    heads values."""

    type: Literal["delta"] = "delta"
    heads: PositiveInt
    kv_heads: PositiveInt
    dim: PositiveInt
    vdim: PositiveInt
    conv: PositiveInt
    unit_eps: float = 1e-6     # of the unit queries and keys


class ClampedGluDims(_Strict):
    """Feed-forward g * sigmoid(alpha g) * (u + shift), gate g clamped
    from above and up-projection u from both sides at `limit`."""

    kind: Literal["dense"] = "dense"
    ff: PositiveInt
    limit: float
    alpha: float = 1.702
    shift: float = 1.0


class XieluDims(_Strict):
    """Feed-forward down(xielu(up)), the activation's two numbers being
    weights of the layer."""

    kind: Literal["xielu"] = "xielu"
    ff: PositiveInt


class ExpertsDims(_Strict):
    """Routed gated-unit experts. Experts form `groups` equal groups of
    neighbours; the `top` experts of the `keep` best groups serve a token,
    weighted by their softmax scores over all experts."""

    kind: Literal["experts"] = "experts"
    ff: PositiveInt
    experts: PositiveInt
    top: PositiveInt
    groups: PositiveInt = 1
    keep: PositiveInt = 1

    @model_validator(mode="after")
    def _check_groups(self):
        if self.experts % self.groups:
            raise ValueError(f"{self.experts} experts do not form "
                             f"{self.groups} equal groups")
        if self.keep > self.groups:
            raise ValueError(f"keep {self.keep} of {self.groups} groups")
        if self.top > self.experts // self.groups * self.keep:
            raise ValueError(f"top {self.top} is more than the experts of "
                             f"{self.keep} groups")
        return self


class LayerDims(_Strict):
    mixer: LatentAttentionDims | AttentionDims | DeltaDims
    mlp: ClampedGluDims | XieluDims | ExpertsDims | None = None


class LayeredDims(BaseModel):
    """A decoder whose layers are described one by one."""

    arch: Literal["kanotar", "bufulorn"]
    vocab_size: PositiveInt
    hidden_size: PositiveInt
    layers: list[LayerDims]
    norm_eps: float
    logit_scale: float = 1.0
    # bounded only by a position table, where the design has one
    max_position_embeddings: PositiveInt = 1 << 20

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    @model_validator(mode="after")
    def _check_sharing(self):
        if not self.layers:
            raise ValueError("a model needs at least one layer")
        for i, layer in enumerate(self.layers):
            m = layer.mixer
            if not isinstance(m, LatentAttentionDims) \
                    and m.heads % m.kv_heads:
                raise ValueError(f"layer {i}: {m.heads} heads are not a "
                                 f"multiple of {m.kv_heads} kv_heads")
            j = getattr(m, "kv_from", None)
            if j is None:
                continue
            if not 0 <= j < i:
                raise ValueError(f"layer {i}: kv_from {j} is not an "
                                 "earlier layer")
            src = self.layers[j].mixer
            if type(src) is not type(m) or src.kv_from is not None:
                raise ValueError(f"layer {i}: kv_from {j} has no keys and "
                                 "values of its own")
            for k, v in m.shared_sizes().items():
                if src.shared_sizes()[k] != v:
                    raise ValueError(f"layer {i}: {k} differs from that "
                                     f"of layer {j}")
        return self


def _take(d: dict, name: str, where: str):
    """The only entry of a nested description."""
    if name not in d or len(d) != 1:
        raise ValueError(f"{where} has keys {sorted(d)}, expected {name}")
    return d[name]


def _kanotar_dims(cfg: dict) -> LayeredDims:
    layers = []
    for i, entry in enumerate(cfg["layers"]):
        if entry["type"] != "latent_attention":
            raise ValueError(f"layer {i}: unknown mixer {entry['type']!r}")
        mixer = dict(entry["mixer"])
        mixer["window"] = _take(mixer.pop("mask"), "size", f"layer {i}: mask")
        mlp = entry.get("mlp")
        layers.append(LayerDims(
            mixer=LatentAttentionDims(**mixer),
            mlp=None if mlp is None else ClampedGluDims(**mlp)))
    return LayeredDims(arch="kanotar", vocab_size=cfg["vocab"],
                       hidden_size=cfg["width"], layers=layers,
                       norm_eps=cfg["norm"]["eps"],
                       logit_scale=cfg["logit_scale"])


def _bufulorn_mlp(mlp: dict, where: str):
    mlp = dict(mlp)
    kind = mlp.pop("kind", None)
    if kind == "dense":
        return XieluDims(**mlp)
    if kind != "moe":
        raise ValueError(f"{where}: unknown feed-forward kind {kind!r}")
    router = dict(mlp.pop("router"))
    groups = dict(router.pop("groups"))
    dims = ExpertsDims(ff=_take(mlp.pop("expert"), "ff", f"{where}: expert"),
                       groups=groups.pop("count"), keep=groups.pop("keep"),
                       **router)
    if mlp or groups:
        raise ValueError(f"{where}: unknown feed-forward keys "
                         f"{sorted({**mlp, **groups})}")
    return dims


def _bufulorn_dims(cfg: dict) -> LayeredDims:
    layers = []
    for i, entry in enumerate(cfg["layers"]):
        mixer = dict(entry["mixer"])
        if entry["type"] == "attention":
            mixer["chunk"] = _take(mixer.pop("mask"), "size",
                                   f"layer {i}: mask")
            mixer = AttentionDims(**mixer)
        elif entry["type"] == "delta":
            mixer = DeltaDims(**mixer)
        else:
            raise ValueError(f"layer {i}: unknown mixer {entry['type']!r}")
        mlp = entry.get("mlp")
        layers.append(LayerDims(
            mixer=mixer,
            mlp=None if mlp is None else _bufulorn_mlp(mlp, f"layer {i}")))
    return LayeredDims(arch="bufulorn", vocab_size=cfg["vocab"],
                       hidden_size=cfg["width"], layers=layers,
                       norm_eps=cfg["norm"]["eps"],
                       max_position_embeddings=cfg["max_positions"])


# config.json "architecture" -> reader of the rest of the file
CONFIG_READERS = {"Kanotar": _kanotar_dims, "Bufulorn": _bufulorn_dims}


def dims_from_checkpoint(path: str | Path) -> LayeredDims | None:
    """Dims from a checkpoint folder's config.json; None when there is no
    such file or it names no architecture that is described in full."""
    f = Path(path) / "config.json"
    if not f.is_file():
        return None
    cfg = json.loads(f.read_text())
    reader = CONFIG_READERS.get(cfg.get("architecture"))
    return reader(cfg) if reader else None


def layered_preset(num_layers: int, hidden: int, vocab: int, heads: int,
                   dim: int, vdim: int, q_rank: int, kv_rank: int, ff: int,
                   windows: list[int], share_from: int | None = None,
                   limit: float = 7.0, logit_scale: float = 1.0,
                   eps: float = 1e-5) -> LayeredDims:
    """Kanotar dims of repeated layers: window i is windows[i % len]; from
    layer share_from on, layers read the latents of layer share_from - 1."""
    layers = []
    for i in range(num_layers):
        shared = share_from is not None and i >= share_from
        layers.append(LayerDims(
            mixer=LatentAttentionDims(
                heads=heads, dim=dim, vdim=vdim, q_rank=q_rank,
                kv_rank=kv_rank, scale=dim ** -0.5,
                window=windows[i % len(windows)],
                kv_from=share_from - 1 if shared else None),
            mlp=ClampedGluDims(ff=ff, limit=limit)))
    return LayeredDims(arch="kanotar", vocab_size=vocab, hidden_size=hidden,
                       layers=layers, norm_eps=eps, logit_scale=logit_scale)


def hybrid_preset(num_layers: int, hidden: int, vocab: int, heads: int,
                  kv_heads: int, dim: int, ff: int, chunk: int,
                  experts: ExpertsDims | None = None,
                  order: str = "AD", share: bool = False,
                  delta_dim: int | None = None, conv: int = 4,
                  max_positions: int = 16384,
                  eps: float = 1e-5) -> LayeredDims:
    """Bufulorn dims of repeated layers: mixers follow `order` (A attention,
    D delta rule), every other feed-forward is `experts` where given. With
    `share`, every other attention layer reads the keys and values of the
    one before."""
    layers, owner = [], None
    for i in range(num_layers):
        if order[i % len(order)] == "A":
            mixer = AttentionDims(
                heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim,
                scale=dim ** -0.5, softcap=30.0, chunk=chunk,
                kv_from=owner if share else None)
            owner = i if owner is None else None
        else:
            mixer = DeltaDims(heads=heads, kv_heads=kv_heads,
                              dim=delta_dim or dim, vdim=dim, conv=conv)
        dense = experts is None or i % 2 == 0
        layers.append(LayerDims(
            mixer=mixer, mlp=XieluDims(ff=ff) if dense else experts))
    return LayeredDims(arch="bufulorn", vocab_size=vocab, hidden_size=hidden,
                       layers=layers, norm_eps=eps,
                       max_position_embeddings=max_positions)


PRESETS: dict[str, ModelDims | LayeredDims] = {
    # S-PubMedBERT / PubMedBERT-base: the reference's headline embed
    # encoder (examples/embed/AMP.nougat.pubmedbert.yaml)
    "pubmedbert-base": ModelDims(
        arch="bert", vocab_size=30528, hidden_size=768, num_layers=12,
        num_heads=12, intermediate_size=3072, max_position_embeddings=512,
        layer_norm_eps=1e-12, gelu="erf",
    ),
    "bert-tiny": ModelDims(  # test-size
        arch="bert", vocab_size=512, hidden_size=128, num_layers=2,
        num_heads=2, intermediate_size=256, max_position_embeddings=128,
    ),
    # RoBERTa-base (FacebookAI/roberta-base): BERT-family encoder with
    # offset position ids and a single token type
    "roberta-base": ModelDims(
        arch="bert", vocab_size=50265, hidden_size=768, num_layers=12,
        num_heads=12, intermediate_size=3072,
        max_position_embeddings=514, layer_norm_eps=1e-5, gelu="erf",
        type_vocab_size=1, position_style="roberta", pad_token_id=1,
    ),
    # ESM2 sizes (facebook/esm2_t33_650M_UR50D etc.)
    "esm2-8m": ModelDims(
        arch="esm2", vocab_size=33, hidden_size=320, num_layers=6,
        num_heads=20, intermediate_size=1280, max_position_embeddings=1026,
        layer_norm_eps=1e-5, gelu="erf",
    ),
    "esm2-650m": ModelDims(
        arch="esm2", vocab_size=33, hidden_size=1280, num_layers=33,
        num_heads=20, intermediate_size=5120, max_position_embeddings=1026,
        layer_norm_eps=1e-5, gelu="erf",
    ),
    # ESMC (EvolutionaryScale; 300m: H=960 L=30 heads=15, 600m: 1152/36/18)
    "esmc-300m": ModelDims(
        arch="esmc", vocab_size=64, hidden_size=960, num_layers=30,
        num_heads=15, intermediate_size=2560, max_position_embeddings=2048,
        layer_norm_eps=1e-5,
    ),
    "esmc-600m": ModelDims(
        arch="esmc", vocab_size=64, hidden_size=1152, num_layers=36,
        num_heads=18, intermediate_size=3072, max_position_embeddings=2048,
        layer_norm_eps=1e-5,
    ),
    # SFR-Embedding-Mistral (7B): the reference's large embedder
    "mistral-7b": ModelDims(
        arch="mistral", vocab_size=32000, hidden_size=4096, num_layers=32,
        num_heads=32, num_kv_heads=8, intermediate_size=14336,
        max_position_embeddings=32768, rms_norm_eps=1e-5, rope_theta=10000.0,
    ),
    "mistral-tiny": ModelDims(
        arch="mistral", vocab_size=1024, hidden_size=256, num_layers=2,
        num_heads=4, num_kv_heads=2, intermediate_size=512,
        max_position_embeddings=512,
    ),
    # Llama-3-8B for the generate/RAG path
    "llama3-8b": ModelDims(
        arch="llama", vocab_size=128256, hidden_size=4096, num_layers=32,
        num_heads=32, num_kv_heads=8, intermediate_size=14336,
        max_position_embeddings=8192, rms_norm_eps=1e-5, rope_theta=500000.0,
    ),
    # 140 GB of bf16 weights: fits — with KV headroom — on ONE 288 GB
    # MI355X, no tensor parallelism required (the reference's vLLM
    # configs needed TP8 for far smaller models on 80 GB cards)
    "llama3-70b": ModelDims(
        arch="llama", vocab_size=128256, hidden_size=8192, num_layers=80,
        num_heads=64, num_kv_heads=8, intermediate_size=28672,
        max_position_embeddings=8192, rms_norm_eps=1e-5, rope_theta=500000.0,
    ),
    "llama-tiny": ModelDims(
        arch="llama", vocab_size=2048, hidden_size=256, num_layers=2,
        num_heads=4, num_kv_heads=2, intermediate_size=512,
        max_position_embeddings=512,
    ),
    # Qwen2-7B-Instruct: llama-family + qkv bias (HF Qwen2ForCausalLM)
    "qwen2-7b": ModelDims(
        arch="qwen2", vocab_size=152064, hidden_size=3584, num_layers=28,
        num_heads=28, num_kv_heads=4, intermediate_size=18944,
        max_position_embeddings=32768, rms_norm_eps=1e-6,
        rope_theta=1_000_000.0, attention_bias=True,
    ),
    "qwen2-tiny": ModelDims(
        arch="qwen2", vocab_size=1024, hidden_size=256, num_layers=2,
        num_heads=4, num_kv_heads=2, intermediate_size=512,
        max_position_embeddings=512, rms_norm_eps=1e-6,
        attention_bias=True,
    ),
    # layers of the llama3-8b size, for like-for-like measurements
    "kanotar-8b": layered_preset(
        32, 4096, 128256, heads=32, dim=128, vdim=128, q_rank=1536,
        kv_rank=512, ff=14336, windows=[4096],
    ),
    "kanotar-tiny": layered_preset(
        3, 256, 1024, heads=4, dim=32, vdim=32, q_rank=64, kv_rank=64,
        ff=512, windows=[48, 32], share_from=2,
    ),
    # attention and delta-rule layers of the llama3-8b size, every other
    # feed-forward routed
    "bufulorn-8b": hybrid_preset(
        32, 4096, 128256, heads=32, kv_heads=8, dim=128, ff=14336,
        chunk=8192, experts=ExpertsDims(ff=1792, experts=32, top=4,
                                        groups=4, keep=2),
    ),
    "bufulorn-tiny": hybrid_preset(
        4, 256, 1024, heads=4, kv_heads=2, dim=32, ff=512, chunk=48,
        experts=ExpertsDims(ff=64, experts=6, top=2, groups=3, keep=2),
        order="AAD", share=True, max_positions=512,
    ),
}


def get_dims(name: str) -> ModelDims | LayeredDims:
    if name not in PRESETS:
        raise KeyError(
            f"unknown model preset {name!r}; available: {sorted(PRESETS)}"
        )
    return PRESETS[name]
