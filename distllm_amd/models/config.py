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
  - Kanotar, Bufulorn, Tebasun and Kedelorn causal LMs: every layer has
    its own description (LayeredDims)
Dims are from the public model cards; weights are random-init here
(no network) or loadable from local safetensors.
"""

from __future__ import annotations

import json
import math
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


def _check_groups(m):
    if m.heads % m.kv_heads:
        raise ValueError(f"{m.heads} heads are not a multiple of "
                         f"{m.kv_heads} kv_heads")
    return m


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


class YarnDims(_Strict):
    """YaRN: frequencies are divided by `factor`, by degrees between the
    pairs that turn `fast` and `slow` times over `original` positions."""

    factor: PositiveFloat
    original: PositiveFloat
    fast: PositiveFloat
    slow: PositiveFloat


class RotaryDims(_Strict):
    """Rotation of the first `dims` numbers of a head: number i pairs with
    number i + dims / 2 and turns by base^(-2i / dims) per position."""

    base: PositiveFloat
    dims: PositiveInt
    scaling: YarnDims | None = None

    @model_validator(mode="after")
    def _check_even(self):
        if self.dims % 2:
            raise ValueError(f"{self.dims} rotated numbers form no pairs")
        return self

    def frequencies(self) -> tuple[list[float], float]:
        """-> frequency of every pair, and the factor on cos and sin."""
        n, half = self.dims, self.dims // 2
        freq = [self.base ** (-2.0 * i / n) for i in range(half)]
        y = self.scaling
        if y is None:
            return freq, 1.0

        def pair_of(turns: float) -> float:
            return (n * math.log(y.original / (2 * math.pi * turns))
                    / (2 * math.log(self.base)))

        lo = max(math.floor(pair_of(y.fast)), 0)
        hi = min(math.ceil(pair_of(y.slow)), n - 1)
        for i in range(half):
            ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
            freq[i] *= ramp / y.factor + 1.0 - ramp
        return freq, 0.1 * math.log(y.factor) + 1.0


class RotaryAttentionDims(_Strict):
    """Causal softmax attention whose values are the keys as projected,
    before norm and rotation. Queries and keys are normed per head, then
    rotated; a learned sink per head takes part in the softmax."""

    type: Literal["rotary_attention"] = "rotary_attention"
    heads: PositiveInt
    kv_heads: PositiveInt
    dim: PositiveInt
    vdim: PositiveInt          # dim, as the values are keys
    rot: RotaryDims
    scale: float

    @model_validator(mode="after")
    def _check_sizes(self):
        if self.vdim != self.dim:
            raise ValueError(f"values are keys: vdim {self.vdim} must be "
                             f"dim {self.dim}")
        if self.rot.dims > self.dim:
            raise ValueError(f"{self.rot.dims} rotated numbers in heads of "
                             f"{self.dim}")
        return _check_groups(self)


class ChannelDeltaDims(_Strict):
    """Gated delta rule with a decay per head and key channel, which
    comes from a pair of products through `decay_rank` numbers; the output
    gate comes from a pair through `gate_rank`."""

    type: Literal["channel_delta"] = "channel_delta"
    heads: PositiveInt
    kv_heads: PositiveInt
    dim: PositiveInt
    vdim: PositiveInt
    conv: PositiveInt
    decay_rank: PositiveInt
    gate_rank: PositiveInt
    unit_eps: float = 1e-6

    @model_validator(mode="after")
    def _check_sizes(self):
        return _check_groups(self)


class RotaryLatentDims(_Strict):
    """Causal attention on a cached latent of kv_rank numbers per token and
    rot_dim rotated key numbers that all heads share; queries have `dim`
    numbers for the keys made from the latent and rot_dim rotated ones. A
    learned sink per head takes part in the softmax; head outputs are
    multiplied by a gate each."""

    type: Literal["rotary_latent"] = "rotary_latent"
    heads: PositiveInt
    dim: PositiveInt           # unrotated query/key size per head
    rot_dim: PositiveInt       # rotated query/key size
    vdim: PositiveInt          # value size per head
    kv_rank: PositiveInt
    rot: RotaryDims
    scale: float
    kv_from: NonNegativeInt | None = None  # layer whose cache this one reads

    @model_validator(mode="after")
    def _check_sizes(self):
        if self.rot.dims != self.rot_dim:
            raise ValueError(f"{self.rot.dims} rotated numbers, but rot_dim "
                             f"{self.rot_dim}")
        return self

    def shared_sizes(self) -> dict:
        return {"kv_rank": self.kv_rank, "rot_dim": self.rot_dim,
                "rot": self.rot}


class RetentionDims(_Strict):
    """Linear attention with a fixed decay per head: a recurrent [dim,
    vdim] state, rotated queries and keys."""

    type: Literal["retention"] = "retention"
    heads: PositiveInt
    dim: PositiveInt
    vdim: PositiveInt
    rot: RotaryDims
    decay: list[float]

    @model_validator(mode="after")
    def _check_sizes(self):
        if len(self.decay) != self.heads:
            raise ValueError(f"{len(self.decay)} decays for {self.heads} "
                             "heads")
        if not all(0.0 < x <= 1.0 for x in self.decay):
            raise ValueError("decays must be above 0 and at most 1")
        if self.rot.dims > self.dim:
            raise ValueError(f"{self.rot.dims} rotated numbers in heads of "
                             f"{self.dim}")
        return self


class ParallelDims(_Strict):
    """Two mixers side by side on the same input:
    left_scale * left + right_scale * right."""

    type: Literal["parallel"] = "parallel"
    left: RotaryAttentionDims
    right: ChannelDeltaDims
    left_scale: float
    right_scale: float


class LruDims(_Strict):
    """Real-gated linear recurrent unit on one branch of `width`, behind a
    causal convolution of `conv` taps, times a GELU branch. Its gates are
    block-diagonal products of `blocks` blocks; decays are
    exp(-decay_scale * gate * softplus(lam))."""

    type: Literal["rglru"] = "rglru"
    width: PositiveInt
    blocks: PositiveInt
    conv: PositiveInt
    decay_scale: float = 8.0

    @model_validator(mode="after")
    def _check_blocks(self):
        if self.width % self.blocks:
            raise ValueError(f"width {self.width} does not split into "
                             f"{self.blocks} equal blocks")
        return self


class ClampedGluDims(_Strict):
    """Feed-forward g * sigmoid(alpha g) * (u + shift), gate g clamped
    from above and up-projection u from both sides at `limit`."""

    kind: Literal["dense"] = "dense"
    ff: PositiveInt
    limit: float
    alpha: float = 1.702
    shift: float = 1.0


class SwigluDims(_Strict):
    """Feed-forward down(silu(gate) * up)."""

    kind: Literal["swiglu"] = "swiglu"
    ff: PositiveInt


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


class GatedExpertsDims(_Strict):
    """Routed squared-ReLU experts. The `top` experts with the largest
    sigmoid scores plus corrections serve a token, weighted by `scale`
    times their scores without them. A shared expert of `shared` columns,
    where there is one, serves every token through a gate of its own."""

    kind: Literal["gated_experts"] = "gated_experts"
    ff: PositiveInt
    experts: PositiveInt
    top: PositiveInt
    scale: float = 1.0
    shared: PositiveInt | None = None

    @model_validator(mode="after")
    def _check_top(self):
        if self.top > self.experts:
            raise ValueError(f"top {self.top} of {self.experts} experts")
        return self


class LayerDims(_Strict):
    mixer: (LatentAttentionDims | AttentionDims | DeltaDims | ParallelDims
            | LruDims | RotaryLatentDims | RetentionDims)
    mlp: (ClampedGluDims | SwigluDims | XieluDims | ExpertsDims
          | GatedExpertsDims | None) = None


class LoopDims(_Strict):
    """Layers start .. stop - 1 run `times` times in a row with the same
    weights; each pass has its own cache and state."""

    start: NonNegativeInt
    stop: PositiveInt
    times: PositiveInt


class LayeredDims(BaseModel):
    """A decoder whose layers are described one by one."""

    arch: Literal["kanotar", "bufulorn", "tebasun", "kedelorn"]
    vocab_size: PositiveInt
    hidden_size: PositiveInt
    layers: list[LayerDims]
    norm_eps: float
    logit_scale: float = 1.0
    embed_scale: float = 1.0
    loop: LoopDims | None = None
    side_dim: PositiveInt | None = None  # per-layer token inputs
    streams: PositiveInt | None = None   # copies of the residual stream
    # bounded only by a position table, where the design has one
    max_position_embeddings: PositiveInt = 1 << 20

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    def layer_runs(self) -> list[tuple[int, int | None]]:
        """Layers in running order, each with the number of the loop's
        pass that begins with it, or None."""
        n = len(self.layers)
        if self.loop is None:
            return [(i, None) for i in range(n)]
        lp, runs = self.loop, []
        for t in range(lp.times):
            runs += [(i, t if i == lp.start else None)
                     for i in range(lp.start, lp.stop)]
        return ([(i, None) for i in range(lp.start)] + runs
                + [(i, None) for i in range(lp.stop, n)])

    @model_validator(mode="after")
    def _check_loop(self):
        lp = self.loop
        if lp is not None and not lp.start < lp.stop <= len(self.layers):
            raise ValueError(f"loop over layers {lp.start} to {lp.stop} of "
                             f"{len(self.layers)}")
        return self

    @model_validator(mode="after")
    def _check_sharing(self):
        if not self.layers:
            raise ValueError("a model needs at least one layer")
        for i, layer in enumerate(self.layers):
            m = layer.mixer
            if isinstance(m, (AttentionDims, DeltaDims)) \
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


def _kanotar_dims(cfg: dict, shapes=None) -> LayeredDims:
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


def _bufulorn_dims(cfg: dict, shapes=None) -> LayeredDims:
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


def _tebasun_dims(cfg: dict, shapes=None) -> LayeredDims:
    layers, sizes = [], shapes()
    for i, entry in enumerate(cfg["layers"]):
        mixer = dict(entry["mixer"])
        if entry["type"] == "parallel":
            # the inner sizes of the two pairs of products are told by
            # their tensors alone
            pre = f"l{i}.mix.right."
            mixer["right"] = dict(mixer["right"],
                                  decay_rank=sizes[pre + "a1"][0],
                                  gate_rank=sizes[pre + "g1"][0])
            mixer = ParallelDims(**mixer)
        elif entry["type"] == "rglru":
            mixer = LruDims(**mixer)
        else:
            raise ValueError(f"layer {i}: unknown mixer {entry['type']!r}")
        mlp = entry.get("mlp")
        if mlp is not None:
            mlp = dict(mlp)
            kind = mlp.pop("kind", None)
            if kind != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward kind "
                                 f"{kind!r}")
            mlp = SwigluDims(**mlp)
        layers.append(LayerDims(mixer=mixer, mlp=mlp))
    loop, side = cfg.get("loop"), cfg.get("token_side")
    return LayeredDims(arch="tebasun", vocab_size=cfg["vocab"],
                       hidden_size=cfg["width"], layers=layers,
                       norm_eps=cfg["norm"]["eps"],
                       embed_scale=cfg["embedding"]["scale"],
                       loop=None if loop is None else LoopDims(**loop),
                       side_dim=None if side is None else side["dim"])


def _kedelorn_mlp(mlp: dict, where: str) -> GatedExpertsDims:
    mlp = dict(mlp)
    kind = mlp.pop("kind", None)
    if kind != "moe":
        raise ValueError(f"{where}: unknown feed-forward kind {kind!r}")
    shared = mlp.pop("shared", None)
    if shared is not None:
        shared = _take(shared, "ff", f"{where}: shared")
    router = dict(mlp.pop("router"))
    dims = GatedExpertsDims(
        ff=_take(mlp.pop("expert"), "ff", f"{where}: expert"), shared=shared,
        experts=router.pop("experts"), top=router.pop("top"),
        scale=router.pop("scale"))
    if mlp or router:
        raise ValueError(f"{where}: unknown feed-forward keys "
                         f"{sorted({**mlp, **router})}")
    return dims


def _kedelorn_dims(cfg: dict, shapes=None) -> LayeredDims:
    layers = []
    for i, entry in enumerate(cfg["layers"]):
        if entry["type"] == "retention":
            mixer = RetentionDims(**entry["mixer"])
        elif entry["type"] == "latent_attention":
            mixer = RotaryLatentDims(**entry["mixer"])
        else:
            raise ValueError(f"layer {i}: unknown mixer {entry['type']!r}")
        mlp = entry.get("mlp")
        layers.append(LayerDims(
            mixer=mixer,
            mlp=None if mlp is None else _kedelorn_mlp(mlp, f"layer {i}")))
    return LayeredDims(arch="kedelorn", vocab_size=cfg["vocab"],
                       hidden_size=cfg["width"], layers=layers,
                       norm_eps=cfg["norm"]["eps"], streams=cfg["streams"])


# config.json "architecture" -> reader of the rest of the file; `shapes`
# returns the checkpoint's tensor shapes
CONFIG_READERS = {"Kanotar": _kanotar_dims, "Bufulorn": _bufulorn_dims,
                  "Tebasun": _tebasun_dims, "Kedelorn": _kedelorn_dims}


def checkpoint_shapes(path: str | Path) -> dict[str, tuple[int, ...]]:
    """Tensor name -> shape, from the headers of a folder's safetensors."""
    from safetensors import safe_open

    shapes = {}
    for f in sorted(Path(path).glob("*.safetensors")):
        with safe_open(str(f), "pt") as src:
            for name in src.keys():
                shapes[name] = tuple(src.get_slice(name).get_shape())
    return shapes


def dims_from_checkpoint(path: str | Path) -> LayeredDims | None:
    """Dims from a checkpoint folder's config.json; None when there is no
    such file or it names no architecture that is described in full."""
    f = Path(path) / "config.json"
    if not f.is_file():
        return None
    cfg = json.loads(f.read_text())
    reader = CONFIG_READERS.get(cfg.get("architecture"))
    return reader(cfg, lambda: checkpoint_shapes(path)) if reader else None


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


def looped_preset(num_layers: int, hidden: int, vocab: int, heads: int,
                  kv_heads: int, dim: int, ff: int, order: str = "PPR",
                  lru_width: int | None = None, blocks: int = 16,
                  rank: int | None = None, side: int = 256,
                  loop: tuple[int, int, int] | None = None,
                  original: int = 8192, eps: float = 1e-5) -> LayeredDims:
    """Tebasun dims of repeated layers: mixers follow `order` (P attention
    beside the delta rule, with half of the heads each; R linear recurrent
    unit)."""
    layers = []
    for i in range(num_layers):
        if order[i % len(order)] == "P":
            mixer = ParallelDims(
                left=RotaryAttentionDims(
                    heads=heads // 2, kv_heads=kv_heads // 2, dim=dim,
                    vdim=dim, scale=dim ** -0.5, rot=RotaryDims(
                        base=500000.0, dims=dim // 2, scaling=YarnDims(
                            factor=4.0, original=original, fast=32.0,
                            slow=1.0))),
                right=ChannelDeltaDims(
                    heads=heads // 2, kv_heads=heads // 2, dim=dim,
                    vdim=dim, conv=4, decay_rank=rank or dim,
                    gate_rank=rank or dim),
                left_scale=0.7, right_scale=0.7)
        else:
            mixer = LruDims(width=lru_width or hidden, blocks=blocks, conv=4)
        layers.append(LayerDims(mixer=mixer, mlp=SwigluDims(ff=ff)))
    lp = loop or (0, num_layers, 1)
    return LayeredDims(arch="tebasun", vocab_size=vocab, hidden_size=hidden,
                       layers=layers, norm_eps=eps,
                       embed_scale=hidden ** 0.5, side_dim=side,
                       loop=LoopDims(start=lp[0], stop=lp[1], times=lp[2]))


def streamed_preset(num_layers: int, hidden: int, vocab: int, heads: int,
                    dim: int, kv_rank: int, mlp: GatedExpertsDims | None,
                    order: str = "RL", rot_dim: int = 64,
                    vdim: int | None = None, streams: int = 4,
                    share: bool = False, original: int = 4096,
                    eps: float = 1e-5) -> LayeredDims:
    """Kedelorn dims of repeated layers: mixers follow `order` (R
    retention, L latent attention). With `share`, every other attention
    layer reads the latents of the one before."""
    layers, owner = [], None
    for i in range(num_layers):
        if order[i % len(order)] == "R":
            mixer = RetentionDims(
                heads=heads, dim=dim, vdim=vdim or dim,
                rot=RotaryDims(base=10000.0, dims=dim),
                decay=[1 - 2.0 ** (-5 - 6 * h / heads)
                       for h in range(heads)])
        else:
            mixer = RotaryLatentDims(
                heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim or dim,
                kv_rank=kv_rank, scale=(dim + rot_dim) ** -0.5,
                rot=RotaryDims(base=10000.0, dims=rot_dim, scaling=YarnDims(
                    factor=4.0, original=original, fast=32.0, slow=1.0)),
                kv_from=owner if share else None)
            owner = i if owner is None else None
        layers.append(LayerDims(mixer=mixer, mlp=mlp))
    return LayeredDims(arch="kedelorn", vocab_size=vocab, hidden_size=hidden,
                       layers=layers, norm_eps=eps, streams=streams)


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
    # attention beside the delta rule, and linear recurrent layers, of the
    # llama3-8b size; the middle layers run twice
    "tebasun-8b": looped_preset(
        24, 4096, 128256, heads=32, kv_heads=16, dim=128, ff=14336,
        loop=(8, 16, 2),
    ),
    "tebasun-tiny": looped_preset(
        4, 256, 1024, heads=8, kv_heads=4, dim=32, ff=512, order="PR",
        blocks=4, rank=16, side=32, loop=(1, 3, 2), original=64,
    ),
    # retention and latent attention of the llama3-8b size on four
    # streams, every feed-forward routed
    "kedelorn-8b": streamed_preset(
        32, 4096, 128256, heads=32, dim=128, kv_rank=512,
        mlp=GatedExpertsDims(ff=1792, experts=32, top=4, scale=2.0,
                             shared=3584), order="RRLL", share=True,
    ),
    "kedelorn-tiny": streamed_preset(
        4, 192, 1024, heads=6, dim=32, kv_rank=64,
        mlp=GatedExpertsDims(ff=64, experts=6, top=2, shared=128),
        order="RLL", rot_dim=16, share=True, streams=2, original=64,
    ),
}


def get_dims(name: str) -> ModelDims | LayeredDims:
    if name not in PRESETS:
        raise KeyError(
            f"unknown model preset {name!r}; available: {sorted(PRESETS)}"
        )
    return PRESETS[name]
