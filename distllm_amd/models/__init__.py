"""Native MI355X model family + factory."""

from __future__ import annotations

import torch

from .bert import BertEncoder
from .bufulorn import BufulornModel
from .config import (PRESETS, LayeredDims, ModelDims, dims_from_checkpoint,
                     get_dims)
from .esm import Esm2Encoder, EsmCEncoder
from .kanotar import KanotarModel
from .kedelorn import KedelornModel
from .mistral import DecoderModel
from .tebasun import TebasunModel

__all__ = [
    "BertEncoder",
    "BufulornModel",
    "DecoderModel",
    "Esm2Encoder",
    "EsmCEncoder",
    "KanotarModel",
    "KedelornModel",
    "LayeredDims",
    "ModelDims",
    "PRESETS",
    "TebasunModel",
    "build_model",
    "dims_from_checkpoint",
    "get_dims",
    "load_pretrained",
]


# decoders that are described layer by layer
LAYERED = {"kanotar": KanotarModel, "bufulorn": BufulornModel,
           "tebasun": TebasunModel, "kedelorn": KedelornModel}


def build_model(name_or_dims: str | ModelDims | LayeredDims, device: str | None = None,
                dtype=torch.bfloat16, **kw):
    dims = (
        get_dims(name_or_dims)
        if isinstance(name_or_dims, str)
        else name_or_dims
    )
    if dims.arch == "bert":
        m = BertEncoder(dims, dtype=dtype, **kw)
    elif dims.arch == "esm2":
        m = Esm2Encoder(dims, dtype=dtype, **kw)
    elif dims.arch == "esmc":
        m = EsmCEncoder(dims, dtype=dtype, **kw)
    elif dims.arch in ("mistral", "llama", "qwen2"):
        m = DecoderModel(dims, dtype=dtype, **kw)
    elif dims.arch in LAYERED:
        # parameters are made where they stay: no host copy of the model
        with torch.device(device or "cpu"):
            m = LAYERED[dims.arch](dims, dtype=dtype, **kw)
    else:
        raise ValueError(f"unknown arch {dims.arch}")
    if device is not None:
        m = m.to(device)
    m.eval()
    return m


def load_pretrained(path, device: str | None = None, dtype=torch.bfloat16,
                    **kw):
    """Model of a checkpoint folder whose config.json describes it in
    full (the file's architecture names the model class)."""
    from .loader import load_weights

    dims = dims_from_checkpoint(path)
    if dims is None:
        raise ValueError(f"{path}/config.json names no known architecture")
    model = build_model(dims, device=device, dtype=dtype, **kw)
    load_weights(model, path)
    return model
