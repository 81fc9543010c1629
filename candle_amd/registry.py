"""Which model class serves a checkpoint: a folder with config.json and model.safetensors, or a GGUF file."""
from __future__ import annotations

import json
import os


def _venizen():
    from .venizen import Model
    return Model


def _kudurax():
    from .kudurax import Model
    return Model


# config.json "architecture" -> class with from_pretrained(path, device, dtype, ctx)
ARCHITECTURES = {"Venizen": _venizen, "Kudurax": _kudurax}


def load_model(path: str, device="cuda:0", dtype: str = "bfloat16", ctx: int = 4096):
    """The model at ``path``.  Folders are dispatched on config.json's architecture; a file is read as GGUF (llama), whose block formats fix its
    precision."""
    if os.path.isdir(path):
        with open(os.path.join(path, "config.json")) as f:
            arch = json.load(f).get("architecture")
        if arch not in ARCHITECTURES:
            raise ValueError(f"{path}: unknown architecture {arch!r} (known: {', '.join(sorted(ARCHITECTURES))})")
        return ARCHITECTURES[arch]().from_pretrained(path, device=device, dtype=dtype, ctx=ctx)
    from . import gguf_file
    from .quantized_llama import ModelWeights
    with open(path, "rb") as f:
        return ModelWeights.from_gguf(gguf_file.Content.read(f), f, device, ctx=ctx)
