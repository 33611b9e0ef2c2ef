"""Opens a text decoder from what holds its weights: a model folder (config.json names the design, which the library's registry
looks up) or the reference's moondream.bin."""
from __future__ import annotations

import os

from . import _lib as L
from . import text_model, weights
from .context import Context


def designs() -> list[str]:
    """Designs a model folder may name."""
    return L.load().moon_text_designs().decode().split(", ")


def open_text_model(path: str, dtype: str | None = None, max_seq: int = 2048, ctx: Context | None = None) -> text_model.TextModel:
    """dtype: "bfloat16" (default) or "float32" for a model folder; moondream.bin is f16 and takes none."""
    if os.path.isdir(path):
        return text_model.TextModel.open(path, dtype or "bfloat16", max_seq, ctx)
    if dtype is not None:
        raise ValueError("moondream.bin runs in f16 only")
    with weights.BinFile(path) as f:
        return text_model.TextModel(text_model.make_config(max_seq=max_seq), weights=f, ctx=ctx)
