"""Opens a text decoder from what holds its weights: a model folder (config.json names the design, which the library's registry
looks up) or the reference's moondream.bin."""
from __future__ import annotations

import ctypes as C
import os

from . import _lib as L
from . import text_model, weights
from .context import Context


def designs() -> list[str]:
    """Designs a model folder may name."""
    return L.load().moon_text_designs().decode().split(", ")


def check_folder(path: str) -> tuple[str, int]:
    """Reads a model folder and checks its tensors against its configuration (no device needed) -> (design, number of layers)."""
    design, layers, err = C.c_char_p(), C.c_size_t(), C.create_string_buffer(512)
    rc = L.load().moon_text_folder_check(os.fsencode(path), C.byref(design), C.byref(layers), err, len(err))
    if rc != L.OK:
        weights._raise(rc, err)
    return design.value.decode(), layers.value


def open_text_model(path: str, dtype: str | None = None, max_seq: int = 2048, ctx: Context | None = None) -> text_model.TextModel:
    """dtype: "bfloat16" (default) or "float32" for a model folder; moondream.bin is f16 and takes none."""
    if os.path.isdir(path):
        return text_model.TextModel.open(path, dtype or "bfloat16", max_seq, ctx)
    if dtype is not None:
        raise ValueError("moondream.bin runs in f16 only")
    with weights.BinFile(path) as f:
        return text_model.TextModel(text_model.make_config(max_seq=max_seq), weights=f, ctx=ctx)
