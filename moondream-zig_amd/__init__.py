"""moondream-zig FP16 matmul + attention hot path on MI355X (gfx950).

A thin host layer over libmoonhip.so (C ABI in include/moonhip.h) that mirrors the
reference's src/core op modules: hgemm, hgemm_trans, attention, rope, ops, plus the
device-resident TextModel / VisionModel sessions; registry opens a decoder from whatever holds its weights.  No CPU fallback exists.
"""
from . import _lib, attention, hgemm, hgemm_trans, ops, registry, rope, sampling, text_model, vision_model, weights  # noqa: F401
from .context import (Context, DeviceBuffer, HipError, IncompatibleTensorShapes, InvalidArgument, InvalidEpsilon,  # noqa: F401
                      InvalidRotationDimension, InvalidTensorDimension, MoonError, NoDevice, OutOfMemory, SequenceTooLong,
                      TokenIdOutOfBounds, default_context)
