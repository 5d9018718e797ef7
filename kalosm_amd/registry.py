"""Model files to decoders, by the architecture a file names: `llama` in GGUF files, the architectures of
csrc/fh_hybrid.hip in folders with config.json and model.safetensors."""
from __future__ import annotations

import json
import os
from typing import Callable, Dict

from .decoder import Decoder
from .fusor import Device


def _llama(device: Device, path: str, dtype: str, ctx: int) -> Decoder:
    from .llama import Model

    if dtype == "float32":
        # quantised weights against activations split into two f16 terms: f32 accuracy, but not 32-bit products
        raise ValueError("GGUF models have no 32-bit mode")
    return Model.from_gguf(device, path, ctx=ctx)


def _hybrid(device: Device, path: str, dtype: str, ctx: int) -> Decoder:
    from .hybrid import HybridModel

    return HybridModel.open(device, path, dtype=dtype, ctx=ctx)


ARCHITECTURES: Dict[str, Callable[[Device, str, str, int], Decoder]] = {"llama": _llama, "Fidasun": _hybrid, "Zovovik": _hybrid}


def architecture(path: str) -> str:
    """The architecture of a GGUF file or of a folder with config.json."""
    if os.path.isdir(path):
        with open(os.path.join(path, "config.json")) as f:
            return json.load(f)["architecture"]
    from .gguf import GgufMetadata

    return GgufMetadata.read(path).get_value("general.architecture")


def load(device: Device, path: str, dtype: str = "bfloat16", ctx: int = 32768) -> Decoder:
    name = architecture(path)
    if name not in ARCHITECTURES:
        raise ValueError(f"unknown architecture {name!r} (known: {', '.join(sorted(ARCHITECTURES))})")
    return ARCHITECTURES[name](device, os.fspath(path), dtype, ctx)
