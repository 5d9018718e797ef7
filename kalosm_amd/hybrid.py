"""Decoders whose configuration lists their layers one by one (csrc/fh_hybrid.hip): latent attention, gated delta rule and
state space mixers with an optional mixture-of-experts feed-forward (Fidasun); retention, and grouped-query attention beside
time mixing, with an optional dense feed-forward (Zovovik).  Weights are bf16 in a safetensors file beside
`config.json`."""
from __future__ import annotations

import ctypes as C
import json
import os
from typing import Callable, Iterable, Optional, Tuple

import numpy as np

from . import synth
from ._lib import DECODER_BF16, F32, check
from .decoder import Decoder
from .fusor import Device

DTYPES = {"bfloat16": DECODER_BF16, "bf16": DECODER_BF16, "float32": F32, "f32": F32}


class HybridModel(Decoder):
    """dtype "bfloat16": operands of the matrix products in bf16, sums, scores, norms, routers, recurrent states and the
    residual stream in 32 bits; "float32": everything in 32 bits."""

    def __init__(self, device: Device, cfg: dict, dtype: str = "bfloat16", ctx: int = 32768):
        h = C.c_void_p()
        check(device._lib.fh_decoder_create(device._h, json.dumps(cfg).encode(), DTYPES[dtype], ctx, C.byref(h)))
        super().__init__(device, h)
        self.cfg = cfg

    @staticmethod
    def open(device: Device, path: str, dtype: str = "bfloat16", ctx: int = 32768) -> "HybridModel":
        """A folder with config.json and model.safetensors."""
        h = C.c_void_p()
        check(device._lib.fh_decoder_open(device._h, os.fspath(path).encode(), DTYPES[dtype], ctx, C.byref(h)))
        m = HybridModel.__new__(HybridModel)
        Decoder.__init__(m, device, h)
        with open(os.path.join(path, "config.json")) as f:
            m.cfg = json.load(f)
        return m

    def load_all(self, tensors: Iterable[Tuple[str, int, int, np.ndarray]]) -> None:
        """(name, n, k, bf16 bit patterns) of every tensor; k is 0 for vectors."""
        for name, n, k, bits in tensors:
            self.load_tensor(name, synth.W_BF16, n, k, bits)
        self.finalize()

    @staticmethod
    def random_init(device: Device, cfg: dict, seed: int = 0, keep: Optional[Callable[[str, np.ndarray], None]] = None,
                    **kw) -> "HybridModel":
        """Random weights, generated tensor by tensor; `keep(name, values)` receives each as f32."""
        m = HybridModel(device, cfg, **kw)
        for name, n, k in synth.hybrid_tensor_specs(cfg):
            bits = synth.hybrid_random_tensor(name, n, k, seed, cfg["architecture"] == "Fidasun")
            m.load_tensor(name, synth.W_BF16, n, k, bits)
            if keep is not None:
                keep(name, synth.from_bf16_bits(bits).reshape((n, k) if k else (n,)))
        m.finalize()
        return m
