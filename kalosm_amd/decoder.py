"""The host-side handle all decoder families share (fh_decoder_* of libfusor_hip.so): forward passes, device-side greedy
and sampled decoding, and `generate`, which chains the two."""
from __future__ import annotations

import ctypes as C
from typing import Optional, Sequence

import numpy as np

from ._lib import check
from .fusor import Device


class Decoder:
    """`handle` is an fh_decoder; `owned` handles are destroyed with the object."""

    def __init__(self, device: Device, handle, owned: bool = True):
        self.device, self._d, self._owned = device, handle, owned

    def _info(self):
        v = [C.c_int32() for _ in range(5)]
        check(self.device._lib.fh_decoder_info(self._d, *[C.byref(x) for x in v]))
        return [x.value for x in v]

    @property
    def vocab(self) -> int:
        return self._info()[0]

    @property
    def d_model(self) -> int:
        return self._info()[1]

    @property
    def n_layers(self) -> int:
        return self._info()[2]

    @property
    def context(self) -> int:
        return self._info()[3]

    @property
    def position(self) -> int:
        """Positions of the current sequence."""
        return self._info()[4]

    def load_tensor(self, name: str, ggml_type: int, n: int, k: int, data: np.ndarray) -> None:
        a = np.ascontiguousarray(data)
        a = a.view(np.uint8).reshape(-1)
        check(self.device._lib.fh_decoder_load_tensor(self._d, name.encode(), ggml_type, n, k, a.ctypes.data_as(C.c_void_p),
                                                      a.nbytes))

    def finalize(self) -> None:
        check(self.device._lib.fh_decoder_finalize(self._d))

    def reset(self) -> None:
        """Ends the sequence; the next forward pass starts at position 0."""
        check(self.device._lib.fh_decoder_reset(self._d))

    def forward(self, tokens, want_hidden: bool = False, want: Optional[Sequence[int]] = None):
        """Model::forward (raw/mod.rs:851-865): logits [vocab] of the last of `tokens`, or [len(want), vocab] of the wanted
        places among them."""
        vocab, d_model = self._info()[:2]
        t = np.ascontiguousarray(tokens, dtype=np.uint32).reshape(-1)
        hidden = np.empty(d_model, np.float32) if want_hidden else None
        places = None if want is None else np.ascontiguousarray(want, dtype=np.int32)
        n = 1 if places is None else places.size
        logits = np.empty((n, vocab), np.float32)
        keep = places if places is not None and places.size else np.zeros(1, np.int32)
        check(self.device._lib.fh_decoder_forward(
            self._d, t.ctypes.data_as(C.c_void_p), t.size, None if places is None else keep.ctypes.data_as(C.c_void_p), n,
            logits.ctypes.data_as(C.c_void_p), None if hidden is None else hidden.ctypes.data_as(C.c_void_p)))
        if places is None:
            logits = logits[0]
        return (logits, hidden) if want_hidden else logits

    def decode_greedy(self, first_token: int, steps: int):
        """Greedy decode of `steps` tokens on the device; returns (token ids, device milliseconds)."""
        out = np.empty(steps, np.uint32)
        ms = C.c_float()
        check(self.device._lib.fh_decoder_decode_greedy(self._d, int(first_token), steps, out.ctypes.data_as(C.c_void_p),
                                                        C.byref(ms)))
        return out, ms.value

    def decode_sampled(self, first_token: int, steps: int, params, randoms, previous_tokens=(), repetition_range: int = 64,
                       mu: Optional[float] = None):
        """Sampled decode of `steps` tokens with the token resident on the device (models/kalosm-llama/src/model/
        inference.rs:38-173).  `params`: GpuStandardSamplerParams or GpuMirostat2SamplerParams (its `random` is
        replaced by `randoms[step]`).  Returns (token ids, device milliseconds, mu after the last step)."""
        out = np.empty(steps, np.uint32)
        rnd = np.ascontiguousarray(randoms, np.float32)
        assert rnd.size >= steps
        prev = np.ascontiguousarray(previous_tokens, np.uint32)
        ms, mu_c = C.c_float(), C.c_float(0.0 if mu is None else mu)
        cp = params.to_c()
        check(self.device._lib.fh_decoder_decode_sampled(
            self._d, int(first_token), steps, C.byref(cp), rnd.ctypes.data_as(C.c_void_p),
            prev.ctypes.data_as(C.c_void_p) if prev.size else None, int(prev.size), int(repetition_range),
            C.byref(mu_c), out.ctypes.data_as(C.c_void_p), C.byref(ms)))
        return out, ms.value, mu_c.value

    def generate(self, prompt, new_tokens: int, params=None, seed: int = 0, mu: float = 10.0, repetition_range: int = 64):
        """`new_tokens` token ids after `prompt` (appended to the current sequence): one prefill pass, then the device-side
        loop - greedy, or sampled when `params` is given.  The first token is picked on the device as well."""
        from .fusor import GpuMirostat2Sampler, GpuMirostat2SamplerParams, Tensor

        prompt = np.ascontiguousarray(prompt, np.uint32).reshape(-1)
        logits = Tensor.from_slice(self.device, self.forward(prompt))
        if params is None:
            first = logits.top_k_pairs_1()
            rest = self.decode_greedy(first, new_tokens - 1)[0] if new_tokens > 1 else np.empty(0, np.uint32)
            return np.concatenate([np.array([first], np.uint32), rest])
        rnd = np.random.default_rng(seed).random(new_tokens).astype(np.float32)
        params.random = float(rnd[0])
        mirostat = isinstance(params, GpuMirostat2SamplerParams)
        tail = prompt[len(prompt) - min(repetition_range, len(prompt)):]
        if mirostat:
            sampler = GpuMirostat2Sampler(self.device, mu)
            first = logits.sample_mirostat2_token(sampler, tail, params)
            mu = sampler.mu
        else:
            first = logits.sample_standard_token(tail, params)
        if first is None:
            raise ValueError("no finite logit to sample from")
        if new_tokens == 1:
            return np.array([first], np.uint32)
        rest, _, _ = self.decode_sampled(first, new_tokens - 1, params, rnd[1:], previous_tokens=prompt,
                                         repetition_range=repetition_range, mu=mu if mirostat else None)
        return np.concatenate([np.array([first], np.uint32), rest])

    def weight_bytes(self) -> int:
        """Bytes of weights a decoded token reads."""
        b = C.c_uint64()
        check(self.device._lib.fh_decoder_weight_bytes(self._d, C.byref(b)))
        return b.value

    def keep_layers(self, on: bool = True) -> None:
        """Keep the residual stream behind every layer of the forward passes (`layer_output`)."""
        check(self.device._lib.fh_decoder_keep_layers(self._d, int(on)))

    def layer_output(self, layer: int, tokens: int) -> np.ndarray:
        """[tokens, d_model] behind `layer` for the last pass (its last portion) of `tokens` tokens."""
        out = np.empty((tokens, self.d_model), np.float32)
        check(self.device._lib.fh_decoder_layer_output(self._d, layer, out.ctypes.data_as(C.c_void_p), out.size))
        return out

    def __del__(self):
        try:
            if self._owned and self._d and self.device._h is not None:
                self.device._lib.fh_decoder_destroy(self._d)
        except Exception:
            pass
