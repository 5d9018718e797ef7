"""Command line: `python -m kalosm_amd info MODEL`, `python -m kalosm_amd generate MODEL --tokens 1,2,3 --new 32`.
MODEL is a GGUF file or a folder with config.json and model.safetensors.  There is no tokenizer: token ids go in and
come out."""
from __future__ import annotations

import argparse
import json
import sys
import time


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="python -m kalosm_amd")
    sub = ap.add_subparsers(dest="command", required=True)
    for name in ("info", "generate"):
        p = sub.add_parser(name)
        p.add_argument("model", help="GGUF file, or folder with config.json and model.safetensors")
        p.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
        p.add_argument("--ctx", type=int, default=8192, help="context length")
    p.add_argument("--tokens", required=True, help="prompt: token ids separated by commas")
    p.add_argument("--new", type=int, default=16, help="tokens to generate")
    p.add_argument("--sampler", choices=("greedy", "standard", "mirostat2"), default="greedy")
    p.add_argument("--top-k", type=int, default=64)
    p.add_argument("--temperature", type=float, default=0.8)
    p.add_argument("--repetition-penalty", type=float, default=1.3)
    p.add_argument("--top-p", type=float, default=1.0)
    p.add_argument("--min-p", type=float, default=0.0)
    p.add_argument("--seed", type=int, default=0)
    a = ap.parse_args(argv)

    from . import registry
    from .fusor import Device, GpuMirostat2SamplerParams, GpuStandardSamplerParams

    dev = Device.gpu(0)
    m = registry.load(dev, a.model, dtype=a.dtype, ctx=a.ctx)
    if a.command == "info":
        print(json.dumps({"architecture": registry.architecture(a.model), "layers": m.n_layers, "width": m.d_model,
                          "vocab": m.vocab, "context": m.context, "weight_bytes_per_token": m.weight_bytes(),
                          "device": dev.info()["name"]}))
        return 0
    params = None
    if a.sampler == "standard":
        params = GpuStandardSamplerParams(a.top_k, a.temperature, a.repetition_penalty, a.top_p, a.min_p, 0.0)
    elif a.sampler == "mirostat2":
        params = GpuMirostat2SamplerParams(a.top_k, a.temperature, a.repetition_penalty, 5.0, 0.1, 0.0)
    t0 = time.perf_counter()
    ids = m.generate([int(t) for t in a.tokens.split(",")], a.new, params, seed=a.seed)
    print(json.dumps({"tokens": [int(t) for t in ids], "seconds": round(time.perf_counter() - t0, 3)}))
    return 0


if __name__ == "__main__":
    sys.exit(main())
