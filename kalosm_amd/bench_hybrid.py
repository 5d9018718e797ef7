"""Prefill and decode throughput of layer-list decoders at layer sizes of real models (random weights), beside the Llama
decoder at equal width, depth and active feed-forward length (`bench.py --hybrid`: Fidasun; `bench.py --zovovik`: Zovovik,
beside Fidasun as well)."""
from __future__ import annotations

import statistics
import time

import numpy as np

from . import synth
from .hybrid import HybridModel
from .llama import Model

HBM_PEAK, MFMA_PEAK = 8e12, 2.5e15


def config(width: int, heads: int, experts: int, top: int, ff: int, window: int, groups: int, vocab: int = 32768) -> dict:
    """Four layers: latent attention, gated delta rule, latent attention, state space, all with experts."""
    rot = {"base": 10000.0, "dims": 64, "scaling": {"factor": 4.0, "original": 4096, "fast": 32.0, "slow": 1.0}}
    latent = {"type": "latent_attention",
              "mixer": {"heads": heads, "dim": 128, "rot_dim": 64, "vdim": 128, "kv_rank": 512, "scale": 192 ** -0.5,
                        "mask": {"size": window}, "rot": rot}}
    delta = {"type": "delta", "mixer": {"heads": heads, "kv_heads": heads // 2, "dim": 128, "vdim": 128, "conv": 4}}
    mamba = {"type": "mamba2", "mixer": {"heads": width * 2 // 64, "vdim": 64, "state": 128, "groups": groups, "conv": 4,
                                         "norm_groups": groups}}
    mlp = {"kind": "moe", "expert": {"ff": ff}, "shared": {"ff": ff},
           "router": {"experts": experts, "top": top, "scale": 1.0}}
    return {"architecture": "Fidasun", "width": width, "vocab": vocab, "norm": {"eps": 1e-6},
            "layers": [dict(l, mlp=mlp) for l in (latent, delta, latent, mamba)]}


def zovovik_config(width: int, heads: int, ff: int, window: int, vocab: int = 32768) -> dict:
    """Four layers: attention beside time mixing, retention, and the same again, all with a dense feed-forward."""
    left = {"heads": heads, "kv_heads": heads // 4, "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "rot": {"base": 500000.0, "dims": 128},
            "mask": {"size": window, "keep_first": 64}}
    pair = {"type": "parallel", "mixer": {"left": left, "right": {"heads": width // 64, "dim": 64}, "left_scale": 1.0, "right_scale": 1.0}}
    ret = {"type": "retention", "mixer": {"heads": width // 256, "dim": 256, "vdim": 256, "rot": {"base": 10000.0, "dims": 256},
                                          "decay": [1.0 - 2.0 ** (-5 - 0.5 * i) for i in range(width // 256)]}}
    return {"architecture": "Zovovik", "width": width, "vocab": vocab, "max_positions": 8192, "norm": {"eps": 1e-6},
            "layers": [dict(l, mlp={"kind": "dense", "ff": ff}) for l in (pair, ret, pair, ret)]}


ZOVOVIK = {"w2048": dict(width=2048, heads=16, ff=8192, window=1024), "w4096": dict(width=4096, heads=32, ff=14336, window=4096)}

SIZES = {"w2048": dict(width=2048, heads=16, experts=64, top=6, ff=1024, window=1024, groups=2),
         "w4096": dict(width=4096, heads=32, experts=32, top=4, ff=2048, window=4096, groups=8)}


def llama_config(c: dict, heads: int, top: int, ff: int) -> dict:
    return dict(n_layers=len(c["layers"]), d_model=c["width"], n_heads=heads, n_kv_heads=heads // 4, head_dim=128,
                ffn=(top + 1) * ff, vocab=c["vocab"], ctx=8192, eps=1e-5, theta=500000.0)


def matrix_flops(c: dict, tokens: int) -> float:
    """Multiply-adds x 2 of the weight matrices of a prompt (routed experts: the chosen ones), without the head."""
    f = 0.0
    for name, n, k in synth.hybrid_tensor_specs(c):
        if not k or name in ("embed", "head", "pos") or name.endswith("conv") or name.endswith(".u"):
            continue
        part = name.split(".")
        if len(part) > 2 and part[1] == "mlp" and part[2].startswith("e") and part[2][1:].isdigit():
            mlp = c["layers"][int(part[0][1:])]["mlp"]
            f += 2.0 * n * k * mlp["router"]["top"] / mlp["router"]["experts"]
        else:
            f += 2.0 * n * k
    return f * tokens


def _model(dev, c: dict) -> HybridModel:
    """Random weights; the experts of all layers share their values (not their memory) to keep the set-up short."""
    m, cache = HybridModel(dev, c, ctx=8192), {}

    def tensors():
        for name, n, k in synth.hybrid_tensor_specs(c):
            part = name.split(".")
            key = (part[-1], n, k) if len(part) == 4 and part[1] == "mlp" else name
            if key not in cache:
                bits = synth.hybrid_random_tensor(name, n, k, 1, c["architecture"] == "Fidasun")
                if key == name:
                    yield name, n, k, bits
                    continue
                cache[key] = bits
            yield name, n, k, cache[key]

    m.load_all(tensors())
    return m


def _measure(m, prompt, steps: int, repeats: int):
    pre, dec = [], []
    for rep in range(repeats + 1):  # the first round warms up and captures the decode step
        m.reset()
        t0 = time.perf_counter()
        lg = m.forward(prompt)
        pre.append(time.perf_counter() - t0)
        _, ms = m.decode_greedy(int(np.argmax(lg)), steps)
        dec.append(ms / steps)
    return statistics.median(pre[1:]), statistics.median(dec[1:])


def run(dev, prompts=(512, 2048), steps: int = 64, repeats: int = 5, only: str = "", zovovik: bool = False) -> dict:
    out = {}
    for name, s in SIZES.items():
        if only and name != only:
            continue
        c = config(**s)
        lc = llama_config(c, s["heads"], s["top"], s["ff"])
        rng = np.random.default_rng(1)
        res = {"config": s, "layers": [l["type"] for l in c["layers"]], "llama": {k: lc[k] for k in ("n_heads", "n_kv_heads", "ffn")},
               "dtype": {"Fidasun": "bf16 weights", "llama": "Q4_K_M weights"}, "runs": []}
        models, configs = {"Fidasun": _model(dev, c)}, {"Fidasun": c}
        if zovovik:
            configs["Zovovik"] = zovovik_config(**ZOVOVIK[name])
            models["Zovovik"] = _model(dev, configs["Zovovik"])
            res["dtype"]["Zovovik"], res["zovovik"] = "bf16 weights", ZOVOVIK[name]
            res["zovovik_layers"] = [l["type"] for l in configs["Zovovik"]["layers"]]
        models["llama"] = Model.random_init(dev, lc, seed=1, sigma=1e-4)
        for n in prompts:
            prompt = rng.integers(0, c["vocab"], n)
            for kind, m in models.items():
                pre, dec = _measure(m, prompt, steps, repeats)
                wb = m.weight_bytes()
                r = {"model": kind, "prompt": n, "prefill_ms": round(pre * 1e3, 3), "prefill_tok_per_s": round(n / pre, 1),
                     "decode_ms": round(dec, 4), "decode_tok_per_s": round(1e3 / dec, 1), "weight_bytes_per_token": wb,
                     "decode_frac_hbm_peak": round(wb / (dec * 1e-3) / HBM_PEAK, 4)}
                if kind in configs:
                    fl = matrix_flops(configs[kind], n)
                else:
                    D, H, K, F = lc["d_model"], lc["n_heads"] * 128, lc["n_kv_heads"] * 128, lc["ffn"]
                    fl = 2.0 * n * lc["n_layers"] * (D * (H + 2 * K) + H * D + 3 * D * F)
                r["prefill_matrix_frac_mfma_peak"] = round(fl / pre / MFMA_PEAK, 4)
                res["runs"].append(r)
        models.clear()
        out[name] = res
    return out
