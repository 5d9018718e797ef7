"""Small configurations and random weights of layer-list decoders for the tests."""
import json
import struct

import numpy as np

from kalosm_amd import synth


def rot(dims, base=10000.0, scaled=True):
    r = {"base": base, "dims": dims}
    if scaled:
        r["scaling"] = {"factor": 4.0, "original": 256, "fast": 16.0, "slow": 2.0}
    return r


def latent(heads=3, dim=24, rot_dim=8, vdim=40, kv_rank=72, window=21, scaled=True, scale=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "rot": rot(rot_dim, scaled=scaled),
         "scale": (dim + rot_dim) ** -0.5 if scale is None else scale}
    if window:
        m["mask"] = {"size": window}
    return {"type": "latent_attention", "mixer": m}


def delta(heads=4, kv_heads=2, dim=48, vdim=20, conv=3):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


def mamba2(heads=6, vdim=24, state=40, groups=3, norm_groups=2, conv=2):
    return {"type": "mamba2", "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "norm_groups": norm_groups,
                                        "conv": conv}}


def moe(experts=5, top=3, ff=56, shared=72, scale=1.7):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top, "scale": scale}}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def attention(heads=6, kv_heads=3, dim=20, vdim=12, window=19, keep=5, dims=14, base=5000.0, scale=0.31):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "rot": {"base": base, "dims": dims},
            "mask": {"size": window, "keep_first": keep}}


def pair(left=None, right=None, scales=(0.7, 1.6)):
    return {"type": "parallel", "mixer": {"left": left or attention(), "right": right or {"heads": 5, "dim": 24},
                                          "left_scale": scales[0], "right_scale": scales[1]}}


def retention(heads=3, dim=28, vdim=40, dims=20, base=900.0, decay=None):
    return {"type": "retention", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "rot": {"base": base, "dims": dims},
                                           "decay": decay or [1.0 - 0.5 ** (2 + 3 * i) for i in range(heads)]}}


def dense(ff=90):
    return {"kind": "dense", "ff": ff}


def config_apart(layers, width=150, vocab=110, eps=3e-6, positions=700):
    return {"architecture": "Zovovik", "width": width, "vocab": vocab, "max_positions": positions, "norm": {"eps": eps}, "layers": layers}


def config(layers, width=200, vocab=130, eps=1e-5):
    return {"architecture": "Fidasun", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": layers}


def with_mlp(layer, mlp):
    return dict(layer, mlp=mlp)


CONFIGS = {
    # sizes that are multiples of nothing in particular, a layer without a feed-forward
    "odd": config([with_mlp(latent(), moe()), with_mlp(delta(), moe(shared=0)), with_mlp(mamba2(), None),
                   with_mlp(latent(heads=4, vdim=24, dim=20, rot_dim=12, kv_rank=50, window=7, scaled=False), moe(experts=7, top=1))]),
    # everything that can be one is one
    "ones": config([with_mlp(latent(heads=1, dim=8, rot_dim=2, vdim=8, kv_rank=8, window=1), moe(1, 1, 16, 16, 1.0)),
                    with_mlp(delta(1, 1, 16, 16, 1), moe(2, 1, 8, 0)), with_mlp(mamba2(1, 16, 16, 1, 1, 1), moe(3, 3, 16, 8))],
                   width=64, vocab=40),
    # no window: the cache grows
    "full": config([with_mlp(latent(window=0, heads=2, dim=40, rot_dim=24, vdim=48, kv_rank=56), moe(8, 2, 64, 64)),
                    with_mlp(mamba2(4, 40, 48, 1, 4, 4), moe(8, 2, 64, 64))], width=128, vocab=96),
    # head sizes of large models: the widest operand shapes of every kernel
    "large": config([with_mlp(latent(heads=2, dim=128, rot_dim=64, vdim=128, kv_rank=512, window=70), moe(4, 2, 112, 80)),
                     with_mlp(delta(4, 2, 128, 128, 4), moe(4, 2, 112, 80)), with_mlp(mamba2(4, 64, 128, 2, 2, 4), None),
                     with_mlp(delta(2, 1, 200, 72, 4), None)], width=256, vocab=200),
    # sublayers normed at their end: sizes that divide nothing, every order of mixers, layers without a feed-forward
    "apart": config_apart([with_mlp(retention(), dense()), with_mlp(pair(), dense(77)), with_mlp(retention(1, 10, 9, 4), None),
                           with_mlp(pair(attention(4, 1, 9, 30, 40, 3, 4, scale=0.5), {"heads": 2, "dim": 40}, (1.3, 0.4)), None)]),
    "apart_ones": config_apart([with_mlp(pair(attention(1, 1, 2, 1, 1, 1, 2), {"heads": 1, "dim": 2}, (1.0, 1.0)), dense(1)),
                                with_mlp(retention(1, 2, 1, 2, decay=[0.5]), dense(3))], width=64, vocab=40, eps=1e-3),
    # a window nothing falls out of, no kept tokens
    "apart_full": config_apart([with_mlp(pair(attention(4, 4, 16, 48, 5000, 0, 16), {"heads": 3, "dim": 16}), dense(128)),
                                with_mlp(pair(attention(5, 5, 48, 16, 3, 0, 10), {"heads": 1, "dim": 100}), dense(64))], width=128, vocab=96),
    # head sizes of large models
    "apart_large": config_apart([with_mlp(pair(attention(8, 1, 128, 128, 70, 9, 96, scale=0.08), {"heads": 2, "dim": 128}), dense(320)),
                                 with_mlp(pair(attention(2, 1, 200, 250, 33, 40, 200, scale=0.07), {"heads": 1, "dim": 200}), dense(112)),
                                 with_mlp(retention(2, 256, 128, 256, decay=[0.999, 0.9]), None),
                                 with_mlp(retention(3, 128, 72, 64), dense(200))], width=256, vocab=200),
    # values wider than one block of the attention kernel, latent rows beyond 640
    "wide": config([with_mlp(latent(heads=3, dim=96, rot_dim=32, vdim=160, kv_rank=640, window=37), None)], width=128, vocab=64),
}


def weights(cfg, seed=0):
    """{name: f32 array} of bf16 values."""
    out = {}
    for name, n, k in synth.hybrid_tensor_specs(cfg):
        out[name] = synth.from_bf16_bits(synth.hybrid_random_tensor(name, n, k, seed, cfg["architecture"] == "Fidasun")).reshape((n, k) if k else (n,))
    return out


def round_bf16(x):
    return synth.from_bf16_bits(synth.to_bf16_bits(np.ascontiguousarray(x, np.float32).reshape(-1))).reshape(np.shape(x))


def tensors(w):
    for name, a in w.items():
        yield name, a.shape[0], a.shape[1] if a.ndim == 2 else 0, synth.to_bf16_bits(a.reshape(-1))


def build(dev, cfg, w, dtype="float32", ctx=4096):
    from kalosm_amd.hybrid import HybridModel

    m = HybridModel(dev, cfg, dtype=dtype, ctx=ctx)
    m.load_all(tensors(w))
    return m


def save(path, cfg, w):
    """config.json and model.safetensors of a model folder."""
    (path / "config.json").write_text(json.dumps(cfg))
    header, parts, at = {"__metadata__": {"format": "pt"}}, [], 0
    for name, a in w.items():
        b = synth.to_bf16_bits(a.reshape(-1)).astype("<u2").tobytes()
        header[name] = {"dtype": "BF16", "shape": list(a.shape), "data_offsets": [at, at + len(b)]}
        parts.append(b)
        at += len(b)
    text = json.dumps(header).encode()
    (path / "model.safetensors").write_bytes(struct.pack("<Q", len(text)) + text + b"".join(parts))


def matching_latent(cfg, w, layer, gain, pairs):
    """Makes the attention of `layer` look for partners: for every (x, y) of `pairs` the query of token x points along the
    key of token y, so a visible y takes nearly all of the weight of a position that holds x."""
    c, p = cfg["layers"][layer]["mixer"], f"l{layer}.mix."
    H, dn, dr, R, D = c["heads"], c["dim"], c["rot_dim"], c["kv_rank"], cfg["width"]
    A = np.random.default_rng(5).standard_normal((dn, D)) / np.sqrt(D)
    for x, y in pairs:
        w["embed"][y] = np.roll(w["embed"][x], 1)
    w[f"l{layer}.norm1"][:] = 0.0
    q = w[p + "q"].reshape(H, dn + dr, D).copy()
    q[:, :dn] = gain * np.roll(A, -1, axis=1)  # q(x) = gain A roll(h_x) = gain A h_y
    q[:, dn:] *= 0.1
    w[p + "q"] = round_bf16(q.reshape(H * (dn + dr), D))
    dkv = w[p + "dkv"].copy()
    dkv[:dn] = A
    w[p + "dkv"] = round_bf16(dkv)
    uk = np.zeros((H, dn, R))
    uk[:, np.arange(dn), np.arange(dn)] = 1.0
    w[p + "uk"] = round_bf16(uk.reshape(H * dn, R))
    w[p + "uv"] = round_bf16(w[p + "uv"] * 2.0)
    return w


def matching_attention(cfg, w, layer, gain, pairs):
    """The same for grouped-query attention beside time mixing: queries are `gain` times unit keys of their partners; rotated
    dimensions, positions and the other mixer stay out of it."""
    c, p = cfg["layers"][layer]["mixer"]["left"], f"l{layer}.mix.left."
    d, dims, D = c["dim"], c["rot"]["dims"], cfg["width"]
    A = np.random.default_rng(5).standard_normal((d, D)) / np.sqrt(D)
    A[:dims] = 0.0
    w["pos"][:] = 0.0
    for x, y in pairs:
        w["embed"][y] = np.roll(w["embed"][x], 1)
    w[p + "q"] = round_bf16(np.tile(np.roll(A, -1, axis=1), (c["heads"], 1)))
    w[p + "k"] = round_bf16(np.tile(A, (c["kv_heads"], 1)))
    w[p + "q.norm"][:] = gain
    w[p + "k.norm"][:] = 1.0
    return w


def rel_err(got, want):
    """Root mean square difference of each row over the standard deviation of the wanted rows."""
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    return np.sqrt(np.mean((got - want) ** 2, axis=-1)) / want.std()
