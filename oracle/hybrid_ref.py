"""Plain numpy restatement of the layer-list decoders (`kalosm_amd.hybrid`): one function per mechanism, token by token
where the mechanism is a recurrence, whole score rows where it is attention.  It is slow and has no cache, no portions
and no batching: a sequence goes in, every position's result comes out.  The tests compare the HIP path with it; it
shares no code with the product.

Arrays are float64 by default (`dtype`), so that what is left of a difference is the product's own rounding."""
from __future__ import annotations

import math

import numpy as np


def silu(z):
    return z / (1.0 + np.exp(-z))


def softplus(z):
    return np.logaddexp(z, 0.0)


def rms(x, eps):
    """x over its root mean square along the last axis, eps inside the root."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def norm_one_plus(x, w, eps):
    """RMS norm whose weight is stored as its distance from one."""
    return rms(x, eps) * (1.0 + w)


# ---------------------------------------------------------------- rotation
def yarn_frequencies(base, dims, scaling=None):
    """Angular frequency of every rotated pair and the factor on cos and sin.  With a scaling (factor, original, fast,
    slow) pairs that turn often inside the original context keep their frequency, slow ones are stretched by `factor`,
    and a linear ramp over the pair index joins the two."""
    f = np.array([float(base) ** (-2.0 * i / dims) for i in range(dims // 2)])
    if not scaling:
        return f, 1.0

    def pair_of(turns):
        return dims * math.log(scaling["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(pair_of(scaling["fast"])), 0)
    hi = min(math.ceil(pair_of(scaling["slow"])), dims - 1)
    ramp = np.clip((np.arange(dims // 2) - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / scaling["factor"] * ramp + f * (1.0 - ramp), 0.1 * math.log(scaling["factor"]) + 1.0


def rotate_interleaved(x, positions, freq, amp, angle32=True):
    """x [..., t, d]: pairs (2i, 2i + 1) of the first 2 len(freq) dimensions turned by position * freq_i, times amp."""
    p = np.asarray(positions, np.float64)
    a = p[:, None] * freq[None, :]
    if angle32:
        a = (p[:, None].astype(np.float32) * freq[None, :].astype(np.float32)).astype(np.float64)
    c, s = np.cos(a) * amp, np.sin(a) * amp
    out = x.copy()
    n = 2 * len(freq)
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    out[..., 0:n:2] = u * c - v * s
    out[..., 1:n:2] = v * c + u * s
    return out


# ---------------------------------------------------------------- latent attention
def sink_softmax(scores, visible, sink):
    """Softmax over the visible keys of each row with exp(sink) added to the denominator."""
    z = np.where(visible, scores, -np.inf)
    m = np.maximum(z.max(axis=-1, keepdims=True), sink)
    e = np.exp(z - m)
    return e / (e.sum(axis=-1, keepdims=True) + np.exp(sink - m))


def latent_attention(h, w, c, eps, dtype=np.float64):
    """h [t, width] -> [t, width].  w: q, dkv, dkv.norm, uk, uv, o and (optional) sink."""
    T = h.shape[0]
    H, dn, dr, dv, R = c["heads"], c["dim"], c["rot_dim"], c["vdim"], c["kv_rank"]
    rot = c["rot"]
    freq, amp = yarn_frequencies(rot["base"], rot["dims"], rot.get("scaling"))
    pos = np.arange(T)
    q = (h @ w["q"].T).reshape(T, H, dn + dr)
    dkv = h @ w["dkv"].T
    lat = rms(dkv[:, :R], eps) * w["dkv.norm"]
    kr = rotate_interleaved(dkv[:, R:], pos, freq, amp)
    k = (lat @ w["uk"].T).reshape(T, H, dn)
    v = (lat @ w["uv"].T).reshape(T, H, dv)
    i, j = pos[:, None], pos[None, :]
    visible = j <= i
    if c.get("mask"):
        visible &= i - j < c["mask"]["size"]
    out = np.zeros((T, H, dv), dtype)
    for n in range(H):
        qr = rotate_interleaved(q[:, n, dn:], pos, freq, amp)
        s = (q[:, n, :dn] @ k[:, n].T + qr @ kr.T) * c["scale"]
        sink = w["sink"][n] if "sink" in w else -np.inf
        out[:, n] = sink_softmax(s, visible, sink) @ v[:, n]
    return out.reshape(T, H * dv) @ w["o"].T


# ---------------------------------------------------------------- recurrent mixers
def short_conv(x, taps_w, bias=None):
    """Depthwise causal convolution, x [t, ch], taps_w [ch, taps] with the oldest tap first."""
    T, K = x.shape[0], taps_w.shape[1]
    out = np.zeros_like(x)
    for t in range(T):
        for i in range(K):
            p = t - (K - 1) + i
            if p >= 0:
                out[t] += x[p] * taps_w[:, i]
    return out if bias is None else out + bias


def unit(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + 1e-6)


def gated_delta(q, k, v, g, beta):
    """One head: q, k [t, d], v [t, e], g, beta [t].  Decay, correct the value stored under the key by beta, read."""
    S = np.zeros((q.shape[1], v.shape[1]), q.dtype)
    out = np.zeros_like(v)
    for t in range(len(q)):
        S = g[t] * S
        u = beta[t] * (v[t] - S.T @ k[t])
        S = S + np.outer(k[t], u)
        out[t] = S.T @ q[t]
    return out


def delta(h, w, c, eps, dtype=np.float64):
    T = h.shape[0]
    H, HK, d, dv = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    pre = {n: silu(short_conv(h @ w[n].T, w[n + ".conv"])) for n in ("q", "k", "v")}
    q = unit(pre["q"].reshape(T, HK, d)) * d ** -0.5
    k = unit(pre["k"].reshape(T, HK, d))
    v = pre["v"].reshape(T, H, dv)
    beta = 1.0 / (1.0 + np.exp(-(h @ w["b"].T)))
    g = np.exp(-np.exp(w["A_log"]) * softplus(h @ w["a"].T + w["dt_bias"]))
    o = np.zeros((T, H, dv), dtype)
    for n in range(H):
        n2 = n // (H // HK)
        o[:, n] = gated_delta(q[:, n2], k[:, n2], v[:, n], g[:, n], beta[:, n])
    o = rms(o, eps) * w["norm"] * silu(h @ w["g"].T).reshape(T, H, dv)
    return o.reshape(T, H * dv) @ w["o"].T


def state_space(x, B, C, dt, A_log, D):
    """One head: x [t, e], B, C [t, N], dt [t]."""
    S = np.zeros((B.shape[1], x.shape[1]), x.dtype)
    y = np.zeros_like(x)
    for t in range(len(x)):
        S = np.exp(-np.exp(A_log) * dt[t]) * S + dt[t] * np.outer(B[t], x[t])
        y[t] = S.T @ C[t] + D * x[t]
    return y


def mamba2(h, w, c, eps, dtype=np.float64):
    T = h.shape[0]
    H, dv, N, G = c["heads"], c["vdim"], c["state"], c["groups"]
    inner = H * dv
    p = h @ w["in"].T
    z, xbc, dt = p[:, :inner], p[:, inner:2 * inner + 2 * G * N], p[:, 2 * inner + 2 * G * N:]
    xbc = silu(short_conv(xbc, w["conv"], w["conv.b"]))
    x = xbc[:, :inner].reshape(T, H, dv)
    B = xbc[:, inner:inner + G * N].reshape(T, G, N)
    C = xbc[:, inner + G * N:].reshape(T, G, N)
    dt = softplus(dt + w["dt_bias"])
    y = np.zeros((T, H, dv), dtype)
    for n in range(H):
        g = n // (H // G)
        y[:, n] = state_space(x[:, n], B[:, g], C[:, g], dt[:, n], w["A_log"][n], w["D"][n])
    y = y.reshape(T, inner) * silu(z)
    y = rms(y.reshape(T, c["norm_groups"], -1), eps).reshape(T, inner) * w["norm"]
    return y @ w["o"].T


MIXERS = {"latent_attention": latent_attention, "delta": delta, "mamba2": mamba2}


# ---------------------------------------------------------------- feed-forward
def expert(h, gate, up, down):
    return (silu(h @ gate.T) * (h @ up.T)) @ down.T


def route(z, top, scale):
    """The `top` experts by softmax score, best first, and scale times those scores."""
    e = np.exp(z - z.max())
    s = e / e.sum()
    idx = np.argsort(-s, kind="stable")[:top]
    return idx, s[idx] * scale


def moe(h, w, c):
    r = c["router"]
    out = np.zeros((h.shape[0], w["e0.down"].shape[0]), h.dtype)
    z = h @ w["router"].T
    for t in range(h.shape[0]):
        idx, s = route(z[t], r["top"], r["scale"])
        for e, wt in zip(idx, s):
            out[t] += wt * expert(h[t], w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"])
    if c.get("shared"):
        out += expert(h, w["shared.gate"], w["shared.up"], w["shared.down"])
    return out


# ---------------------------------------------------------------- model
def _under(weights, prefix):
    n = len(prefix)
    return {k[n:]: v for k, v in weights.items() if k.startswith(prefix)}


def forward(cfg, weights, tokens, dtype=np.float64):
    """Logits of every position [t, vocab] and the residual stream after every layer [layers, t, width]."""
    W = {k: np.asarray(v, dtype) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    x = W["embed"][np.asarray(tokens)]
    layers = []
    for i, lc in enumerate(cfg["layers"]):
        L = _under(W, f"l{i}.")
        h = norm_one_plus(x, L["norm1"], eps)
        y = MIXERS[lc["type"]](h, _under(L, "mix."), lc["mixer"], eps, dtype)
        if lc.get("mlp"):
            y = y + moe(h, _under(L, "mlp."), lc["mlp"])
        x = x + y
        layers.append(x)
    return norm_one_plus(x, W["final.norm"], eps) @ W["head"].T, np.stack(layers)
