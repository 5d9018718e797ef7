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


def rotated_halves(x, positions, freq):
    """x [..., t, d]: of the first n = 2 len(freq) dimensions, i and i + n / 2 form a pair, turned by position * freq_i."""
    p = np.asarray(positions, np.float32)
    a = (p[:, None] * freq[None, :].astype(np.float32)).astype(np.float64)
    c, s = np.cos(a), np.sin(a)
    out = x.copy()
    n = len(freq)
    u, v = x[..., :n], x[..., n:2 * n]
    out[..., :n] = u * c - v * s
    out[..., n:2 * n] = v * c + u * s
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


# ---------------------------------------------------------------- grouped-query attention with kept first tokens
def kept_window(T, size, keep):
    """visible[i, j]: j not after i, and less than `size` positions behind it or among the first `keep`."""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    return (j <= i) & ((i - j < size) | (j < keep))


def grouped_attention(h, w, c, eps, dtype=np.float64):
    """h [t, width] -> [t, width].  w: q, k, v, q.norm, k.norm, o and (optional) sink."""
    T = h.shape[0]
    H, G, d, dv = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    freq, _ = yarn_frequencies(c["rot"]["base"], c["rot"]["dims"])
    pos = np.arange(T)
    q = rms((h @ w["q"].T).reshape(T, H, d), eps) * w["q.norm"]
    k = rms((h @ w["k"].T).reshape(T, G, d), eps) * w["k.norm"]
    v = (h @ w["v"].T).reshape(T, G, dv)
    m = c.get("mask")
    visible = kept_window(T, m["size"], m.get("keep_first", 0)) if m else kept_window(T, T, 0)
    out = np.zeros((T, H, dv), dtype)
    for n in range(H):
        g = n // (H // G)
        s = rotate_interleaved(q[:, n], pos, freq, 1.0) @ rotate_interleaved(k[:, g], pos, freq, 1.0).T * c["scale"]
        out[:, n] = sink_softmax(s, visible, w["sink"][n] if "sink" in w else -np.inf) @ v[:, g]
    return out.reshape(T, H * dv) @ w["o"].T


# ---------------------------------------------------------------- recurrences without a short convolution
def fixed_decay(q, k, v, decay):
    """One head: the state forgets by a constant factor per token."""
    S = np.zeros((q.shape[1], v.shape[1]), q.dtype)
    out = np.zeros_like(v)
    for t in range(len(q)):
        S = decay * S + np.outer(k[t], v[t])
        out[t] = S.T @ q[t]
    return out


def retention(h, w, c, eps, dtype=np.float64):
    T = h.shape[0]
    H, d, dv = c["heads"], c["dim"], c["vdim"]
    freq, _ = yarn_frequencies(c["rot"]["base"], c["rot"]["dims"])
    q, k, v = ((h @ w[n].T).reshape(T, H, -1) for n in ("q", "k", "v"))
    o = np.zeros((T, H, dv), dtype)
    for n in range(H):
        qr, kr = (rotated_halves(x[:, n], np.arange(T), freq) for x in (q, k))
        o[:, n] = fixed_decay(qr, kr * d ** -0.5, v[:, n], c["decay"][n])
    return (rms(o, eps).reshape(T, H * dv) * silu(h @ w["g"].T)) @ w["o"].T


def channel_decay(r, k, v, g, u):
    """One head: r, k, g [t, d], v [t, e], u [d].  Every key channel forgets at its own rate; the current token's own
    contribution is read with the bonus u before it joins the state."""
    S = np.zeros((r.shape[1], v.shape[1]), r.dtype)
    out = np.zeros_like(v)
    for t in range(len(r)):
        kv = np.outer(k[t], v[t])
        out[t] = (S + u[:, None] * kv).T @ r[t]
        S = g[t][:, None] * S + kv
    return out


def shifted(h, mu):
    """Every channel moved by mu towards the previous token's (zeros ahead of the first)."""
    prev = np.concatenate([np.zeros_like(h[:1]), h[:-1]])
    return h + (prev - h) * mu


def time_mixing(h, w, c, eps, dtype=np.float64):
    """w: r, k, v, g, w1, w2, w0, u, norm, o and mu.r ... mu.w."""
    T = h.shape[0]
    H, d = c["heads"], c["dim"]
    r, k, v = ((shifted(h, w["mu." + n]) @ w[n].T).reshape(T, H, d) for n in ("r", "k", "v"))
    gate = silu(shifted(h, w["mu.g"]) @ w["g"].T)
    z = np.tanh(shifted(h, w["mu.w"]) @ w["w1"].T) @ w["w2"].T + w["w0"]
    g = np.exp(-np.exp(z)).reshape(T, H, d)
    o = np.zeros((T, H, d), dtype)
    for n in range(H):
        o[:, n] = channel_decay(r[:, n], k[:, n], v[:, n], g[:, n], w["u"][n])
    return (rms(o, eps).reshape(T, H * d) * w["norm"] * gate) @ w["o"].T


def side_by_side(h, w, c, eps, dtype=np.float64):
    """Attention and time mixing on the same input, added with their scales."""
    left = grouped_attention(h, _under(w, "left."), c["left"], eps, dtype)
    right = time_mixing(h, _under(w, "right."), c["right"], eps, dtype)
    return c["left_scale"] * left + c["right_scale"] * right


MIXERS = {"latent_attention": latent_attention, "delta": delta, "mamba2": mamba2, "retention": retention,
          "parallel": side_by_side}


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


def dense(h, w, c):
    """Two matrices with the square of relu between them."""
    return np.square(np.maximum(h @ w["up"].T, 0.0)) @ w["down"].T


# ---------------------------------------------------------------- model
def _under(weights, prefix):
    n = len(prefix)
    return {k[n:]: v for k, v in weights.items() if k.startswith(prefix)}


def parallel_residual_layer(x, L, lc, eps, dtype):
    """One norm feeds mixer and feed-forward."""
    h = norm_one_plus(x, L["norm1"], eps)
    y = MIXERS[lc["type"]](h, _under(L, "mix."), lc["mixer"], eps, dtype)
    return x + (y + moe(h, _under(L, "mlp."), lc["mlp"]) if lc.get("mlp") else y)


def output_norm_layer(x, L, lc, eps, dtype):
    """Mixer and feed-forward read the residual stream as it is; what they give is normed before it is added."""
    x = x + rms(MIXERS[lc["type"]](x, _under(L, "mix."), lc["mixer"], eps, dtype), eps) * L["norm1"]
    return x + rms(dense(x, _under(L, "mlp."), lc["mlp"]), eps) * L["norm2"] if lc.get("mlp") else x


def forward(cfg, weights, tokens, dtype=np.float64):
    """Logits of every position [t, vocab] and the residual stream after every layer [layers, t, width]."""
    W = {k: np.asarray(v, dtype) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    zovovik = cfg["architecture"] == "Zovovik"
    layer = output_norm_layer if zovovik else parallel_residual_layer
    x = W["embed"][np.asarray(tokens)]
    if zovovik:
        x = x + W["pos"][:len(x)]
    layers = []
    for i, lc in enumerate(cfg["layers"]):
        x = layer(x, _under(W, f"l{i}."), lc, eps, dtype)
        layers.append(x)
    h = rms(x, eps) * W["final.norm"] if zovovik else norm_one_plus(x, W["final.norm"], eps)
    return h @ W["head"].T, np.stack(layers)
