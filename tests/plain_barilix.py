"""A plain implementation of the Barilix decoder, for tests: one function per mechanism, float64, whole sequences at
once (no cache, no state carried between calls, no batching), written from the design's equations and sharing nothing
with the engine.

A model is (config, weights): `config` is the config.json dict, `weights` a dict of float64 tensors by the
checkpoint's names.  `forward(config, weights, tokens)` returns the logits of every position and the residual
stream after every layer.
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64
NOISE = None          # a torch.Generator while `noisy` runs: every product's input and result are then moved by a rounding


def product(x, w):
    """x W^T, W stored [out, in]."""
    if NOISE is None:
        return x @ w.T
    return moved(moved(x) @ w.T)


def moved(x):
    """x, each element moved by as much as rounding to bfloat16 may move it (2^-9 of itself), at random."""
    return x * (1.0 + 2.0 ** -9 * (2.0 * torch.rand(x.shape, generator=NOISE, dtype=F64) - 1.0))


def stored(x):
    """x as a cache or a buffer of 16 bits would give it back, while `noisy` runs."""
    return x if NOISE is None else moved(x)


def noisy(seed, run):
    """run() with every product's input and result, and attention's queries, keys and values, moved at random: what 16-bit
    storage alone does to a result."""
    global NOISE
    NOISE = torch.Generator().manual_seed(seed)
    try:
        return run()
    finally:
        NOISE = None


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.log1p(torch.exp(-z.abs())) + torch.clamp(z, min=0.0)


def unit_rms(x, eps):
    """x divided by its root mean square over the last axis, eps inside the root."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def unit_length(x, eps=1e-6):
    """x divided by its length over the last axis, eps inside the root."""
    return x / torch.sqrt((x * x).sum(dim=-1, keepdim=True) + eps)


def centred_norm(x, weight, eps):
    """(x - mean) / sqrt(variance + eps) * weight."""
    centred = x - x.mean(dim=-1, keepdim=True)
    return unit_rms(centred, eps) * weight


def channel_conv(u, taps):
    """y_t = sum_j taps[:, j] u_(t - n + 1 + j) on each channel, zeros before the first token.  u: [T, channels]."""
    n = taps.shape[1]
    padded = torch.cat([torch.zeros(n - 1, u.shape[1], dtype=F64), u], dim=0)
    out = torch.zeros_like(u)
    for j in range(n):
        out = out + taps[:, j] * padded[j:j + u.shape[0]]
    return out


def frequencies(rot):
    """One a rotated pair: base^(-2i / dims), slowed down for wavelengths that are long beside `original`."""
    dims, base, scaling = int(rot["dims"]), float(rot["base"]), rot.get("scaling")
    out = []
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if scaling is not None:
            factor, low, high, original = (float(scaling[key]) for key in ("factor", "low", "high", "original"))
            wavelength = 2.0 * math.pi / f
            if wavelength > original / low:
                f = f / factor
            elif wavelength >= original / high:
                s = (original / wavelength - low) / (high - low)
                f = (1.0 - s) * f / factor + s * f
        out.append(f)
    return out


def rotate_halves(x, positions, rot):
    """x: [T, heads, dim].  Of the first rot.dims dims of every head, dim i turns with dim i + dims / 2; the rest pass."""
    out, half = x.clone(), int(rot["dims"]) // 2
    for i, f in enumerate(frequencies(rot)):
        angle = positions.to(F64) * f
        cos, sin = torch.cos(angle)[:, None], torch.sin(angle)[:, None]
        u, v = x[..., i], x[..., i + half]
        out[..., i] = u * cos - v * sin
        out[..., i + half] = v * cos + u * sin
    return out


def window_mask(T, size):
    """[T, T]: row i sees column j with 0 <= i - j < size (None: every earlier token)."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    seen = i >= j
    return seen if size is None else seen & (i - j < size)


# ---- the two sides of a `parallel` layer ------------------------------------------------------------------
def conv_attention(mixer, w, prefix, h, positions, eps):
    """Grouped softmax attention over a sliding window; q, k and v pass a short convolution, q and k a norm a head."""
    H, G, dim, vdim = mixer["heads"], mixer["kv_heads"], mixer["dim"], mixer["vdim"]
    T = h.shape[0]

    def projected(name, heads, size):
        return channel_conv(product(h, w[prefix + name]) + w[f"{prefix}{name}.b"], w[f"{prefix}{name}.conv"]).reshape(T, heads, size)
    q = unit_rms(projected("q", H, dim), eps) * w[prefix + "q.norm"]
    k = unit_rms(projected("k", G, dim), eps) * w[prefix + "k.norm"]
    v = projected("v", G, vdim)
    if mixer.get("rot") is not None:
        q, k = rotate_halves(q, positions, mixer["rot"]), rotate_halves(k, positions, mixer["rot"])
    q, k, v = stored(q), stored(k), stored(v)
    mask = window_mask(T, (mixer.get("mask") or {}).get("size"))
    heads = []
    for head in range(H):
        group = head // (H // G)
        scores = (q[:, head] @ k[:, group].T) * float(mixer["scale"])
        heads.append(torch.softmax(scores.masked_fill(~mask, -math.inf), dim=-1) @ v[:, group])
    return product(torch.cat(heads, dim=-1), w[prefix + "o"]) + w[prefix + "o.b"]


def state_space_walk(x, B, C, dt, A, D):
    """One head.  x: [T, vdim]; B, C: [T, N]; dt: [T]; S_t = exp(A dt_t) S_(t-1) + dt_t B_t x_t^T, y_t = S_t^T C_t + D x_t."""
    S = torch.zeros(B.shape[1], x.shape[1], dtype=F64)
    out = torch.zeros_like(x)
    for t in range(x.shape[0]):
        S = torch.exp(A * dt[t]) * S + dt[t] * B[t][:, None] * x[t][None, :]
        out[t] = S.T @ C[t] + D * x[t]
    return out


def state_space(mixer, w, prefix, h, eps):
    H, vdim, N, G = mixer["heads"], mixer["vdim"], mixer["state"], mixer["groups"]
    inner, T = H * vdim, h.shape[0]
    z, xbc, dt = torch.split(product(h, w[prefix + "in"]), [inner, inner + 2 * G * N, H], dim=-1)
    xbc = silu(channel_conv(xbc, w[prefix + "conv"]) + w[prefix + "conv.b"])
    x, B, C = torch.split(xbc, [inner, G * N, G * N], dim=-1)
    x, B, C = x.reshape(T, H, vdim), B.reshape(T, G, N), C.reshape(T, G, N)
    dt = softplus(dt + w[prefix + "dt_bias"])
    heads = [state_space_walk(x[:, head], B[:, head // (H // G)], C[:, head // (H // G)], dt[:, head],
                              -torch.exp(w[prefix + "A_log"][head]), w[prefix + "D"][head]) for head in range(H)]
    y = torch.cat(heads, dim=-1) * silu(z)
    parts = int(mixer["norm_groups"])
    y = unit_rms(y.reshape(T, parts, inner // parts), eps).reshape(T, inner) * w[prefix + "norm"]
    return product(y, w[prefix + "o"])


def parallel(mixer, w, prefix, h, positions, eps):
    left = unit_rms(conv_attention(mixer["left"], w, prefix + "left.", h, positions, eps), eps) * w[prefix + "left.out"]
    right = unit_rms(state_space(mixer["right"], w, prefix + "right.", h, eps), eps) * w[prefix + "right.out"]
    return 0.5 * (left + right)


# ---- the gated delta rule -------------------------------------------------------------------------------------
def delta_walk(q, k, v, g, beta):
    """One head.  q, k: [T, dim]; v: [T, vdim]; g, beta: [T].  The state is decayed, then what it holds under k is moved
    towards v, then it is read."""
    S = torch.zeros(k.shape[1], v.shape[1], dtype=F64)
    out = torch.zeros_like(v)
    for t in range(q.shape[0]):
        S = g[t] * S
        u = beta[t] * (v[t] - S.T @ k[t])
        S = S + k[t][:, None] * u[None, :]
        out[t] = S.T @ q[t]
    return out


def delta(mixer, w, prefix, h, positions, eps):
    H, G, dim, vdim = mixer["heads"], mixer["kv_heads"], mixer["dim"], mixer["vdim"]
    T = h.shape[0]

    def projected(name, heads, size):
        return silu(channel_conv(product(h, w[prefix + name]), w[f"{prefix}{name}.conv"])).reshape(T, heads, size)
    q = unit_length(projected("q", G, dim)) * dim ** -0.5
    k = unit_length(projected("k", G, dim))
    v = projected("v", H, vdim)
    beta = torch.sigmoid(product(h, w[prefix + "b"]))
    g = torch.exp(-torch.exp(w[prefix + "A_log"]) * softplus(product(h, w[prefix + "a"]) + w[prefix + "dt_bias"]))
    gate = silu(product(h, w[prefix + "g"])).reshape(T, H, vdim)
    heads = []
    for head in range(H):
        group = head // (H // G)
        o = delta_walk(q[:, group], k[:, group], v[:, head], g[:, head], beta[:, head])
        heads.append(unit_rms(o, eps) * w[prefix + "norm"] * gate[:, head])
    return product(torch.cat(heads, dim=-1), w[prefix + "o"])


MIXERS = {"parallel": parallel, "delta": delta}


# ---- feed-forward ---------------------------------------------------------------------------------------------
def dense(w, prefix, h):
    return product(silu(product(h, w[prefix + "gate"])) * product(h, w[prefix + "up"]), w[prefix + "down"])


def mixture(mlp, w, prefix, h, tokens):
    """A token's id names its experts; each counts the same."""
    table = w[prefix + "table"].long()[tokens]                        # [T, top]
    out = torch.zeros_like(h)
    for e in range(int(mlp["router"]["experts"])):
        used = (table == e).any(dim=-1)
        if bool(used.any()):
            out[used] = out[used] + dense(w, f"{prefix}e{e}.", h[used]) / float(table.shape[1])
    if mlp.get("shared") is not None:
        out = out + dense(w, prefix + "shared.", h)
    return out


def feed_forward(mlp, w, prefix, h, tokens):
    return dense(w, prefix, h) if mlp["kind"] == "dense" else mixture(mlp, w, prefix, h, tokens)


# ---- the model ------------------------------------------------------------------------------------------
def forward(config, weights, tokens):
    w, eps = weights, float(config["norm"]["eps"])
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    positions = torch.arange(tokens.shape[0])
    x = w["embed"][tokens] * float(config["embedding"]["scale"])
    residuals = []
    for index, layer in enumerate(config["layers"]):
        prefix = f"l{index}."
        x = x + centred_norm(MIXERS[layer["type"]](layer["mixer"], w, prefix + "mix.", x, positions, eps), w[prefix + "norm1"], eps)
        if layer.get("mlp") is not None:
            x = x + centred_norm(feed_forward(layer["mlp"], w, prefix + "mlp.", x, tokens), w[prefix + "norm2"], eps)
        residuals.append(x)
    return product(centred_norm(x, w["final.norm"], eps), w["head"]), torch.stack(residuals)
