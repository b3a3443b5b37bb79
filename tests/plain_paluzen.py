"""A plain implementation of the Paluzen decoder, for tests: one function per mechanism, float64, whole sequences at
once (no cache, no state carried between calls, no batching), written from the design's equations and sharing nothing
with the engine.

A model is (config, weights): `config` is the config.json dict, `weights` a dict of float64 tensors by the
checkpoint's names.  `forward(config, weights, tokens)` returns the logits of every position and the residual
stream after every layer that runs (a looped layer counts each time).
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


def noisy(seed, run):
    """run() with every product's input and result moved at random: what 16-bit storage alone does to a result."""
    global NOISE
    NOISE = torch.Generator().manual_seed(seed)
    try:
        return run()
    finally:
        NOISE = None


def silu(z):
    return z * torch.sigmoid(z)


def unit_rms(x, eps):
    """x divided by its root mean square over the last axis, eps inside the root."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def rms_norm(x, weight, eps):
    return unit_rms(x, eps) * weight


def previous(h):
    """h of the token before, zeros before the first: [T, width]."""
    out = torch.zeros_like(h)
    out[1:] = h[:-1]
    return out


def blend(h, mu):
    """h + (h' - h) * mu, element by element, h' the token before's h."""
    return h + (previous(h) - h) * mu


def rotate_halves(x, positions, dims, base):
    """x: [T, heads, dim].  Of the first `dims` dims of every head, dim i turns with dim i + dims / 2 by the
    angle position * base^(-2i / dims); the rest pass."""
    out = x.clone()
    half = dims // 2
    for i in range(half):
        angle = positions.to(F64) * base ** (-2.0 * i / dims)
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
def windowed_attention(mixer, w, prefix, h, positions):
    """Grouped softmax attention over a sliding window; a factor of the scores and a gate on the result, one a head."""
    H, G, dim, vdim = mixer["heads"], mixer["kv_heads"], mixer["dim"], mixer["vdim"]
    T = h.shape[0]
    q = product(h, w[prefix + "q"]).reshape(T, H, dim)
    k = product(h, w[prefix + "k"]).reshape(T, G, dim)
    v = product(h, w[prefix + "v"]).reshape(T, G, vdim)
    rot = mixer.get("rot")
    if rot is not None:
        q = rotate_halves(q, positions, int(rot["dims"]), float(rot["base"]))
        k = rotate_halves(k, positions, int(rot["dims"]), float(rot["base"]))
    size = (mixer.get("mask") or {}).get("size")
    mask = window_mask(T, size)
    gate = torch.sigmoid(product(h, w[prefix + "g"]))                       # [T, H]
    heads = []
    for head in range(H):
        group = head // (H // G)
        scores = q[:, head] @ k[:, group].T * float(mixer["scale"]) * w[prefix + "temp"][head]
        weights = torch.softmax(scores.masked_fill(~mask, -math.inf), dim=-1)
        heads.append(weights @ v[:, group] * gate[:, head:head + 1])
    return product(torch.cat(heads, dim=-1), w[prefix + "o"])


def decayed_state_walk(q, k, v, decay, bonus=None):
    """One head.  q, k, decay: [T, dim] (decay per key channel and token), v: [T, vdim].
    Without bonus: S_t = diag(decay_t) S_(t-1) + k_t v_t^T, o_t = S_t^T q_t.
    With bonus u [dim]: o_t = (S_(t-1) + diag(u) k_t v_t^T)^T q_t, and then the same update of S."""
    T, dim = q.shape
    S = torch.zeros(dim, v.shape[1], dtype=F64)
    out = torch.zeros(T, v.shape[1], dtype=F64)
    for t in range(T):
        outer = k[t][:, None] * v[t][None, :]
        if bonus is not None:
            out[t] = (S + bonus[:, None] * outer).T @ q[t]
            S = decay[t][:, None] * S + outer
        else:
            S = decay[t][:, None] * S + outer
            out[t] = S.T @ q[t]
    return out


def time_mixing(mixer, w, prefix, h, eps):
    """Every projection reads its own blend of the token and the one before it; a decay per head and key channel."""
    H, dim = mixer["heads"], mixer["dim"]
    T = h.shape[0]
    mixed = {name: blend(h, w[prefix + "mu." + name]) for name in "rkvgw"}
    r, k, v = (product(mixed[name], w[prefix + name]).reshape(T, H, dim) for name in "rkv")
    gate = silu(product(mixed["g"], w[prefix + "g"]))
    z = torch.tanh(product(mixed["w"], w[prefix + "w1"])) @ w[prefix + "w2"].T + w[prefix + "w0"]
    decay = torch.exp(-torch.exp(z)).reshape(T, H, dim)
    heads = [unit_rms(decayed_state_walk(r[:, head], k[:, head], v[:, head], decay[:, head], bonus=w[prefix + "u"][head]), eps)
             for head in range(H)]
    return product(torch.cat(heads, dim=-1) * w[prefix + "norm"] * gate, w[prefix + "o"])


def parallel(mixer, w, prefix, h, positions, eps):
    left = windowed_attention(mixer["left"], w, prefix + "left.", h, positions)
    right = time_mixing(mixer["right"], w, prefix + "right.", h, eps)
    return float(mixer["left_scale"]) * left + float(mixer["right_scale"]) * right


# ---- lightning attention ------------------------------------------------------------------------------------
def lightning(mixer, w, prefix, h, positions, eps):
    H, dim, vdim = mixer["heads"], mixer["dim"], mixer["vdim"]
    T = h.shape[0]
    q = silu(product(h, w[prefix + "q"])).reshape(T, H, dim)
    k = silu(product(h, w[prefix + "k"])).reshape(T, H, dim)
    v = silu(product(h, w[prefix + "v"])).reshape(T, H, vdim)
    heads = []
    for head in range(H):
        decay = torch.full((T, dim), float(mixer["decay"][head]), dtype=F64)
        heads.append(decayed_state_walk(q[:, head], k[:, head], v[:, head], decay))
    joined = rms_norm(torch.cat(heads, dim=-1), w[prefix + "norm"], eps)       # all heads together
    return product(joined * torch.sigmoid(product(h, w[prefix + "g"])), w[prefix + "o"])


MIXERS = {"parallel": parallel, "lightning": lightning}


# ---- feed-forward ---------------------------------------------------------------------------------------------
def relu_squared(z):
    return torch.clamp(z, min=0.0) ** 2


def dense(w, prefix, h):
    return product(relu_squared(product(h, w[prefix + "up"])), w[prefix + "down"])


def router_choice(z, correction, top, groups=None):
    """z: [T, n] logits -> (scores [T, n], chosen [T, top], weights [T, top]).  The correction moves the choice only; of
    the groups of neighbours only the `keep` with the largest best choice score may be chosen from."""
    scores = torch.softmax(z, dim=-1)
    choice = scores + correction
    if groups is not None:
        T, n = choice.shape
        size = n // int(groups["count"])
        best = choice.reshape(T, int(groups["count"]), size).amax(dim=-1)
        kept = torch.topk(best, int(groups["keep"]), dim=-1).indices
        open_groups = torch.zeros_like(best, dtype=torch.bool).scatter_(1, kept, True)
        choice = choice.masked_fill(~open_groups.repeat_interleave(size, dim=1), -math.inf)
    chosen = torch.topk(choice, top, dim=-1).indices
    weights = torch.gather(scores, 1, chosen)
    return scores, chosen, weights / (weights.sum(dim=-1, keepdim=True) + 1e-20)


def router_margin(z, correction, top, groups=None):
    """How far each token's choice is from another one ([T]): the smaller of the gap between its `top`-th and its next
    choice score among the experts that can be chosen, and (with groups) the gap between the last kept group's score
    and the first dropped one's."""
    choice = torch.softmax(z, dim=-1) + correction
    T, n = choice.shape
    margin = torch.full((T,), math.inf, dtype=z.dtype)
    if groups is not None and int(groups["keep"]) < int(groups["count"]):
        count, keep = int(groups["count"]), int(groups["keep"])
        best = choice.reshape(T, count, n // count).amax(dim=-1)
        ordered = torch.sort(best, dim=-1, descending=True).values
        margin = torch.minimum(margin, ordered[:, keep - 1] - ordered[:, keep])
        kept = torch.topk(best, keep, dim=-1).indices
        open_groups = torch.zeros_like(best, dtype=torch.bool).scatter_(1, kept, True)
        choice = choice.masked_fill(~open_groups.repeat_interleave(n // count, dim=1), -math.inf)
    ordered = torch.sort(choice, dim=-1, descending=True).values
    if top < n:
        margin = torch.minimum(margin, ordered[:, top - 1] - ordered[:, top])
    return margin


def mixture(mlp, w, prefix, h, margins=None):
    """margins: a list that takes, per call, every token's `router_margin`."""
    router = mlp["router"]
    experts, top = int(router["experts"]), int(router["top"])
    z = product(h, w[prefix + "router"])
    correction = w[prefix + "correction"]
    _, chosen, weights = router_choice(z, correction, top, router.get("groups"))
    if margins is not None:
        margins.append(router_margin(z, correction, top, router.get("groups")))
    out = torch.zeros_like(h)
    for e in range(z.shape[1]):
        share = ((chosen == e).to(F64) * weights).sum(dim=-1, keepdim=True)
        out = out + share * (dense(w, f"{prefix}e{e}.", h) if e < experts else h)       # (the last are identities)
    return out


def feed_forward(mlp, w, prefix, h, margins=None):
    return dense(w, prefix, h) if mlp["kind"] == "dense" else mixture(mlp, w, prefix, h, margins)


# ---- the model ------------------------------------------------------------------------------------------
def run_order(config):
    """[(layer, whether a pass of the loop begins with it)] in the order in which layers run."""
    count = len(config["layers"])
    loop = config.get("loop")
    if loop is None:
        return [(index, False) for index in range(count)]
    start, stop, times = int(loop["start"]), int(loop["stop"]), int(loop["times"])
    one_pass = [(index, index == start) for index in range(start, stop)]
    return [(index, False) for index in range(start)] + one_pass * times + [(index, False) for index in range(stop, count)]


def forward(config, weights, tokens, margins=None):
    """margins: a list that takes every router's margins, one tensor [T] per routed feed-forward that runs."""
    w = weights
    eps = float(config["norm"]["eps"])
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    positions = torch.arange(tokens.shape[0])
    first = w["embed"][tokens]
    x = first
    residuals = []
    for index, enters in run_order(config):
        layer = config["layers"][index]
        prefix = f"l{index}."
        if enters:
            x = product(torch.cat([x, first], dim=-1), w["loop.in"])
        h = blend(rms_norm(x, w[prefix + "norm1"], eps), w[prefix + "shift"])
        x = x + MIXERS[layer["type"]](layer["mixer"], w, prefix + "mix.", h, positions, eps)
        if layer.get("mlp") is not None:
            x = x + feed_forward(layer["mlp"], w, prefix + "mlp.", rms_norm(x, w[prefix + "norm2"], eps), margins)
        residuals.append(x)
    logits = product(rms_norm(x, w["final.norm"], eps), w["embed"])
    cap = config.get("logit_softcap")
    if cap is not None:
        logits = float(cap) * torch.tanh(logits / float(cap))
    return logits, torch.stack(residuals)
