"""What the Barilix tests share: configurations of their own, model folders of random weights, and the comparison with
the plain implementation.

The configurations differ from each other in every size and option, and use values that make faults visible: fewer
key/value heads than heads (down to one), value heads of another size than the keys, windows that are no multiple of a page
(1, 7, 37 positions on pages of 16) and none, rotations over a part of a head, over all of it and none, frequencies that a
scaling keeps, slows down and blends, convolutions of one to eight taps (other numbers on the two sides of a layer), state
sizes, head sizes and groups that are no power of two, norms in one part and in several, experts of which a token uses one,
some and all, with a shared expert that is a multiple of an expert's size, one that is not, and none, layers without a
feed-forward.
"""
import json
import os

import torch
from safetensors.torch import load_file

import plain_barilix


def moe(experts, top, ff, shared=None):
    mlp = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared is not None:
        mlp["shared"] = {"ff": shared}
    return mlp


def dense(ff):
    return {"kind": "dense", "ff": ff}


def parallel(left, right, window=None, rot=None):
    """left: (heads, kv_heads, dim, vdim, taps, scale); right: (heads, vdim, state, groups, norm_groups, taps); rot: (base, dims)
    and optionally the scaling (factor, low, high, original)."""
    heads, groups, dim, vdim, taps, scale = left
    side = {"heads": heads, "kv_heads": groups, "dim": dim, "vdim": vdim, "conv": taps, "scale": scale}
    if window is not None:
        side["mask"] = {"size": window}
    if rot is not None:
        side["rot"] = {"base": rot[0], "dims": rot[1]}
        if len(rot) > 2:
            side["rot"]["scaling"] = dict(zip(("factor", "low", "high", "original"), rot[2]))
    heads, vdim, state, groups, parts, taps = right
    return {"left": side, "right": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "norm_groups": parts, "conv": taps}}


def delta(heads, kv_heads, dim, vdim, taps):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": taps}


CONFIG_R = {
    "architecture": "Barilix", "vocab": 181, "width": 72, "norm": {"eps": 1e-5}, "embedding": {"scale": 3.5},
    "layers": [
        {"type": "parallel", "mixer": parallel((4, 2, 16, 24, 3, 0.3), (6, 10, 12, 3, 2, 5), window=7, rot=(90.0, 8, (3.0, 0.5, 2.0, 40))), "mlp": dense(56)},
        {"type": "delta", "mixer": delta(6, 2, 24, 40, 2), "mlp": moe(5, 3, 24, shared=40)},
        {"type": "parallel", "mixer": parallel((6, 1, 32, 32, 1, 0.2), (2, 72, 33, 1, 1, 4), window=37, rot=(20000.0, 32)), "mlp": None},
        {"type": "delta", "mixer": delta(3, 3, 8, 130, 4), "mlp": moe(6, 2, 16)},
    ],
}
CONFIG_S = {        # no windows and no turning keys, odd sizes
    "architecture": "Barilix", "vocab": 120, "width": 50, "norm": {"eps": 1e-6}, "embedding": {"scale": 0.7},
    "layers": [
        {"type": "delta", "mixer": delta(1, 1, 12, 12, 1), "mlp": None},
        {"type": "parallel", "mixer": parallel((3, 3, 10, 6, 8, 0.4), (5, 9, 7, 5, 3, 1)), "mlp": moe(4, 1, 12, shared=24)},
        {"type": "parallel", "mixer": parallel((2, 1, 40, 40, 4, 0.2), (1, 33, 5, 1, 11, 2), window=1), "mlp": moe(3, 3, 20, shared=20)},
    ],
}
CONFIG_T = {        # sizes the matrix cores and the wide kernels take, experts whose products run over pairs of experts and tokens
    "architecture": "Barilix", "vocab": 96, "width": 128, "norm": {"eps": 1e-5}, "embedding": {"scale": 11.0},
    "layers": [
        {"type": "parallel", "mixer": parallel((4, 2, 64, 64, 4, 0.13), (4, 32, 64, 2, 4, 4), window=24, rot=(30000.0, 32, (8.0, 1.0, 4.0, 64))), "mlp": moe(7, 2, 64, shared=128)},
        {"type": "delta", "mixer": delta(4, 2, 64, 64, 4), "mlp": dense(264)},
        {"type": "parallel", "mixer": parallel((2, 2, 48, 48, 4, 0.15), (3, 16, 160, 1, 1, 4), window=80, rot=(100.0, 48)), "mlp": moe(8, 8, 16)},
    ],
}
CONFIGS = {"R": CONFIG_R, "S": CONFIG_S, "T": CONFIG_T}
DTYPES = ["float32", "bfloat16"]
# a row's largest error relative to the row's largest value, against float64 on the same stored weights
# (bfloat16: rows that rounding alone moves further are held to a multiple of that instead, see `allowed_rows`)
TOLERANCE = {"float32": 3e-5, "bfloat16": 4e-2}
SINGLE_LAYER_TOLERANCE = {"float32": 3e-5, "bfloat16": 4e-2}
# two cuts of the same request through the same engine: in 32-bit a sequence that brings many tokens takes the scans in chunks,
# whose sums run in another order
CUT_TOLERANCE_32 = 1e-5


def make_model(folder, raw_config, seed, std=0.08, norm_std=0.1):
    """Weights are stored in bfloat16, as the design's files are: a float32 run widens the same values."""
    from tlie_amd import write_random_model
    from tlie_amd.registry import config_from_dict
    write_random_model(str(folder), config_from_dict(raw_config), seed, std=std, norm_std=norm_std, dtype=torch.bfloat16)
    return str(folder)


def load_plain(folder):
    with open(os.path.join(folder, "config.json"), "r", encoding="utf-8") as handle:
        raw = json.load(handle)
    weights = {name: tensor.double() for name, tensor in load_file(os.path.join(folder, "model.safetensors")).items()}
    return raw, weights


def rewrite(folder, changes):
    """Applies `changes(weights)` to the folder's float64 weights and stores them again, in bfloat16 (the tables as integers)."""
    from tlie_amd.weights.safetensors_io import write_safetensors
    _, weights = load_plain(folder)
    changes(weights)
    write_safetensors(os.path.join(folder, "model.safetensors"),
                      {name: tensor.to(torch.int32 if name.endswith(".table") else torch.bfloat16).contiguous() for name, tensor in weights.items()})
    return load_plain(folder)


def allowed_rows(config, weights, tokens, dtype, want, draws=8):
    """Per row of logits, how far a run in `dtype` may be from `want`, relative to the row's largest value.  In bfloat16 the
    design amplifies rounding at some tokens (a key that is small before it is made a unit vector, a result divided by its
    own size), so the plain implementation is run `draws` times more with every product's input and result (and what the cache stores) moved
    by as much as rounding moves them: a row may be off by the tolerance, or by four times what those runs differ at that row."""
    allowed = torch.full((len(tokens),), TOLERANCE[dtype], dtype=torch.float64)
    if dtype == "float32":
        return allowed
    for seed in range(draws):
        moved = plain_barilix.noisy(seed, lambda: plain_barilix.forward(config, weights, list(tokens))[0])
        allowed = torch.maximum(allowed, 4.0 * row_errors(moved, want))
    return allowed


def plain_generate_greedy(config, weights, prompt, count):
    tokens, out = list(prompt), []
    for _ in range(count):
        token = int(torch.argmax(plain_barilix.forward(config, weights, tokens)[0][-1]))
        out.append(token)
        tokens.append(token)
    return out


def row_errors(got: torch.Tensor, want: torch.Tensor) -> torch.Tensor:
    got, want = got.double().cpu(), want.double().cpu()
    assert got.shape == want.shape, (got.shape, want.shape)
    return (got - want).abs().amax(dim=-1) / want.abs().amax(dim=-1)


def run_cut(engine, request, tokens, cuts):
    """The request's tokens in portions of the sizes `cuts` (repeated as needed); returns logits [T, vocab]."""
    from tlie_amd import StepEntry
    engine.admit(request)
    rows, at, index = [], 0, 0
    while at < len(tokens):
        count = min(cuts[index % len(cuts)], len(tokens) - at)
        rows.append(engine.step([StepEntry(request, tokens[at:at + count], list(range(count)))]).clone())
        at += count
        index += 1
    engine.finish(request)
    return torch.cat(rows, dim=0)
