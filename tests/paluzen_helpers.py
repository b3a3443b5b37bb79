"""What the Paluzen tests share: configurations of their own, model folders of random weights, and the comparison with
the plain implementation.

The configurations differ from each other in every size and option, and use values that make faults visible: fewer
key/value groups than heads (down to one), value heads of another size than the keys, windows that are no multiple of a
page (1, 7, 37 positions on pages of 16) and none, rotations over a part of a head, over all of it and none, heads beside
them of other numbers and sizes, scales of the two sides that are negative, zero and one, decays of 0 and 1, a loop that
starts after the first layer and runs three times, one of a single layer that begins the model, and none, routers that use
one, some and all of their experts, with and without groups and identities, groups that hold experts and identities
together, layers without a feed-forward, models with and without capped logits.
"""
import json
import os

import torch
from safetensors.torch import load_file

import plain_paluzen


def moe(experts, top, ff, groups=None, identity=None):
    router = {"experts": experts, "top": top}
    if groups is not None:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    if identity is not None:
        router["identity"] = identity
    return {"kind": "moe", "expert": {"ff": ff}, "router": router}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def parallel(left, right, scales, window=None, rot=None):
    heads, groups, dim, vdim, scale = left
    side = {"heads": heads, "kv_heads": groups, "dim": dim, "vdim": vdim, "scale": scale}
    if window is not None:
        side["mask"] = {"size": window}
    if rot is not None:
        side["rot"] = {"base": rot[0], "dims": rot[1]}
    return {"left": side, "right": {"heads": right[0], "dim": right[1]}, "left_scale": scales[0], "right_scale": scales[1]}


def lightning(dim, vdim, decay):
    return {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": list(decay)}


CONFIG_U = {
    "architecture": "Paluzen", "vocab": 181, "width": 72, "norm": {"eps": 1e-5}, "logit_softcap": 14.0,
    "loop": {"start": 1, "stop": 3, "times": 3},
    "layers": [
        {"type": "parallel", "mixer": parallel((4, 1, 16, 24, 0.3), (3, 20), (1.2, -0.6), window=7, rot=(90.0, 8)), "mlp": dense(56)},
        {"type": "lightning", "mixer": lightning(24, 40, [1.0, 0.9, 0.0]), "mlp": moe(5, 3, 24, groups=(4, 2), identity=3)},
        {"type": "parallel", "mixer": parallel((6, 3, 32, 32, 0.2), (2, 72), (0.7, 1.0), window=37, rot=(20000.0, 32)), "mlp": None},
        {"type": "lightning", "mixer": lightning(8, 130, [0.99, 0.5]), "mlp": moe(6, 2, 16)},
    ],
}
CONFIG_V = {        # no loop, logits as they are, no windows and no turning keys
    "architecture": "Paluzen", "vocab": 120, "width": 50, "norm": {"eps": 1e-6},
    "layers": [
        {"type": "lightning", "mixer": lightning(12, 12, [0.97]), "mlp": None},
        {"type": "parallel", "mixer": parallel((3, 3, 10, 6, 0.4), (5, 8), (-0.5, 1.5)), "mlp": moe(4, 5, 12, groups=(2, 2), identity=2)},
        {"type": "parallel", "mixer": parallel((2, 1, 40, 40, 0.2), (1, 33), (1.0, 0.4), window=1), "mlp": moe(3, 1, 20, groups=(3, 1))},
    ],
}
CONFIG_W = {        # a loop of the first layer alone; head sizes the matrix cores take, experts whose products run over pairs of experts and tokens
    "architecture": "Paluzen", "vocab": 96, "width": 128, "norm": {"eps": 1e-5}, "logit_softcap": 25.0,
    "loop": {"start": 0, "stop": 1, "times": 2},
    "layers": [
        {"type": "parallel", "mixer": parallel((4, 2, 64, 64, 0.13), (4, 32), (1.0, 1.0), window=24, rot=(30000.0, 32)), "mlp": moe(7, 2, 64, groups=(4, 3), identity=1)},
        {"type": "lightning", "mixer": lightning(160, 64, [0.999, 0.8]), "mlp": dense(264)},
        {"type": "parallel", "mixer": parallel((2, 2, 48, 48, 0.15), (2, 64), (0.9, 0.3), window=80, rot=(100.0, 48)), "mlp": moe(8, 8, 16, identity=4)},
    ],
}
CONFIGS = {"U": CONFIG_U, "V": CONFIG_V, "W": CONFIG_W}
DTYPES = ["float32", "bfloat16"]
# a row's largest error relative to the row's largest value, against float64 on the same stored weights
# (bfloat16: rows that rounding alone moves further are held to a multiple of that instead, see `allowed_rows`)
TOLERANCE = {"float32": 3e-5, "bfloat16": 4e-2}
SINGLE_LAYER_TOLERANCE = {"float32": 3e-5, "bfloat16": 4e-2}
# two cuts of the same request through the same engine: in 32-bit a sequence that brings many tokens takes the scan's sliced
# walk, whose sums run in another order
CUT_TOLERANCE_32 = 1e-5


def make_model(folder, raw_config, seed, std=0.08, norm_std=0.1, settled=False):
    """Weights are stored in bfloat16, as the design's files are: a float32 run widens the same values.
    settled: numbers of which rounding to bfloat16 decides nothing (see `settle`)."""
    from tlie_amd import write_random_model
    from tlie_amd.registry import config_from_dict
    write_random_model(str(folder), config_from_dict(raw_config), seed, std=std, norm_std=norm_std, dtype=torch.bfloat16)
    if settled:
        rewrite(str(folder), lambda weights: settle(weights, seed))
    return str(folder)


def settle(weights, seed):
    """Two places of the design turn on rounding with random weights.  A router's choice is a step function: its
    corrections are set so far apart that no score moves it.  And a head of the token-shift mixing is divided by its root
    mean square: where it forgets fast and the current token's bonus is next to nothing, its result is often a small
    difference of a few products, whose direction is rounding's; decays near 0.95 and a bonus near 1 make it a sum of
    many."""
    generator = torch.Generator().manual_seed(seed)
    for name in sorted(weights):
        if name.endswith("mlp.correction"):
            count = weights[name].numel()
            weights[name] = 1.25 * torch.randperm(count, generator=generator).double() - 2.0       # (a score lies in 0 .. 1)
        elif name.endswith("right.w0"):
            weights[name] -= 3.0
        elif name.endswith("right.u"):
            weights[name] += 1.0


def load_plain(folder):
    with open(os.path.join(folder, "config.json"), "r", encoding="utf-8") as handle:
        raw = json.load(handle)
    weights = {name: tensor.double() for name, tensor in load_file(os.path.join(folder, "model.safetensors")).items()}
    return raw, weights


def rewrite(folder, changes):
    """Applies `changes(weights)` to the folder's float64 weights and stores them again, in bfloat16."""
    from tlie_amd.weights.safetensors_io import write_safetensors
    _, weights = load_plain(folder)
    changes(weights)
    write_safetensors(os.path.join(folder, "model.safetensors"), {name: tensor.to(torch.bfloat16).contiguous() for name, tensor in weights.items()})
    return load_plain(folder)


def allowed_rows(config, weights, tokens, dtype, want, draws=4):
    """Per row of logits, how far a run in `dtype` may be from `want`, relative to the row's largest value.  In bfloat16 the
    design amplifies rounding at some tokens (a head's result that is a small difference of products is divided by its own
    size), so the plain implementation is run `draws` times more with every product's input and result moved by as much as
    rounding moves them: a row may be off by the tolerance, or by four times what those runs differ at that row."""
    allowed = torch.full((len(tokens),), TOLERANCE[dtype], dtype=torch.float64)
    if dtype == "float32":
        return allowed
    for seed in range(draws):
        moved = plain_paluzen.noisy(seed, lambda: plain_paluzen.forward(config, weights, list(tokens))[0])
        allowed = torch.maximum(allowed, 4.0 * row_errors(moved, want))
    return allowed


def plain_generate_greedy(config, weights, prompt, count):
    tokens, out = list(prompt), []
    for _ in range(count):
        token = int(torch.argmax(plain_paluzen.forward(config, weights, tokens)[0][-1]))
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
