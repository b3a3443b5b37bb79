"""The Barilix decoder on the GPU against the plain implementation (tests/plain_barilix.py): each mechanism alone, inputs
made so that a fault shows, then whole models through the engine's step function, cache and state manager, scheduler and
entry point, however the work is cut."""
import math
import random
from types import SimpleNamespace

import pytest
import torch

import plain_barilix as plain
from barilix_helpers import (CONFIGS, CUT_TOLERANCE_32, DTYPES, SINGLE_LAYER_TOLERANCE, allowed_rows, delta, dense, load_plain, make_model, moe,
                             parallel, plain_generate_greedy, rewrite, row_errors, run_cut)

pytestmark = pytest.mark.gpu
CASES = [(name, dtype) for name in CONFIGS for dtype in DTYPES]
DEVICE = "cuda:0"
F64 = torch.float64


def tokens_of(seed, count, vocab, avoid=()):
    rng = random.Random(seed)
    out = []
    while len(out) < count:
        token = rng.randrange(vocab)
        if token not in avoid:
            out.append(token)
    return out


@pytest.fixture(scope="module")
def setups(tmp_path_factory):
    """A model per configuration and number format."""
    made = {}

    def get(name, dtype="float32"):
        if (name, dtype) not in made:
            folder = make_model(tmp_path_factory.mktemp(f"barilix_{name}_{dtype}"), CONFIGS[name], seed=53)
            raw, weights = load_plain(folder)
            made[name, dtype] = {"folder": folder, "raw": raw, "weights": weights, "dtype": dtype, "plain": {}, "allowed": {}}
        return made[name, dtype]
    return get


def plain_logits(setup, tokens):
    key = tuple(tokens)
    if key not in setup["plain"]:
        setup["plain"][key] = plain.forward(setup["raw"], setup["weights"], list(tokens))[0]
        setup["allowed"][key] = allowed_rows(setup["raw"], setup["weights"], tokens, setup["dtype"], setup["plain"][key])
    return setup["plain"][key]


def assert_plain(got, setup, tokens, what, places=None):
    """got: logits at `places` of the request (default: all), against the plain implementation's."""
    places = list(range(len(tokens))) if places is None else list(places)
    want = plain_logits(setup, tokens)[places]
    excess = row_errors(got, want) - setup["allowed"][tuple(tokens)][places]
    worst = int(excess.argmax())
    assert float(excess.max()) <= 0.0, (f"{what}: row {worst} is off by {float(row_errors(got, want)[worst]):.3g} of its largest value "
                                        f"(allowed {float(setup['allowed'][tuple(tokens)][places][worst]):.3g})")


def new_engine(setup, dtype, max_tokens=640, page_size=16, max_requests=4, **options):
    from tlie_amd import Engine
    return Engine(setup["folder"], dtype=dtype, max_tokens=max_tokens, page_size=page_size, max_requests=max_requests, **options)


def assert_rows(got, want, tolerance, what):
    errors = row_errors(got, want)
    worst = int(errors.argmax())
    assert float(errors.max()) <= tolerance, f"{what}: row {worst} is off by {float(errors[worst]):.3g} of its largest value (allowed {tolerance})"


def split_product(dense_rows, nsplit, generator):
    """A product as `nsplit` float partial sums that add up to `dense_rows`."""
    from tlie_amd import ops
    if nsplit == 1:
        return ops.Product(dense_rows.to(DEVICE).contiguous(), 1)
    parts = torch.randn(nsplit, *dense_rows.shape, generator=generator)
    parts[0] += dense_rows.float() - parts.sum(0)
    return ops.Product(parts.to(DEVICE).contiguous(), nsplit)


def step_arrays(counts, slots):
    """The arrays of a step in which sequence i brings counts[i] tokens and sits in slots[i]; one sequence more without
    a slot and without tokens stands for the padding of a recorded step."""
    starts, token_seq, token_slot = [0], [], []
    for index, (count, slot) in enumerate(zip(counts, slots)):
        starts.append(starts[-1] + count)
        token_seq += [index] * count
        token_slot += [slot] * count
    as_int = lambda values: torch.tensor(values, dtype=torch.int32, device=DEVICE)     # noqa: E731
    return SimpleNamespace(seq_start=as_int(starts + [starts[-1]]), seq_slot=as_int(list(slots) + [-1]), token_seq=as_int(token_seq),
                           token_slot=as_int(token_slot), max_new=max(counts)), starts


def in_steps(lengths, steps, slots, run):
    """Walks sequences of `lengths` through `steps` (per step the tokens each sequence brings; 0: it pauses) and
    returns, per sequence, what run(ctx, pieces) gave for its tokens; pieces[i] = (sequence, from, to) of the step's i-th
    live sequence."""
    got, at = [[] for _ in lengths], [0] * len(lengths)
    for counts in steps:
        live = [s for s in range(len(lengths)) if counts[s] > 0]
        ctx, starts = step_arrays([counts[s] for s in live], [slots[s] for s in live])
        out = run(ctx, [(s, at[s], at[s] + counts[s]) for s in live])
        for i, s in enumerate(live):
            got[s].append(out[..., starts[i]:starts[i + 1], :].cpu())
            at[s] += counts[s]
    assert at == list(lengths)
    return [torch.cat(pieces, dim=-2) for pieces in got]


SHORT_STEPS = ([23, 9], [(1, 4), (5, 0), (2, 1), (1, 1), (14, 3)])
LONG_STEPS = ([260, 41], [(97, 1), (1, 30), (130, 0), (31, 9), (1, 1)])


# ---- each mechanism alone ----------------------------------------------------------------------------------
def conv_reference(u, taps, bias, silu):
    """One sequence, from its start: float64 [T, channels]."""
    y = plain.channel_conv(u.double(), taps.double())
    if bias is not None:
        y = y + bias.double()
    return plain.silu(y) if silu else y


@pytest.mark.parametrize("head,heads,taps,plan,nsplit,dtype,silu,bias", [
    (8, 3, 4, SHORT_STEPS, 1, "bfloat16", True, True), (8, 3, 4, LONG_STEPS, 3, "float32", True, False), (24, 2, 4, LONG_STEPS, 1, "bfloat16", False, True),
    (5, 4, 4, SHORT_STEPS, 1, "float32", True, True), (64, 5, 4, LONG_STEPS, 2, "float32", False, False), (256, 2, 4, SHORT_STEPS, 1, "bfloat16", True, False),
    (7, 9, 1, SHORT_STEPS, 1, "float32", True, True), (12, 3, 2, LONG_STEPS, 1, "bfloat16", True, True), (130, 2, 8, SHORT_STEPS, 2, "float32", True, True),
    (16, 6, 3, LONG_STEPS, 1, "float32", False, True)])
def test_the_short_convolution_in_three_layouts(head, heads, taps, plan, nsplit, dtype, silu, bias):
    """Heads of unit length times a number, heads divided by their root mean square times a weight, and a plain stretch of
    channels, token by token and head by head, in steps of unequal portions, slots out of order, columns on both sides."""
    from tlie_amd import ops
    generator = torch.Generator().manual_seed(head * 100 + taps)
    stored = torch.bfloat16 if dtype == "bfloat16" else torch.float32
    out_dtype = torch.float32
    channels, col, extra = 3 * heads * head, 8, 5 if nsplit > 1 else 8
    w = (0.5 * torch.randn(channels, taps, generator=generator)).to(stored)
    b = (0.3 * torch.randn(channels, generator=generator)).to(stored) if bias else None
    norm = 1.0 + 0.2 * torch.randn(head, generator=generator)
    lengths, steps = plan
    inputs = [torch.randn(length, channels, generator=generator).to(stored) for length in lengths]
    wanted = []
    for u in inputs:
        y = conv_reference(u, w, b, silu).reshape(len(u), 3, heads, head)
        wanted.append(torch.stack([plain.unit_length(y[:, 0], 1e-3) * 0.7, plain.unit_rms(y[:, 1], 1e-3) * norm.double(), y[:, 2]], dim=1).reshape(len(u), -1))
    stride = ops.short_conv_state_floats(channels, taps) + 4
    for layout in ("out", "heads"):
        state = torch.zeros(4, stride, device=DEVICE)
        state[2] = 7.0                                         # (a slot of nobody's)
        parts = heads * head
        segments = [ops.ConvSegment(parts, head, "length", None, 1e-3, 0.7, target=layout),
                    ops.ConvSegment(parts, head, "rms", norm.to(DEVICE), 1e-3, target=layout, out_col=parts), ops.ConvSegment(parts, head, target=layout, out_col=2 * parts)]

        def run(ctx, pieces):
            rows = torch.cat([inputs[s][first:last] for s, first, last in pieces])
            wide = torch.cat([torch.full((len(rows), col), 9.0, dtype=stored), rows, torch.full((len(rows), extra), -9.0, dtype=stored)], dim=1)
            fused = split_product(wide, nsplit, generator)
            got = ops.short_conv(fused, col, w.to(DEVICE), b.to(DEVICE) if b is not None else None, state if taps > 1 else None, ctx, segments, channels, out_dtype,
                                 silu=silu)
            if layout == "heads":
                count, planes = len(rows), ops.plane_rows(len(rows))
                assert got.shape == (planes, channels)
                got = got.reshape(3 * heads, planes, head)[:, :count].transpose(0, 1).reshape(count, channels)
            return got
        for got, want, u in zip(in_steps(lengths, steps, [3, 0], run), wanted, inputs):
            assert float((got.double() - want).abs().max()) < 2e-5, layout
        if taps > 1:
            for slot, u in zip([3, 0], inputs):
                kept = state[slot, :(taps - 1) * channels].cpu().reshape(taps - 1, channels)
                assert float((kept - u[-(taps - 1):].float()).abs().max()) < 1e-5
            assert float((state[:, (taps - 1) * channels:stride][[0, 3]]).abs().max()) == 0.0 and bool((state[2] == 7.0).all())


@pytest.mark.parametrize("heads,groups,d,dv,rot,taps,start", [(4, 2, 16, 24, 8, 4, 0), (3, 1, 10, 6, 4, 3, 5), (8, 2, 64, 64, 64, 4, 0), (2, 2, 48, 48, 16, 4, 3),
                                                              (6, 3, 32, 32, 0, 8, 0), (4, 1, 128, 128, 128, 4, 13), (5, 5, 16, 16, 4, 1, 2), (2, 1, 256, 256, 8, 4, 0)])
@pytest.mark.parametrize("dtype", DTYPES)
def test_placement_behind_a_convolution(heads, groups, d, dv, rot, taps, start, dtype):
    """Queries, keys and values of a prompt's portion that begins at position `start` (in the middle of a page or not), on pages
    in any order: convolution, norm a head, rotation; keys [row][dim] and values [dim][row] of every token, and nothing else."""
    from tlie_amd import ops
    generator = torch.Generator().manual_seed(d + heads)
    stored = torch.bfloat16 if dtype == "bfloat16" else torch.float32
    page_size, tokens = 16, 45
    channels = (heads + groups) * d + groups * dv
    w = (0.5 * torch.randn(channels, taps, generator=generator)).to(stored)
    q_norm, k_norm = (1.0 + 0.2 * torch.randn(d, generator=generator) for _ in range(2))
    before, u = (torch.randn(count, channels, generator=generator).to(stored) for count in (taps - 1, tokens))
    y = conv_reference(torch.cat([before, u]), w, None, False)[taps - 1:]
    rotation = {"base": 50.0, "dims": rot}
    positions = torch.arange(start, start + tokens)
    turn = (lambda x: plain.rotate_halves(x, positions, rotation)) if rot else (lambda x: x)
    want_q = turn(plain.unit_rms(y[:, :heads * d].reshape(tokens, heads, d), 1e-4) * q_norm.double())
    want_k = turn(plain.unit_rms(y[:, heads * d:(heads + groups) * d].reshape(tokens, groups, d), 1e-4) * k_norm.double())
    want_v = y[:, (heads + groups) * d:].reshape(tokens, groups, dv)
    pages = torch.randperm(6, generator=generator)[:4].tolist()
    slots = torch.tensor([pages[p // page_size] * page_size + p % page_size for p in positions.tolist()], dtype=torch.int32)
    shape = (6, 2, groups, page_size * d) if d == dv else (6, groups, page_size * (d + dv))
    cache = torch.full(shape, 5.0, dtype=stored, device=DEVICE)
    state = torch.zeros(3, ops.short_conv_state_floats(channels, taps), device=DEVICE)
    state[1, :(taps - 1) * channels] = before.float().flatten().to(DEVICE)
    ctx, _ = step_arrays([tokens], [1])
    ctx.positions = positions.to(torch.int32).to(DEVICE)
    freq = torch.tensor(plain.frequencies(rotation), dtype=torch.float32, device=DEVICE) if rot else None
    segments = [ops.ConvSegment(heads * d, d, "rms", q_norm.to(DEVICE), 1e-4, rotated=rot > 0), ops.ConvSegment(groups * d, d, "rms", k_norm.to(DEVICE), 1e-4, rotated=rot > 0, target="keys"),
                ops.ConvSegment(groups * dv, dv, target="values")]
    got = ops.short_conv(ops.Product(u.to(DEVICE), 1), 0, w.to(DEVICE), None, state if taps > 1 else None, ctx, segments, heads * d, stored, inv_freq=freq, rot_dim=rot, cache=cache,
                         slot_map=slots.to(DEVICE), num_kv_heads=groups, head_dim=d, value_dim=dv)
    tolerance = 2e-5 if dtype == "float32" else 2.0 ** -8
    assert float(((got.cpu().double().reshape(tokens, heads, d) - want_q).abs() - tolerance * want_q.abs().clamp(min=1.0)).max()) <= 0.0
    flat = cache.cpu().double().reshape(6, -1)
    keys, values = flat[:, :groups * page_size * d].reshape(6, groups, page_size, d), flat[:, groups * page_size * d:].reshape(6, groups, dv, page_size)
    untouched = torch.ones(6, page_size, dtype=torch.bool)
    for t, slot in enumerate(slots.tolist()):
        page, row = slot // page_size, slot % page_size
        untouched[page, row] = False
        assert float(((keys[page, :, row] - want_k[t]).abs() - tolerance * want_k[t].abs().clamp(min=1.0)).max()) <= 0.0, t
        assert float(((values[page, :, :, row] - want_v[t]).abs() - tolerance * want_v[t].abs().clamp(min=1.0)).max()) <= 0.0, t
    assert bool((keys.transpose(1, 2)[untouched] == 5.0).all()) and bool((values.permute(0, 3, 1, 2)[untouched] == 5.0).all())


def scan_reference(kind, q, k, v, z_a, z_b, rate, bias, skip):
    """One sequence: q, k [T, G, dim], v [T, H, vdim], z_a, z_b [T, H], all float64."""
    heads, groups = v.shape[1], k.shape[1]
    out = []
    for h in range(heads):
        g = h // (heads // groups)
        step = plain.softplus(z_a[:, h] + bias[h])
        if kind == "delta":
            out.append(plain.delta_walk(q[:, g], k[:, g], v[:, h], torch.exp(-torch.exp(rate[h]) * step), torch.sigmoid(z_b[:, h])))
        else:
            out.append(plain.state_space_walk(v[:, h], k[:, g], q[:, g], step, -torch.exp(rate[h]), skip[h]))
    return torch.stack(out, dim=1).reshape(len(q), -1)


SCANS = [(4, 2, 16, 24, None), (3, 3, 5, 7, None), (2, 1, 64, 130, None), (6, 1, 33, 64, None), (1, 1, 256, 20, None), (8, 4, 128, 128, None), (5, 1, 130, 16, None), (16, 2, 48, 64, 32),
         (40, 1, 20, 32, None), (2, 2, 100, 300, 150)]


@pytest.mark.parametrize("kind", ["additive", "delta"])
@pytest.mark.parametrize("heads,groups,dim,vdim,width", SCANS)
@pytest.mark.parametrize("plan,nsplit,dtype", [(SHORT_STEPS, 2, "float32"), (LONG_STEPS, 1, "bfloat16")])
def test_the_gated_scans(kind, heads, groups, dim, vdim, width, plan, nsplit, dtype):
    """Both updates, walked token by token and in chunks, against the plain walks; the rates span three decades (heads that
    forget at once, heads that keep), some keys repeat, and a token forgets nearly everything now and then."""
    from tlie_amd import ops
    generator = torch.Generator().manual_seed(heads * 1000 + dim)
    lengths, steps = plan
    stored = torch.bfloat16 if dtype == "bfloat16" else torch.float32
    rate, bias = torch.linspace(-4.0, 3.0, heads), torch.randn(heads, generator=generator) * 0.5 - 1.0
    skip = torch.randn(heads, generator=generator)
    q, k, v, z = [], [], [], []
    for length in lengths:
        keys = torch.randn(length, groups, dim, generator=generator)
        for t in range(1, length):
            if t % 5 == 0:
                keys[t] = keys[t - 1]
        if kind == "delta":
            keys = keys / keys.norm(dim=-1, keepdim=True)
        q.append(torch.randn(length, groups, dim, generator=generator) / math.sqrt(dim))
        k.append(keys / (1.0 if kind == "delta" else math.sqrt(dim)))
        v.append(torch.randn(length, heads, vdim, generator=generator))
        gates = torch.randn(length, 2 * heads, generator=generator)
        gates[::17, :heads] += 30.0                            # (softplus of it: the whole state goes)
        gates[1::3, heads:] += 6.0                             # (the delta rule's w next to 1)
        z.append(gates.to(stored))
    want = [scan_reference(kind, a.double(), b.double(), c.double(), d[:, :heads].double(), d[:, heads:].double(), rate.double(), bias.double(), skip.double())
            for a, b, c, d in zip(q, k, v, z)]
    width = width or vdim
    channels = 2 * groups * dim + heads * vdim
    state = torch.zeros(3, ops.gated_scan_state_floats(heads, dim, vdim) + 8, device=DEVICE)

    def planes_of(x, size, rows):
        x = x.reshape(len(x), -1, size).transpose(0, 1)
        return torch.cat([x, torch.full((x.shape[0], rows - x.shape[1], size), math.nan)], dim=1).flatten()       # (rows beyond the tokens are no one's)

    def run(ctx, pieces):
        cut = lambda lists: torch.cat([lists[s][first:last] for s, first, last in pieces])      # noqa: E731
        tokens = len(cut(q))
        rows = ops.plane_rows(tokens)
        flat = torch.cat([planes_of(cut(v).reshape(tokens, -1), width, rows), planes_of(cut(k).reshape(tokens, -1), dim, rows), planes_of(cut(q).reshape(tokens, -1), dim, rows)])
        product = split_product(torch.cat([torch.full((tokens, 3), 4.0, dtype=stored), cut(z)], dim=1), nsplit, generator)
        return ops.gated_scan(flat.reshape(rows, channels).to(DEVICE), heads * vdim + groups * dim, heads * vdim, 0, product, 3, rate.to(DEVICE), bias.to(DEVICE), state, ctx,
                              heads, groups, dim, vdim, b_col=3 + heads if kind == "delta" else None, skip=skip.to(DEVICE) if kind == "additive" else None, value_width=width)
    for got, exact in zip(in_steps(lengths, steps, [2, 0], run), want):
        assert bool(torch.isfinite(got).all())
        assert float((got.double() - exact).abs().max()) < 2e-5 * float(exact.abs().max())
    assert float(state[1].abs().max()) == 0.0 and float(state[:, -8:].abs().max()) == 0.0


def test_scans_of_many_sequences_in_one_step():
    """Sequences on both sides of the length from which chunks are taken, and padding: each its own result and state."""
    from tlie_amd import ops
    generator = torch.Generator().manual_seed(4)
    counts, slots = [23, 24, 1, 33, 64, 2, 25], [6, 0, 3, 5, 1, 7, 2]
    heads, groups, dim, vdim = 4, 2, 20, 32
    total = sum(counts)
    q, k = (torch.randn(total, groups, dim, generator=generator) / math.sqrt(dim) for _ in range(2))
    k = k / k.norm(dim=-1, keepdim=True)
    v, z = torch.randn(total, heads, vdim, generator=generator), torch.randn(total, 2 * heads, generator=generator)
    rate, bias = torch.zeros(heads), torch.zeros(heads) - 2.0
    state = torch.zeros(8, ops.gated_scan_state_floats(heads, dim, vdim), device=DEVICE)
    ctx, starts = step_arrays(counts, slots)
    rows = ops.plane_rows(total)
    pad = lambda x, size: torch.cat([x.reshape(total, -1, size).transpose(0, 1), torch.zeros(x.numel() // total // size, rows - total, size)], dim=1).flatten()      # noqa: E731
    planes = torch.cat([pad(q, dim), pad(k, dim), pad(v, vdim)]).reshape(rows, -1).to(DEVICE)
    product = ops.Product(z.to(DEVICE), 1)
    got = ops.gated_scan(planes, 0, groups * dim, 2 * groups * dim, product, 0, rate.to(DEVICE), bias.to(DEVICE), state, ctx, heads, groups, dim, vdim, b_col=heads).cpu()
    for index, count in enumerate(counts):
        part = slice(starts[index], starts[index + 1])
        exact = scan_reference("delta", *(x[part].double() for x in (q, k, v)), z[part, :heads].double(), z[part, heads:].double(), rate.double(), bias.double(), None)
        assert float((got[part].double() - exact).abs().max()) < 1e-5, index
    assert float(state[4].abs().max()) == 0.0 and all(float(state[slot].abs().max()) > 0.0 for slot in slots)


@pytest.mark.parametrize("tokens,hidden,nsplit,dtype,out", [(6, 80, 1, torch.float32, torch.float32), (3, 203, 2, torch.float32, torch.bfloat16), (20, 2056, 1, torch.bfloat16, torch.bfloat16),
                                                            (5, 72, 3, torch.float32, torch.bfloat16), (2, 6000, 1, torch.bfloat16, torch.bfloat16), (4, 33, 1, torch.bfloat16, torch.float32)])
@pytest.mark.parametrize("form", ["plain", "sum", "pair"])
@pytest.mark.parametrize("centred", [True, False])
def test_a_result_is_normed_before_it_joins(tokens, hidden, nsplit, dtype, out, form, centred):
    from tlie_amd import ops
    generator = torch.Generator().manual_seed(hidden)
    w_dtype = torch.bfloat16 if out == torch.bfloat16 or dtype == torch.bfloat16 else torch.float32
    residual = torch.randn(tokens, hidden, generator=generator)
    first, second = (0.5 + 2.0 * torch.randn(tokens, hidden, generator=generator).to(dtype) for _ in range(2))
    weight, bias, last, side1, side2 = ((1.0 + 0.3 * torch.randn(hidden, generator=generator)).to(w_dtype) for _ in range(5))
    parts = [split_product(x, nsplit, generator) for x in (first, second)]
    if form == "plain":
        value, exact = parts[0], first.double()
    elif form == "sum":
        value, exact = ops.ScaledSum(parts[0], 0.7, parts[1], -1.3), 0.7 * first.double() - 1.3 * second.double()
    else:
        value = ops.NormedPair(parts[0], side1.to(DEVICE), parts[1], side2.to(DEVICE), 1e-2, 0.5)
        exact = 0.5 * (plain.unit_rms(first.double(), 1e-2) * side1.double() + plain.unit_rms(second.double(), 1e-2) * side2.double())
    norm = (lambda x, w, eps: plain.centred_norm(x, w, eps)) if centred else (lambda x, w, eps: plain.unit_rms(x, eps) * w)
    want = residual.double() + norm(exact, weight.double(), 1e-3) + bias.double()
    params = ops.NormParams(weight.to(DEVICE), bias.to(DEVICE), 1e-3, centred)
    last_params = ops.NormParams(last.to(DEVICE), None, 1e-5, centred)
    tolerance = 3e-6 if out == torch.float32 else 2.0 ** -8
    delta_ = ops.PostNormed(value, params)
    on = residual.to(DEVICE)
    rows = torch.tensor([tokens - 1, 0], dtype=torch.int32, device=DEVICE)
    got = ops.post_norm(on, delta_, out, last=last_params, rows=rows).cpu().double()
    exact_last = norm(want, last.double(), 1e-5)[[tokens - 1, 0]]
    assert float((got - exact_last).abs().max()) < tolerance * float(exact_last.abs().max())
    assert torch.equal(on.cpu(), residual)                                 # (rows alone leave the residual as it was)
    got = ops.post_norm(on, delta_, out).cpu().double()
    scale = float(want.abs().max())
    assert float((on.cpu().double() - want).abs().max()) < 3e-6 * scale and float((got - want).abs().max()) < tolerance * scale
    assert ops.post_norm(on, None) is None and torch.equal(ops.post_norm(on, None, torch.float32), on)
    if form == "pair":
        assert float((value.dense().cpu().double() - exact).abs().max()) < 1e-5 * float(exact.abs().max())


@pytest.mark.parametrize("parts,size,nsplit,dtype", [(1, 24, 2, "float32"), (3, 20, 1, "float32"), (1, 1048, 1, "bfloat16"), (2, 2048, 1, "bfloat16"), (4, 64, 1, "bfloat16"),
                                                     (1, 700, 1, "float32"), (5, 13, 1, "bfloat16"), (1, 6152, 3, "float32")])
def test_a_gate_that_joins_before_the_norm(parts, size, nsplit, dtype):
    from tlie_amd import ops
    generator = torch.Generator().manual_seed(size)
    stored = torch.bfloat16 if dtype == "bfloat16" else torch.float32
    a, weight = torch.randn(9, parts * size, generator=generator), (1.0 + 0.3 * torch.randn(parts * size, generator=generator)).to(stored)
    z = torch.randn(9, parts * size + 16, generator=generator).to(stored)
    got = ops.head_combine(a.to(DEVICE), parts, size, 1e-3, stored, weight=weight.to(DEVICE), gate=split_product(z, nsplit, generator), gate_col=8, gate_kind="silu", gate_first=True)
    gated = a.double() * plain.silu(z[:, 8:8 + parts * size].double())
    want = plain.unit_rms(gated.reshape(9, parts, size), 1e-3).reshape(9, -1) * weight.double()
    assert float((got.cpu().double() - want).abs().max()) < (2e-5 if dtype == "float32" else 2.0 ** -7) * float(want.abs().max())


def test_a_table_names_a_tokens_experts():
    from tlie_amd import ops
    table = torch.tensor([[3, 0], [1, 2], [2, 0]], dtype=torch.int32)
    got = ops.table_scale(torch.tensor([2, 0, 1, 0], dtype=torch.int32, device=DEVICE), table.to(DEVICE), 5, always=2).cpu()
    want = torch.zeros(4, 7)
    want[:, 5:] = 1.0
    for t, names in enumerate(([2, 0], [3, 0], [1, 2], [3, 0])):
        want[t, names] = 0.5
    assert torch.equal(got, want)
    assert ops.table_scale(torch.tensor([1], dtype=torch.int32, device=DEVICE), table[:, :1].contiguous().to(DEVICE), 4).cpu().tolist() == [[0.0, 1.0, 0.0, 0.0]]


@pytest.mark.parametrize("tokens,experts,top,width,size", [(300, 5, 2, 128, 64), (65, 3, 1, 64, 192), (1000, 12, 4, 192, 64), (70, 9, 9, 64, 128)])
def test_gated_products_over_the_pairs_of_experts_and_tokens(tokens, experts, top, width, size):
    from tlie_amd import ops
    generator = torch.Generator().manual_seed(tokens)
    x = torch.randn(tokens, width, generator=generator).bfloat16()
    gate_up = (torch.randn(experts * 2 * size, width, generator=generator) / math.sqrt(width)).bfloat16()
    down = (torch.randn(width, experts * size, generator=generator) / math.sqrt(size)).bfloat16()
    scale = torch.zeros(tokens, experts)
    for t in range(tokens):
        used = torch.randperm(experts, generator=generator)[:top]
        scale[t, used] = 0.3 + torch.rand(top, generator=generator)
    plan = ops.route_plan(scale.to(DEVICE), experts, top)
    got = ops.routed_sum(ops.routed_down(ops.routed_gated(x.to(DEVICE), gate_up.to(DEVICE), plan), down.to(DEVICE), plan), plan).cpu().double()
    want = torch.zeros(tokens, width, dtype=F64)
    for e in range(experts):
        w = gate_up[e * 2 * size:(e + 1) * 2 * size].double()
        hidden = plain.silu(x.double() @ w[0::2].T) * (x.double() @ w[1::2].T) * scale[:, e:e + 1].double()
        want += hidden @ down[:, e * size:(e + 1) * size].double().T
    assert float((got - want).abs().max()) < 2e-2 * float(want.abs().max())


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_a_scaled_embedding_with_a_copy(dtype):
    from tlie_amd import ops
    generator = torch.Generator().manual_seed(3)
    table, tokens = torch.randn(20, 70, generator=generator).to(dtype), torch.tensor([3, 19, 0, 3], dtype=torch.int32)
    residual, copy = ops.embed_gather(tokens.to(DEVICE), table.to(DEVICE), 1.7, copy=True)
    want = table[tokens.long()].float() * 1.7
    assert torch.equal(residual.cpu(), want) and torch.equal(copy.cpu(), want.bfloat16())
    assert torch.equal(ops.embed_gather(tokens.to(DEVICE), table.to(DEVICE)).cpu(), table[tokens.long()].float())


# ---- single layers through the engine: a mixer's result from its input, and inputs made so that a fault shows ---------
def _single_layer(tmp_path, layer, seed, vocab=97, width=48, changes=None, scale=6.0):
    raw = {"architecture": "Barilix", "vocab": vocab, "width": width, "norm": {"eps": 1e-5}, "embedding": {"scale": scale}, "layers": [layer]}
    folder = make_model(tmp_path, raw, seed=seed)
    config, weights = load_plain(folder)
    if changes is not None:
        config, weights = rewrite(folder, changes)
    return folder, config, weights


def _traced(folder, tokens, dtype, cuts, names):
    """Named tensors of every token of the only layer, from the traces of steps of the sizes `cuts`."""
    from tlie_amd import Engine, StepEntry
    engine = Engine(folder, dtype=dtype, max_tokens=1024, page_size=16, max_requests=2)
    engine.admit("a")
    kept, at, index = [[] for _ in names], 0, 0
    while at < len(tokens):
        count = min(cuts[index % len(cuts)], len(tokens) - at)
        trace = {}
        engine.step([StepEntry("a", tokens[at:at + count], [count - 1])], trace=trace)
        for rows, name in zip(kept, names):
            rows.append(trace["layer0." + name].cpu())
        at += count
        index += 1
    return [torch.cat(rows).double() for rows in kept]


def assert_result(got, run, dtype, what, draws=3):
    """got against run(), the plain implementation's result; in bfloat16 a row may also be off by four times what rounding
    every product's input and result moves it (see `allowed_rows`)."""
    want = run()
    allowed = torch.full((len(want),), SINGLE_LAYER_TOLERANCE[dtype], dtype=F64)
    if dtype == "bfloat16":
        for seed in range(draws):
            allowed = torch.maximum(allowed, 4.0 * row_errors(plain.noisy(seed, run), want))
    excess = row_errors(got, want) - allowed
    assert float(excess.max()) <= 0.0, f"{what}: row {int(excess.argmax())} is off by {float(row_errors(got, want)[int(excess.argmax())]):.3g}"


PARALLELS = [
    parallel((4, 2, 16, 24, 4, 0.3), (3, 24, 12, 1, 2, 4), window=9, rot=(500.0, 8, (4.0, 1.0, 4.0, 60))),
    parallel((6, 6, 32, 32, 2, 0.2), (4, 18, 40, 4, 3, 6), window=150, rot=(10000.0, 32)),
    parallel((2, 1, 8, 70, 8, 0.5), (2, 160, 6, 2, 1, 1), rot=(20.0, 4, (2.0, 0.5, 8.0, 30))),
    parallel((8, 2, 96, 96, 4, 0.1), (10, 8, 16, 2, 5, 4), window=16, rot=(10000.0, 40)),
    parallel((2, 2, 16, 16, 1, 0.25), (2, 64, 130, 1, 1, 3), window=1),
]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("mixer", PARALLELS)
def test_attention_beside_a_state_space_mixer(tmp_path, mixer, dtype):
    folder, config, weights = _single_layer(tmp_path, {"type": "parallel", "mixer": mixer, "mlp": None}, seed=9)
    tokens = tokens_of(10, 300, 97)             # (long enough for the keys to be cut into parts that are merged)
    for cuts in ([300], [33, 1, 2, 20, 150], [280] + [1] * 20):
        h, got = _traced(folder, tokens, dtype, cuts, ["input_norm", "attention_output"])
        assert_result(got, lambda: plain.parallel(mixer, weights, "l0.mix.", h, torch.arange(len(tokens)), 1e-5), dtype, f"cuts {cuts[:5]}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("mixer", [delta(3, 3, 16, 20, 4), delta(4, 2, 130, 8, 2), delta(4, 1, 6, 70, 1), delta(6, 2, 64, 128, 4)])
def test_the_gated_delta_rule_alone(tmp_path, mixer, dtype):
    folder, config, weights = _single_layer(tmp_path, {"type": "delta", "mixer": mixer, "mlp": None}, seed=7)
    tokens = tokens_of(8, 150, 97)
    for cuts in ([150], [30, 1, 2, 9, 100], [1]):
        h, got = _traced(folder, tokens, dtype, cuts, ["input_norm", "attention_output"])
        assert_result(got, lambda: plain.delta(mixer, weights, "l0.mix.", h, None, 1e-5), dtype, f"cuts {cuts}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("mlp,width", [(dense(40), 48), (dense(264), 48), (moe(6, 3, 16, shared=24), 48), (moe(5, 1, 13), 48), (moe(4, 4, 24, shared=24), 48),
                                       (moe(9, 2, 64, shared=64), 64), (moe(8, 1, 128, shared=256), 128), (moe(7, 3, 64), 64)])
def test_feed_forwards_alone(tmp_path, mlp, width, dtype):
    """A layer's second sublayer from its input, the residual itself."""
    layer = {"type": "delta", "mixer": delta(2, 1, 8, 8, 3), "mlp": mlp}
    folder, config, weights = _single_layer(tmp_path, layer, seed=15, width=width)
    tokens = tokens_of(16, 100, 97)
    ids = torch.tensor(tokens)
    for cuts in ([100], [2], [1], [9, 1, 70]):
        x0, h, got = _traced(folder, tokens, dtype, cuts, ["input_norm", "post_attention_norm", "mlp_output"])
        assert_result(got, lambda: plain.feed_forward(mlp, weights, "l0.mlp.", h, ids), dtype, f"cuts {cuts}")
        assert_rows(x0, weights["embed"][ids] * 6.0, 1e-6 if dtype == "float32" else 4e-3, "what the mixer reads")


def _listener(window, dim, vdim, A, B):
    """A `parallel` mixer and the change of its weights that makes head 0 look at one position only: token B's key and
    token A's query are large in a dim that does not turn, and in nobody else's."""
    mixer = parallel((2, 1, dim, vdim, 4, 0.3), (2, 8, 6, 1, 1, 4), window=window, rot=(100.0, 8))

    def boost(weights):
        weights["embed"][:, :2] = 0.0
        weights["embed"][B, 0], weights["embed"][A, 1] = 1.0, 1.0
        for name in ("q", "k"):
            weights[f"l0.mix.left.{name}"][10] = 0.0                   # head 0, dim 10 (past the rotated 8)
            weights[f"l0.mix.left.{name}.b"][10] = 0.0
            weights[f"l0.mix.left.{name}.conv"][10] = torch.tensor([0.0, 0.0, 0.0, 1.0], dtype=F64)        # the token alone
            weights[f"l0.mix.left.{name}.norm"][10] = 6.0
        weights["l0.mix.left.q"][10, 1] = weights["l0.mix.left.k"][10, 0] = 8.0
        weights["l0.mix.left.v"][:, 0] *= 20.0
        weights["l0.mix.left.v.conv"][:] = torch.tensor([0.0, 0.0, 0.0, 1.0], dtype=F64)
        weights["l0.mix.right.out"] *= 0.02
    return mixer, boost


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("dim,vdim", [(12, 20), (16, 16)])          # the plain attention kernel, and in bfloat16 the matrix cores'
@pytest.mark.parametrize("window", [37, 64, None])
def test_one_key_decides_the_result_inside_the_window_and_not_outside(tmp_path, dtype, dim, vdim, window):
    """B stands just inside or just outside A's window, at a page's first or last row, or hundreds of positions back
    (without a window); A comes last, in a prompt's portion and decoded alone."""
    A, B, length = 95, 96, 300
    mixer, boost = _listener(window, dim, vdim, A, B)
    folder, config, weights = _single_layer(tmp_path, {"type": "parallel", "mixer": mixer, "mlp": None}, seed=11, changes=boost)
    from tlie_amd import Engine
    engine = Engine(folder, dtype=dtype, max_tokens=640, page_size=16, max_requests=2)
    last = length - 1
    if window is None:
        places = {far: True for far in (0, 1, 15, 16, 250)}
    else:
        places = {last - window + 1: True, last - window: False, last - 4: True, last - window - 1: False}
    for far, inside in places.items():
        tokens = tokens_of(12, length, 97, avoid=(A, B))
        tokens[far], tokens[-1] = B, A
        other = list(tokens)
        other[far] = tokens[far - 1] if far else tokens[5]
        want, lost = plain.forward(config, weights, tokens)[0], plain.forward(config, weights, other)[0]
        moved = float(row_errors(lost[-1:], want[-1:]))
        assert moved > 0.15 if inside else moved < 0.05, f"B at {far}: {moved}"            # the test shows a key that is lost
        for cuts in ([length], [length - 1, 1], [7, 64, 2]):
            got = run_cut(engine, "a", tokens, cuts)
            assert_rows(got[-1:], want[-1:], SINGLE_LAYER_TOLERANCE[dtype], f"B at {far}, cuts {cuts}")


@pytest.mark.parametrize("dtype", DTYPES)
def test_windows_pass_over_decoded_tokens(tmp_path, dtype):
    """The same head; A asks again and again while B, which came in a decoded step too, leaves its window."""
    A, B, window = 95, 96, 40
    mixer, boost = _listener(window, 16, 16, A, B)
    folder, config, weights = _single_layer(tmp_path, {"type": "parallel", "mixer": mixer, "mlp": None}, seed=11, changes=boost)
    tokens = tokens_of(31, 160, 97, avoid=(A, B))
    tokens[70] = B
    asks = [75, 95, 108, 109, 110, 111, 150]                    # 109 = 70 + 39 sees B, 110 does not
    for place in asks:
        tokens[place] = A
    want = plain.forward(config, weights, tokens)[0]
    assert float(row_errors(want[109:110], want[110:111])) > 0.15
    from tlie_amd import Engine
    engine = Engine(folder, dtype=dtype, max_tokens=176, page_size=16, max_requests=1)
    for cuts in ([60] + [1] * 100, [160], [3, 50, 2, 17]):
        got = run_cut(engine, "a", tokens, cuts)
        assert_rows(got[asks], want[asks], SINGLE_LAYER_TOLERANCE[dtype], f"cuts {cuts[:4]}")
        engine.cache.check()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["delta", "parallel"])
def test_what_the_state_took_in_long_ago_is_still_there(tmp_path, dtype, kind):
    """Rates next to nothing, and a key and value written at the third token that stand out: token B alone has a large
    channel 0, which its key and its value read, and token A alone a large channel 1, which the query reads.  A comes last.
    A state that is lost or zeroed on the way (between steps, at a chunk's edge, in a slot that is used again) changes the
    last token's result."""
    A, B, length = 95, 96, 260
    own = torch.tensor([0.0, 0.0, 0.0, 1.0], dtype=F64)         # a convolution that reads the token alone
    if kind == "delta":
        mixer = delta(1, 1, 12, 12, 4)
    else:
        mixer = parallel((2, 1, 8, 8, 4, 0.3), (1, 12, 12, 1, 1, 4), window=20, rot=(100.0, 8))

    def boost(weights):
        weights["embed"][:, :2] = 0.0
        weights["embed"][B, 0], weights["embed"][A, 1] = 1.0, 1.0
        if kind == "delta":
            for name in "qk":
                weights[f"l0.mix.{name}"][10] = 0.0
                weights[f"l0.mix.{name}.conv"][:] = own
            weights["l0.mix.q"][10, 1] = weights["l0.mix.k"][10, 0] = 6.0
            weights["l0.mix.v"][:, 0] = torch.linspace(3.0, 9.0, 12, dtype=F64)
            weights["l0.mix.v.conv"][:] = own
            weights["l0.mix.b"][:, 0] = 4.0
            weights["l0.mix.A_log"][:] = -9.0
        else:
            # the rows of the first product: z | x | B | C | dt
            weights["l0.mix.right.in"][24:48] = 0.0              # B and C speak up for B and A alone
            weights["l0.mix.right.in"][24 + 10, 0] = weights["l0.mix.right.in"][36 + 10, 1] = 3.0
            weights["l0.mix.right.in"][12:24, 0] = torch.linspace(3.0, 9.0, 12, dtype=F64)
            weights["l0.mix.right.conv"][:] = own
            weights["l0.mix.right.conv.b"][12:] = 0.0
            weights["l0.mix.right.D"][:] = 0.0
            weights["l0.mix.right.A_log"][:] = -9.0
            weights["l0.mix.left.out"] *= 0.1
    folder, config, weights = _single_layer(tmp_path, {"type": kind, "mixer": mixer, "mlp": None}, seed=13, changes=boost)
    tokens = tokens_of(14, length, 97, avoid=(A, B))
    tokens[2], tokens[-1] = B, A
    other = list(tokens)
    other[2] = tokens[3]
    want, lost = plain.forward(config, weights, tokens)[0], plain.forward(config, weights, other)[0]
    assert float(row_errors(lost[-1:], want[-1:]).min()) > 0.1                      # the test shows a state that is lost
    from tlie_amd import Engine
    engine = Engine(folder, dtype=dtype, max_tokens=640, page_size=16, max_requests=1)      # one slot: used again by every cut
    for cuts in ([length], [length - 40] + [1] * 40, [5, 64, 2, 1], [3, 96, 33, 97]):
        got = run_cut(engine, "a", tokens, cuts)
        assert_rows(got[-1:], want[-1:], SINGLE_LAYER_TOLERANCE[dtype], f"cuts {cuts[:4]}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["delta", "parallel"])
def test_the_first_tokens_of_a_request_see_nothing_of_the_slots_last_owner(tmp_path, dtype, kind):
    """One slot, two requests after each other: the second's first tokens (whose convolutions and states start from zeros)
    equal the plain implementation's, and differ from what a kept state would give."""
    from tlie_amd import Engine
    mixer = delta(2, 1, 8, 12, 4) if kind == "delta" else parallel((2, 1, 8, 8, 4, 0.3), (2, 12, 8, 1, 1, 3), window=11, rot=(100.0, 8))
    folder, config, weights = _single_layer(tmp_path, {"type": kind, "mixer": mixer, "mlp": dense(40)}, seed=21)
    first, second = tokens_of(22, 50, 97), tokens_of(23, 9, 97)
    want = plain.forward(config, weights, second)[0]
    joined = plain.forward(config, weights, first + second)[0][len(first):]
    assert float(row_errors(joined[:1], want[:1])) > 0.02
    engine = Engine(folder, dtype=dtype, max_tokens=64, page_size=16, max_requests=1)
    for cuts in ([9], [1], [2, 1]):
        run_cut(engine, "x", first, [50])
        got = run_cut(engine, "y", second, cuts)
        setup = {"raw": config, "weights": weights, "dtype": dtype, "plain": {}, "allowed": {}}
        assert_plain(got, setup, second, f"cuts {cuts}")


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_token_reads_the_last_inputs_of_the_convolutions_across_steps(tmp_path, dtype):
    """Keys, queries and values, and what the state-space side takes in, are the input three tokens back alone: a window of
    the convolution that is lost or shifted between two steps changes everything."""
    mixer = parallel((2, 1, 16, 16, 4, 0.3), (2, 8, 6, 1, 1, 4), window=9, rot=(100.0, 8))

    def boost(weights):
        for name in ("left.q.conv", "left.k.conv", "left.v.conv", "right.conv"):
            weights["l0.mix." + name][:] = torch.tensor([1.0, 0.0, 0.0, 0.0], dtype=F64)
    folder, config, weights = _single_layer(tmp_path, {"type": "parallel", "mixer": mixer, "mlp": None}, seed=17, changes=boost)
    tokens = tokens_of(18, 40, 97)
    setup = {"raw": config, "weights": weights, "dtype": dtype, "plain": {}, "allowed": {}}
    from tlie_amd import Engine
    engine = Engine(folder, dtype=dtype, max_tokens=64, page_size=16, max_requests=1)
    for cuts in ([40], [1], [2], [3], [4, 1], [5, 2, 1, 1, 1], [7, 3]):
        assert_plain(run_cut(engine, "a", tokens, cuts), setup, tokens, f"cuts {cuts}")


# ---- whole models through the engine -----------------------------------------------------------------------
@pytest.mark.parametrize("name,dtype", CASES)
def test_whole_prompt_matches_the_plain_implementation(setups, name, dtype):
    setup = setups(name, dtype)
    tokens = tokens_of(1, 150, CONFIGS[name]["vocab"])
    engine = new_engine(setup, dtype)
    assert_plain(run_cut(engine, "r", tokens, [len(tokens)]), setup, tokens, f"{name} {dtype}")
    # (the rows that rounding alone moves far are few)
    assert float((setup["allowed"][tuple(tokens)] < 0.1).double().mean()) > 0.7
    engine.cache.check()


@pytest.mark.parametrize("name", list(CONFIGS))
def test_every_layer_matches_the_plain_implementation(setups, name):
    from tlie_amd import StepEntry
    setup = setups(name)
    tokens = tokens_of(2, 45, CONFIGS[name]["vocab"])
    _, residuals = plain.forward(setup["raw"], setup["weights"], tokens)
    engine = new_engine(setup, "float32")
    engine.admit("r")
    trace = {}
    engine.step([StepEntry("r", tokens, [len(tokens) - 1])], trace=trace)
    for index in range(residuals.shape[0]):
        got = trace[f"layer{index}.output"].cpu().double()
        scale = float(residuals[index].abs().max())
        assert float((got - residuals[index]).abs().max()) < 3e-5 * scale, f"{name}: the residual after layer {index}"


@pytest.mark.parametrize("name,dtype", CASES)
def test_cuts_agree_with_each_other_and_with_the_plain_implementation(setups, name, dtype):
    """Whole, token by token from the first token, in portions of two, and in portions of changing sizes that end inside
    pages, windows and the scans' chunks."""
    setup = setups(name, dtype)
    tokens = tokens_of(3, 130, CONFIGS[name]["vocab"])
    engine = new_engine(setup, dtype, max_tokens=160)
    whole = run_cut(engine, "w", tokens, [len(tokens)])
    for cuts in ([1], [2], [3, 5, 2, 1, 17], [40, 1, 1, 1, 70, 2]):
        got = run_cut(engine, "c", tokens, cuts)
        assert_plain(got, setup, tokens, f"{name} {dtype} cut {cuts}")
        if dtype == "float32":
            assert_rows(got, whole, CUT_TOLERANCE_32, f"{name} cut {cuts} against the whole prompt")
    engine.cache.check()


@pytest.mark.parametrize("name,dtype", CASES)
def test_batches_of_unequal_requests_with_pages_and_slots_used_again(setups, name, dtype):
    """Up to three live requests of unequal lengths in three slots more than once: portions of some beside single tokens
    of others, requests that pause for a step, a pool that only holds what is live."""
    from tlie_amd import StepEntry
    setup = setups(name, dtype)
    vocab = CONFIGS[name]["vocab"]
    lengths = {"a": 70, "b": 9, "c": 41, "d": 1, "e": 55, "f": 30}
    prompts = {key: tokens_of(10 + index, length, vocab) for index, (key, length) in enumerate(lengths.items())}
    engine = new_engine(setup, dtype, max_tokens=192, max_requests=3)
    rng = random.Random(5)
    waiting, live, at, rows = list(prompts), [], {}, {key: [] for key in prompts}
    steps = 0
    while waiting or live:
        while waiting and len(live) < 3 and sum((lengths[key] + 15) // 16 * 16 for key in live + [waiting[0]]) <= 192:
            key = waiting.pop(0)
            engine.admit(key)
            live.append(key)
            at[key] = 0
        entries, counts = [], {}
        for key in live:
            if len(live) > 1 and rng.random() < 0.25:
                continue                                              # left out of this step
            count = min(lengths[key] - at[key], rng.choice([1, 1, 2, 3, 9, 30]))
            entries.append(StepEntry(key, prompts[key][at[key]:at[key] + count], list(range(count))))
            counts[key] = count
        if not entries:
            continue
        logits = engine.step(entries)
        row = 0
        for entry in entries:
            rows[entry.request].append(logits[row:row + counts[entry.request]].clone())
            row += counts[entry.request]
            at[entry.request] += counts[entry.request]
            if at[entry.request] == lengths[entry.request]:
                engine.finish(entry.request)
                live.remove(entry.request)
        engine.cache.check()
        steps += 1
    assert steps > 12
    for key, tokens in prompts.items():
        assert_plain(torch.cat(rows[key]), setup, tokens, f"{name} {dtype} request {key}")


@pytest.mark.parametrize("name", list(CONFIGS))
def test_recorded_steps_equal_launched_steps_bit_for_bit(setups, name):
    from tlie_amd import StepEntry
    setup = setups(name, "bfloat16")
    vocab = CONFIGS[name]["vocab"]
    prompts = [tokens_of(40 + index, length, vocab) for index, length in enumerate((37, 20, 50))]
    results = []
    for capture in (True, False):
        engine = new_engine(setup, "bfloat16", capture_graphs=capture)
        rows = []
        for key in range(3):
            engine.admit(key)
        at = [0, 0, 0]
        for counts in [(5, 3, 0), (1, 1, 1), (1, 1, 1), (6, 2, 9), (1, 1, 1), (5, 3, 0), (1, 1, 1), (6, 0, 9), (1, 1, 1), (1, 0, 1)]:
            entries = [StepEntry(key, prompts[key][at[key]:at[key] + count], [count - 1]) for key, count in enumerate(counts) if count]
            rows.append(engine.step(entries).clone())
            for key, count in enumerate(counts):
                at[key] += count
        results.append(torch.cat(rows))
    assert torch.equal(results[0], results[1])
    assert bool(torch.isfinite(results[0]).all())


@pytest.mark.parametrize("name", list(CONFIGS))
def test_greedy_generation_through_the_scheduler(setups, name):
    setup = setups(name)
    vocab = CONFIGS[name]["vocab"]
    prompts = [tokens_of(70 + index, length, vocab) for index, length in enumerate((45, 3, 18))]
    want = [plain_generate_greedy(setup["raw"], setup["weights"], prompt, 10) for prompt in prompts]
    engine = new_engine(setup, "float32", max_tokens=256)
    assert engine.generate(prompts, max_tokens=10, chunk_size=16, max_tokens_per_step=24) == want
    assert engine.generate([prompts[1]], max_tokens=10) == [want[1]]
    engine.cache.check()
    assert len(new_engine(setups(name, "bfloat16"), "bfloat16").generate(prompts, max_tokens=5)[2]) == 5


def test_a_preempted_request_is_recomputed_from_a_state_of_zero(setups):
    setup = setups("S")
    prompts = [tokens_of(90 + index, 40, CONFIGS["S"]["vocab"]) for index in range(4)]
    want = [plain_generate_greedy(setup["raw"], setup["weights"], prompt, 20) for prompt in prompts]
    engine = new_engine(setup, "float32", max_tokens=176, max_requests=4)
    assert engine.generate(prompts, max_tokens=20, admit_partial=True) == want
    engine.cache.check()


@pytest.mark.parametrize("name,dtype", [("R", "float32"), ("T", "float32"), ("T", "bfloat16")])
def test_long_decoding_keeps_to_the_plain_implementation(setups, name, dtype):
    """A short prompt, then 200 tokens one by one: windows pass over decoded tokens many times, pages fill and go back to
    the pool while the request runs."""
    setup = setups(name, dtype)
    tokens = tokens_of(4, 205, CONFIGS[name]["vocab"])
    engine = new_engine(setup, dtype, max_tokens=256)
    got = run_cut(engine, "r", tokens, [5] + [1] * 200)
    assert_plain(got, setup, tokens, f"{name} {dtype}")
    engine.cache.check()


def test_the_command_line_and_the_replay_program_run_the_design(setups, tmp_path):
    import json
    import os
    import subprocess
    import sys
    import numpy
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    setup = setups("R")
    vocab = CONFIGS["R"]["vocab"]
    tokens, other = tokens_of(61, 40, vocab), tokens_of(62, 21, vocab)
    prompt = "ids:" + ",".join(str(token) for token in tokens[:9])
    run = subprocess.run([sys.executable, os.path.join(root, "bin", "tinyllama_amd"), "generate", setup["folder"], prompt, "6", "--dtype", "float32"],
                         capture_output=True, text=True, timeout=300)
    assert run.returncode == 0, run.stderr
    assert json.loads(run.stdout)["generated_tokens"] == plain_generate_greedy(setup["raw"], setup["weights"], tokens[:9], 6)
    lines = [{"step": 0, "entries": [{"id": "a", "tokens": tokens[:30], "want": [0, 29]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": tokens[30:31], "want": [0]}, {"id": "b", "tokens": other, "want": [20]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "c", "tokens": other[:7], "want": []}], "end": []},
             {"step": 3, "entries": [{"id": "a", "tokens": tokens[31:], "want": [8]}, {"id": "c", "tokens": other[7:], "want": [13]}], "end": ["a", "c"]}]
    for dtype in DTYPES:
        made = setups("R", dtype)
        out = tmp_path / dtype
        run = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", made["folder"], "--dtype", dtype,
                              "--out", str(out), "--max-tokens", "128", "--max-requests", "2"],
                             input="".join(json.dumps(line) + "\n" for line in lines), capture_output=True, text=True, timeout=300)
        assert run.returncode == 0 and run.stdout.split() == ["done", "0", "done", "1", "done", "2", "done", "3"], run.stderr
        assert not (out / "2.f32").exists()
        read = lambda step: torch.from_numpy(numpy.fromfile(out / f"{step}.f32", dtype="<f4").reshape(-1, vocab))      # noqa: E731
        assert_plain(read(0), made, tokens, f"{dtype} step 0", places=[0, 29])
        assert_plain(read(1)[:1], made, tokens, f"{dtype} step 1", places=[30])
        assert_plain(read(1)[1:], made, other, f"{dtype} step 1, the other request", places=[20])
        assert_plain(read(3)[:1], made, tokens, f"{dtype} step 3", places=[39])
        assert_plain(read(3)[1:], made, other, f"{dtype} step 3, the third request", places=[20])


# ---- configurations drawn at random ---------------------------------------------------------------------------
def drawn_configuration(seed):
    """Every size, count, constant and option of the design, in ranges that the given configurations do not cover."""
    rng = random.Random(seed)
    width = rng.choice([24, 36, 50, 64, 72, 100, 132])
    taps = lambda: rng.choice([1, 2, 3, 4, 4, 4, 7])      # noqa: E731
    layers = []
    for _ in range(rng.randint(1, 4)):
        kind = rng.choice(["parallel", "delta"])
        if kind == "parallel":
            groups = rng.choice([1, 2, 3])
            dim = rng.choice([4, 6, 10, 16, 24, 32, 48, 64, 80])
            left = (groups * rng.choice([1, 2, 4]), groups, dim, rng.choice([dim, dim, 5, 12, 40]), taps(), rng.choice([0.1, 0.25, 0.4]) * (16.0 / dim) ** 0.5)
            rot = None
            if rng.random() < 0.8:
                rot = (rng.choice([10.0, 1000.0, 500000.0]), rng.choice([d for d in (2, 4, 8, dim - dim % 2) if d <= dim]))
                if rng.random() < 0.6:
                    rot = (*rot, (rng.choice([2.0, 8.0]), 1.0, rng.choice([1.5, 4.0]), rng.choice([20, 64, 300])))
            space = rng.choice([1, 2, 3])
            heads, vdim = space * rng.choice([1, 2, 3]), rng.choice([3, 8, 20, 32, 64])
            parts = rng.choice([p for p in (1, 2, 3, 4, heads) if (heads * vdim) % p == 0])
            mixer = parallel(left, (heads, vdim, rng.choice([4, 7, 16, 33, 64]), space, parts, taps()), window=rng.choice([None, 1, 2, 5, 16, 17, 33, 64]), rot=rot)
        else:
            groups = rng.choice([1, 2, 3])
            mixer = delta(groups * rng.choice([1, 2, 3]), groups, rng.choice([3, 8, 16, 40, 96]), rng.choice([4, 16, 65, 128]), taps())
        mlp = None
        if rng.random() < 0.85:
            if rng.random() < 0.3:
                mlp = dense(rng.choice([3, 40, 150]))
            else:
                experts, ff = rng.randint(1, 7), rng.choice([3, 8, 20, 33, 64])
                mlp = moe(experts, rng.randint(1, experts), ff, shared=rng.choice([None, ff, 2 * ff, 11]))
        layers.append({"type": kind, "mixer": mixer, "mlp": mlp})
    return {"architecture": "Barilix", "vocab": rng.choice([31, 100, 257]), "width": width, "norm": {"eps": rng.choice([1e-6, 1e-5, 1e-3])},
            "embedding": {"scale": rng.choice([0.3, 1.0, 8.0])}, "layers": layers}


@pytest.mark.parametrize("seed", range(16))
def test_drawn_configurations_in_32_bit(tmp_path, seed):
    """Sizes and constants nobody chose: whole, in portions of changing sizes beside a second request, and token by token,
    against the plain implementation, pages of 16 or 32 rows (held to 1e-4: what is divided by its own root mean square may
    be a small difference, and nobody chose weights that avoid it)."""
    from tlie_amd import Engine, StepEntry
    raw = drawn_configuration(seed)
    folder = make_model(tmp_path / "model", raw, seed=seed)
    config, weights = load_plain(folder)
    rng = random.Random(100 + seed)
    tokens, other = tokens_of(seed, rng.randint(40, 110), raw["vocab"]), tokens_of(seed + 50, rng.randint(1, 30), raw["vocab"])
    want, want_other = plain.forward(config, weights, tokens)[0], plain.forward(config, weights, other)[0]
    engine = Engine(folder, dtype="float32", max_tokens=256, page_size=rng.choice([16, 32]), max_requests=2)
    assert_rows(run_cut(engine, "w", tokens, [len(tokens)]), want, 1e-4, f"seed {seed} whole: {raw}")
    engine.admit("a")
    engine.admit("b")
    rows, at, fed = [], 0, 0
    while at < len(tokens):
        count = min(rng.choice([1, 1, 2, 3, 7, 20, 40]), len(tokens) - at)
        entries = [StepEntry("a", tokens[at:at + count], list(range(count)))]
        if fed < len(other):
            entries.append(StepEntry("b", other[fed:fed + 1], [0]))
        logits = engine.step(entries)
        rows.append(logits[:count].clone())
        if fed < len(other):
            assert_rows(logits[count:], want_other[fed:fed + 1], 1e-4, f"seed {seed}, the second request's token {fed}: {raw}")
            fed += 1
        at += count
    assert_rows(torch.cat(rows), want, 1e-4, f"seed {seed} in portions: {raw}")
    engine.finish("a")
    engine.finish("b")
    engine.cache.check()
    assert_rows(run_cut(engine, "t", tokens[:24], [1]), want[:24], 1e-4, f"seed {seed} token by token: {raw}")


@pytest.mark.parametrize("seed", range(16))
def test_drawn_configurations_in_bfloat16(tmp_path, seed):
    """The same configurations through the bfloat16 kernels (head sizes that the matrix cores take and others side by side):
    whole and with the last tokens decoded one by one."""
    from tlie_amd import Engine
    raw = drawn_configuration(seed)
    folder = make_model(tmp_path / "model", raw, seed=seed)
    config, weights = load_plain(folder)
    setup = {"raw": config, "weights": weights, "dtype": "bfloat16", "plain": {}, "allowed": {}}
    tokens = tokens_of(seed, 90, raw["vocab"])
    engine = Engine(folder, dtype="bfloat16", max_tokens=128, page_size=16, max_requests=2)
    assert_plain(run_cut(engine, "w", tokens, [len(tokens)]), setup, tokens, f"seed {seed} whole: {raw}")
    assert_plain(run_cut(engine, "c", tokens, [70] + [1] * 20), setup, tokens, f"seed {seed} decoded: {raw}")
    engine.cache.check()
