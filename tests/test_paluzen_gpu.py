"""The Paluzen decoder on the GPU against the plain implementation (tests/plain_paluzen.py): each mechanism alone, inputs
made so that a fault shows, then whole models through the engine's step function, cache and state manager, scheduler and
entry point, however the work is cut."""
import math
import random
from types import SimpleNamespace

import pytest
import torch

import plain_paluzen as plain
from paluzen_helpers import (CONFIGS, CUT_TOLERANCE_32, DTYPES, SINGLE_LAYER_TOLERANCE, allowed_rows, dense, lightning, load_plain, make_model,
                             moe, parallel, plain_generate_greedy, rewrite, row_errors, run_cut)

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
    """A model per configuration and number format: those of the bfloat16 runs have numbers of which rounding decides
    nothing (`paluzen_helpers.settle`); those of the 32-bit runs have corrections as small as the scores, so that the
    routers' choices change from token to token."""
    made = {}

    def get(name, dtype="float32"):
        if (name, dtype) not in made:
            folder = make_model(tmp_path_factory.mktemp(f"paluzen_{name}_{dtype}"), CONFIGS[name], seed=53,
                                settled=dtype == "bfloat16")
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
@pytest.mark.parametrize("tokens,hidden,nsplit,out_dtype", [(6, 80, 1, torch.float32), (3, 203, 2, torch.bfloat16), (20, 32, 3, torch.float32),
                                                            (5, 2056, 1, torch.bfloat16)])
def test_the_rms_norm_adds_both_summands_of_a_part_with_a_number_a_row(tokens, hidden, nsplit, out_dtype):
    from tlie_amd import ops
    generator = torch.Generator().manual_seed(hidden)
    x, a, b = (torch.randn(tokens, hidden, generator=generator) for _ in range(3))
    x = x * 2.0 + 3.0                                           # (a mean that an RMS norm must not take off)
    weight = torch.randn(hidden, generator=generator).to(out_dtype)
    numbers = torch.randn(tokens, 4, generator=generator)       # the last of a row is the second summand's
    tolerance = 2e-5 if out_dtype == torch.float32 else 3e-2
    for row_scale in (None, numbers):
        both = ops.ScaledSum(split_product(a, nsplit, generator), 0.8, split_product(b, 1, generator), -1.7,
                             row_scale=row_scale.to(DEVICE) if row_scale is not None else None)
        factor = 1.0 if row_scale is None else numbers[:, -1:].double()
        summed = x.double() + 0.8 * a.double() - 1.7 * factor * b.double()
        want = plain.rms_norm(summed, weight.double(), 1e-5)
        residual = x.clone().to(DEVICE)
        got = ops.layer_norm(residual, both, weight.to(DEVICE), None, 1e-5, out_dtype, centred=False)
        assert got.dtype == out_dtype and float((residual.cpu().double() - summed).abs().max()) < 2e-5
        assert float((got.cpu().double() - want).abs().max()) < tolerance
        # only some rows: nothing but the result is written
        rows = torch.tensor([tokens - 1, 0], dtype=torch.int32, device=DEVICE)
        residual = x.clone().to(DEVICE)
        got = ops.layer_norm(residual, both, weight.to(DEVICE), None, 1e-5, out_dtype, rows=rows, centred=False)
        assert torch.equal(residual.cpu(), x) and float((got.cpu().double() - want[[tokens - 1, 0]]).abs().max()) < tolerance
        # no norm: the residual is brought up to date; what nobody fuses is added up the same way
        residual = x.clone().to(DEVICE)
        assert ops.layer_norm(residual, both, None, None, 0.0, out_dtype, want_out=False) is None
        assert float((residual.cpu().double() - summed).abs().max()) < 2e-5
        assert float((ops.as_product(both).dense().cpu().double() - (summed - x.double())).abs().max()) < 2e-5


def test_bfloat16_summands_join_a_float_residual_without_a_norm():
    from tlie_amd import ops
    generator = torch.Generator().manual_seed(2)
    x, a, b = (torch.randn(9, 48, generator=generator) for _ in range(3))
    both = ops.ScaledSum(ops.Product(a.bfloat16().to(DEVICE), 1), 2.0, ops.Product(b.bfloat16().to(DEVICE), 1), 0.5)
    residual = x.clone().to(DEVICE)
    ops.layer_norm(residual, both, None, None, 0.0, torch.bfloat16, want_out=False)
    want = x.double() + 2.0 * a.bfloat16().double() + 0.5 * b.bfloat16().double()
    assert float((residual.cpu().double() - want).abs().max()) < 1e-5


@pytest.mark.parametrize("width,plan,dtype", [(80, SHORT_STEPS, "float32"), (50, LONG_STEPS, "float32"), (64, LONG_STEPS, "bfloat16")])
def test_the_token_shift_in_front_of_a_mixer(width, plan, dtype):
    from tlie_amd.config.spec import PartSpec
    from tlie_amd.registry import lookup
    activation = torch.float32 if dtype == "float32" else torch.bfloat16
    generator = torch.Generator().manual_seed(width)
    (lengths, steps), slots = plan, [2, 0]
    part = lookup("sublayer_input", "token_shift")(PartSpec("token_shift", {"size": width, "tensor": ""}), activation, DEVICE)
    mu = torch.rand(width, generator=generator).to(activation)
    part.load({"l3.shift": mu.to(DEVICE)}, "l3.shift")
    inputs = [torch.randn(length, width, generator=generator) for length in lengths]
    state = torch.zeros(3, *part.state_shape(), device=DEVICE)
    state[1] = 5.0

    def run(ctx, pieces):
        return part.forward(torch.cat([inputs[s][a:b] for s, a, b in pieces]).to(DEVICE), ctx, state)
    got = in_steps(lengths, steps, slots, run)
    for s in (0, 1):
        want = plain.blend(inputs[s].double(), mu.double())
        assert float((got[s].double() - want).abs().max()) < (1e-5 if dtype == "float32" else 2e-2)
        assert torch.equal(state[slots[s], 0].cpu(), inputs[s][-1])                  # the input as it was, not what it became
    assert float((state[1] - 5.0).abs().max()) == 0.0


@pytest.mark.parametrize("heads,groups,d,dv,rot,extra", [(4, 2, 16, 24, 8, 4), (3, 1, 10, 10, 0, 3), (6, 3, 32, 32, 32, 0)])
def test_the_placement_multiplies_every_query_head_by_its_number(heads, groups, d, dv, rot, extra):
    from tlie_amd import ops
    generator = torch.Generator().manual_seed(d)
    tokens, page_size = 6, 4
    fused = torch.randn(tokens, (heads + groups) * d + groups * dv + extra, generator=generator)
    numbers = torch.randn(heads, generator=generator)
    positions = torch.tensor([0, 1, 2, 7, 8, 5000], dtype=torch.int32, device=DEVICE)
    slots = torch.tensor([5, 6, 7, 0, 1, -1], dtype=torch.int32, device=DEVICE)
    inv = (100.0 ** (-2.0 * torch.arange(rot // 2, dtype=F64) / rot)).float().to(DEVICE) if rot else None
    shape = (2, 2, groups, page_size * d) if d == dv else (2, groups, page_size * (d + dv))
    plain_cache, cache = torch.zeros(shape, device=DEVICE), torch.zeros(shape, device=DEVICE)
    args = (positions, slots, inv, rot)
    product = ops.Product(fused.to(DEVICE), 1)
    without = ops.qkv_place(product, *args, plain_cache, heads, groups, d, dv, torch.float32, extra_cols=extra)
    got = ops.qkv_place(product, *args, cache, heads, groups, d, dv, torch.float32, extra_cols=extra, head_scale=numbers.to(DEVICE))
    want = without.cpu().double().reshape(tokens, heads, d) * numbers.double()[None, :, None]
    assert float((got.cpu().double().reshape(tokens, heads, d) - want).abs().max()) < 1e-5
    assert torch.equal(cache, plain_cache)                                                # keys and values as they were
    turned = fused[:, :heads * d].double().reshape(tokens, heads, d)
    if rot:
        turned = plain.rotate_halves(turned, positions.cpu(), rot, 100.0)
    assert float((got.cpu().double().reshape(tokens, heads, d) - turned * numbers.double()[None, :, None]).abs().max()) < 1e-3


@pytest.mark.parametrize("heads,groups,d,rot,extra", [(4, 2, 16, 8, 8), (3, 1, 32, 32, 5), (6, 3, 64, 0, 0), (2, 2, 48, 16, 3)])
@pytest.mark.parametrize("dtype", DTYPES)
def test_rotation_and_cache_write_with_a_number_a_head_and_columns_beside(heads, groups, d, rot, extra, dtype):
    """The kernel for any step, and for few rows the product that does the same itself: against the placement of any sizes,
    with the weight's rows in paired order."""
    from tlie_amd import ops
    activation = torch.float32 if dtype == "float32" else torch.bfloat16
    generator = torch.Generator().manual_seed(d + extra)
    tokens, page_size, inner = 6, 16, 128
    placed = (heads + 2 * groups) * d
    x, w = torch.randn(tokens, inner, generator=generator).to(activation), (torch.randn(placed + extra, inner, generator=generator) / 11.0).to(activation)
    numbers = torch.randn(heads, generator=generator).to(DEVICE)
    positions = torch.tensor([0, 1, 2, 7, 8, 500], dtype=torch.int32, device=DEVICE)
    slots = torch.tensor([5, 6, 7, 0, 1, -1], dtype=torch.int32, device=DEVICE)
    inv = (100.0 ** (-2.0 * torch.arange(rot // 2, dtype=F64) / rot)).float().to(DEVICE) if rot else None
    order = torch.cat([ops.paired_rows(heads, groups, d, rot), torch.arange(placed, placed + extra)]) if rot else torch.arange(placed + extra)
    caches = [torch.zeros(2, 2, groups, page_size * d, dtype=activation, device=DEVICE) for _ in range(3)]
    full = (x.double() @ w.double().T).float()
    want = ops.qkv_place(ops.Product(full.to(DEVICE), 1), positions, slots, inv, rot, caches[0], heads, groups, d, d, activation, extra_cols=extra,
                         head_scale=numbers)
    got = ops.rope_cache(ops.Product(full[:, order].to(DEVICE).contiguous(), 1), positions, slots, inv, rot, caches[1], heads, groups, d, activation,
                         paired=rot > 0, extra_cols=extra, head_scale=numbers)
    assert float((got.float() - want.float()).abs().max()) <= (2e-6 if dtype == "float32" else 1e-2) * float(want.abs().max())
    assert float((caches[0].float() - caches[1].float()).abs().max()) <= (2e-6 if dtype == "float32" else 1e-2) * float(caches[0].abs().max())
    if dtype == "bfloat16":
        target = ops.RopeTarget(positions, slots, inv, rot, caches[2], heads, groups, d, extra_cols=extra, head_scale=numbers)
        got = ops.gemm_rows(x.to(DEVICE), w[order].to(DEVICE).contiguous(), None, "rope", rope=target)
        if extra:
            got, beside = got
            assert float((beside.dense().cpu() - full[:, placed:]).abs().max()) < 1e-4
        assert float((got.float() - want.float()).abs().max()) <= 1e-2 * float(want.abs().max())
        assert float((caches[0].float() - caches[2].float()).abs().max()) <= 1e-2 * float(caches[0].abs().max())


def _scale_matrix(tokens, experts, columns, top, generator, unused=()):
    scale = torch.zeros(tokens, columns)
    for t in range(tokens):
        count = int(torch.randint(0, top + 1, (1,), generator=generator))
        usable = [e for e in torch.randperm(experts, generator=generator).tolist() if e not in unused][:count]
        scale[t, usable] = torch.rand(len(usable), generator=generator) + 0.1
    scale[:, experts:] = 9.0                                                # (columns after the experts' are someone else's)
    return scale


@pytest.mark.parametrize("tokens,experts,columns,top,unused", [(300, 7, 8, 3, (2,)), (1, 3, 3, 1, ()), (1500, 70, 71, 5, (0, 69)), (65, 130, 130, 2, ()),
                                                               (40, 4, 4, 4, (0, 1, 2, 3)), (2048, 2, 2, 1, (0,))])
def test_the_plan_of_pairs(tokens, experts, columns, top, unused):
    from tlie_amd import ops
    generator = torch.Generator().manual_seed(tokens + experts)
    scale = _scale_matrix(tokens, experts, columns, top, generator, unused)
    plan = ops.route_plan(scale.to(DEVICE), experts, top)
    for e in range(experts):
        users = scale[:, e].nonzero().flatten()
        assert int(plan.counts[e]) == len(users)
        assert torch.equal(plan.lists[e, :len(users)].cpu().long(), users)
        assert torch.equal(plan.ranks[users.to(DEVICE), e].cpu().long(), torch.arange(len(users)))


@pytest.mark.parametrize("tokens,experts,columns,top,width,size,unused", [
    (300, 7, 8, 3, 128, 64, (2,)), (1, 3, 4, 1, 64, 192, ()), (700, 5, 5, 2, 192, 128, (0, 4)), (150, 70, 70, 4, 64, 64, (3,)), (500, 2, 3, 1, 320, 64, ()),
    (20, 4, 4, 4, 64, 64, (0, 1, 2, 3))])
def test_products_over_the_pairs_of_experts_and_tokens(tokens, experts, columns, top, width, size, unused):
    """Experts that no token uses, that few and that many use (more and less than a tile, no multiple of one), tokens that
    use none, against each expert alone; the pairs of one token alone give the same bits as among all."""
    from tlie_amd import ops
    generator = torch.Generator().manual_seed(tokens)
    scale = _scale_matrix(tokens, experts, columns, top, generator, unused)
    x = torch.randn(tokens, width, generator=generator).bfloat16()
    up = (torch.randn(experts * size, width, generator=generator) / math.sqrt(width)).bfloat16()
    down = (torch.randn(width, experts * size, generator=generator) / math.sqrt(size)).bfloat16()
    assert ops.routed_tiles_take(up, down, experts)

    def run(rows):
        plan = ops.route_plan(scale[rows].to(DEVICE).contiguous(), experts, top)
        hidden = ops.routed_relu_squared(x[rows].to(DEVICE).contiguous(), up.to(DEVICE), plan)
        return hidden, ops.routed_sum(ops.routed_down(hidden, down.to(DEVICE), plan), plan)
    hidden, got = run(list(range(tokens)))
    want, at = torch.zeros(tokens, width, dtype=F64), 0
    for e in range(experts):
        users = scale[:, e].nonzero().flatten()
        act = plain.relu_squared(x[users].double() @ up[e * size:(e + 1) * size].double().T) * scale[users, e:e + 1].double()
        if len(users):
            assert float((hidden[at:at + len(users)].cpu().double() - act).abs().max()) < 1e-2 * float(act.abs().max())
            want[users] += hidden[at:at + len(users)].cpu().double() @ down[:, e * size:(e + 1) * size].double().T
        at += len(users)
    assert float((got.cpu().double() - want).abs().max()) <= 1e-2 * max(float(want.abs().max()), 1e-30)
    for t in {0, tokens // 2, tokens - 1}:
        assert torch.equal(run([t])[1][0], got[t])


@pytest.mark.parametrize("heads,dv,col,nsplit,dtype", [(4, 24, 7, 1, torch.float32), (3, 5, 0, 2, torch.float32), (8, 64, 16, 1, torch.bfloat16),
                                                       (2, 256, 3, 3, torch.bfloat16)])
def test_a_gate_a_head(heads, dv, col, nsplit, dtype):
    from tlie_amd import ops
    generator = torch.Generator().manual_seed(dv)
    values, pre = torch.randn(7, heads * dv, generator=generator).to(dtype), torch.randn(7, col + heads + 2, generator=generator)
    product = split_product(pre.to(dtype) if nsplit == 1 else pre, nsplit, generator)
    got = ops.head_gate(values.to(DEVICE).clone(), product, col, heads).cpu().double()
    z = (pre.to(dtype) if nsplit == 1 else pre).double()[:, col:col + heads]
    want = values.double() * torch.sigmoid(z).repeat_interleave(dv, dim=1)
    assert float((got - want).abs().max()) < (2e-6 if dtype == torch.float32 else 2e-2)


@pytest.mark.parametrize("heads,dim,vdim,plan,nsplit,dtype", [
    (3, 24, 40, SHORT_STEPS, 2, torch.float32), (1, 160, 16, LONG_STEPS, 1, torch.float32), (4, 32, 64, LONG_STEPS, 1, torch.bfloat16),
    (2, 6, 130, LONG_STEPS, 1, torch.float32)])
def test_the_lightning_scan_reads_silu_of_its_columns(heads, dim, vdim, plan, nsplit, dtype):
    from tlie_amd import ops
    generator = torch.Generator().manual_seed(dim + vdim)
    (lengths, steps), slots = plan, [2, 0]
    decay = torch.tensor([1.0, 0.0, 0.93, 0.5][:heads])
    fused = [torch.randn(length, 2 * heads * dim + heads * vdim, generator=generator).to(dtype) for length in lengths]
    state = torch.zeros(3, *ops.decay_scan_state_shape(heads, dim, vdim), device=DEVICE)
    state[1] = 5.0

    def run(ctx, pieces):
        rows = torch.cat([fused[s][a:b] for s, a, b in pieces])
        product = split_product(rows, nsplit, generator) if dtype == torch.float32 else ops.Product(rows.to(DEVICE).contiguous(), 1)
        return ops.decay_scan((product, 0), (product, heads * dim), (product, 2 * heads * dim), state, ctx.seq_start, ctx.seq_slot,
                              heads, dim, vdim, head_decay=decay.to(DEVICE), max_new=ctx.max_new, activation="silu")
    got = in_steps(lengths, steps, slots, run)
    for s in (0, 1):
        active = plain.silu(fused[s].double())
        q, k = active[:, :heads * dim].reshape(-1, heads, dim), active[:, heads * dim:2 * heads * dim].reshape(-1, heads, dim)
        v = active[:, 2 * heads * dim:].reshape(-1, heads, vdim)
        want = torch.cat([plain.decayed_state_walk(q[:, h], k[:, h], v[:, h], torch.full((lengths[s], dim), float(decay[h]), dtype=F64))
                          for h in range(heads)], dim=1)
        assert float((got[s].double() - want).abs().max()) < 2e-5 * float(want.abs().max()), f"sequence {s}"
    assert float((state[1] - 5.0).abs().max()) == 0.0


@pytest.mark.parametrize("heads,dv,nsplit,dtype", [(1, 40, 1, torch.float32), (1, 520, 2, torch.float32), (1, 6152, 1, torch.bfloat16),
                                                   (2, 1024, 1, torch.bfloat16), (1, 777, 1, torch.float32)])
def test_all_heads_normed_as_one_row(heads, dv, nsplit, dtype):
    from tlie_amd import ops
    generator = torch.Generator().manual_seed(dv)
    tokens, eps = 5, 1e-5
    a = torch.randn(tokens, heads * dv, generator=generator) * 4.0
    a[0] = 1e-3                                                    # a row whose mean square is of eps' size
    gate, weight = torch.randn(tokens, 16 + heads * dv, generator=generator).to(dtype), torch.randn(heads * dv, generator=generator).to(dtype)
    product = split_product(gate, nsplit, generator)
    want = plain.unit_rms(a.double().reshape(tokens, heads, dv), eps).reshape(tokens, -1) * weight.double() * torch.sigmoid(gate.double()[:, 16:])
    got = ops.head_combine(a.to(DEVICE), heads, dv, eps, dtype, weight=weight.to(DEVICE), gate=product, gate_col=16)
    assert float((got.cpu().double() - want).abs().max()) < (5e-5 if dtype == torch.float32 else 5e-2)


def _want_scale(z, correction, top, groups, identities):
    _, chosen, weights = plain.router_choice(z, correction, top, {"count": groups[0], "keep": groups[1]})
    full = torch.zeros_like(z).scatter_(1, chosen, weights)
    experts = z.shape[1] - identities
    return torch.cat([full[:, :experts], full[:, experts:].sum(1, keepdim=True)], dim=1) if identities else full


@pytest.mark.parametrize("tokens,inner,experts,identities,top,groups,dtype", [
    (50, 96, 14, 6, 3, (5, 3), torch.float32), (9, 1000, 13, 3, 16, (4, 4), torch.bfloat16), (30, 80, 6, 0, 1, (3, 1), torch.float32),
    (12, 50, 5, 7, 3, (2, 1), torch.float32), (7, 64, 200, 56, 70, (64, 40), torch.float32), (4, 16, 1, 0, 1, (1, 1), torch.bfloat16)])
def test_the_grouped_router(tokens, inner, experts, identities, top, groups, dtype):
    from tlie_amd import ops
    outputs = experts + identities
    generator = torch.Generator().manual_seed(inner + top)
    x = torch.randn(tokens, inner, generator=generator).to(dtype)
    weight = (2.0 * torch.randn(outputs, inner, generator=generator) / math.sqrt(inner)).to(dtype)
    correction = torch.randn(outputs, generator=generator) * 0.5 - 0.6        # most choice scores are negative
    z = x.double() @ weight.double().T
    assert float(plain.router_margin(z, correction.double(), top, {"count": groups[0], "keep": groups[1]}).min()) > 1e-5
    want = _want_scale(z, correction.double(), top, groups, identities)
    got = ops.grouped_router(x.to(DEVICE), weight.to(DEVICE), correction.to(DEVICE), top, identities, *groups).cpu().double()
    assert float((got - want).abs().max()) < 1e-5
    assert torch.allclose(got.sum(1), torch.ones(tokens, dtype=F64), atol=1e-5)


def test_the_grouped_router_takes_the_lower_of_equals_and_bounds_tiny_sums():
    from tlie_amd import ops
    x = torch.zeros(2, 8, device=DEVICE)                                     # every score the same
    got = ops.grouped_router(x, torch.ones(6, 8, device=DEVICE), None, 2, 1, 3, 2).cpu()
    assert torch.allclose(got, torch.tensor([[0.5, 0.5, 0.0, 0.0, 0.0, 0.0]] * 2))
    # a group whose best is the identity; scores whose chosen ones are next to nothing
    x = torch.ones(1, 4, device=DEVICE)
    weight = torch.zeros(4, 4, device=DEVICE)
    weight[0] = 40.0                                                         # z_0 = 160: the others' scores underflow
    got = ops.grouped_router(x, weight, torch.tensor([-5.0, 0.0, 0.0, 1.0], device=DEVICE), 2, 1, 2, 1).cpu()
    assert torch.isfinite(got).all() and float(got.sum()) == 0.0             # 0 / (0 + 1e-20)


@pytest.mark.parametrize("tokens,blocks,block,nsplit,dtype", [(5, 4, 6, 1, torch.float32), (3, 7, 24, 2, torch.float32), (18, 3, 8, 1, torch.bfloat16),
                                                              (40, 1, 1000, 1, torch.bfloat16)])
def test_squared_relu_with_a_number_a_block(tokens, blocks, block, nsplit, dtype):
    from tlie_amd import ops
    generator = torch.Generator().manual_seed(block)
    z = 2.0 * torch.randn(tokens, blocks * block, generator=generator).to(dtype)
    scale = torch.rand(tokens, blocks + 1, generator=generator)              # (a column more than there are blocks: not read)
    scale[:, 0] = 0.0
    z[0, 0] = math.inf if nsplit == 1 else z[0, 0]                           # what an unused expert would give does not matter
    want = plain.relu_squared(z.double())
    tolerance = 1e-5 if dtype == torch.float32 else 0.2
    finite = torch.isfinite(want)
    got = ops.relu_squared(split_product(z, nsplit, generator), dtype).float().cpu().double()
    assert float((got - want)[finite].abs().max()) < tolerance
    got = ops.relu_squared(split_product(z, nsplit, generator), dtype, scale.to(DEVICE), block).float().cpu().double()
    weighed = torch.where(finite, want, torch.zeros_like(want)) * scale[:, :blocks].double().repeat_interleave(block, dim=1)
    assert bool(torch.isfinite(got).all()) and float((got - weighed).abs().max()) < tolerance


@pytest.mark.parametrize("rows,outputs,inner,block", [(1, 96, 64, 24), (8, 1000, 136, 100), (16, 72, 2048, 8), (9, 4096, 64, 512), (5, 30, 200, 30)])
def test_products_of_few_rows_apply_the_squared_relu_themselves(rows, outputs, inner, block):
    from tlie_amd import ops
    generator = torch.Generator().manual_seed(outputs)
    x = torch.randn(rows, inner, generator=generator).bfloat16()
    w = (torch.randn(outputs, inner, generator=generator) / math.sqrt(inner)).bfloat16()
    scale = torch.rand(rows, -(-outputs // block), generator=generator)
    scale[0, 0] = 0.0
    want = plain.relu_squared(x.double() @ w.double().T)
    got = ops.gemm_rows(x.to(DEVICE), w.to(DEVICE), None, "relu2").float().cpu().double()
    assert float((got - want).abs().max()) < 1e-2 * float(want.max())
    got = ops.gemm_rows(x.to(DEVICE), w.to(DEVICE), None, "relu2", act_scale=scale.to(DEVICE), act_block=block).float().cpu().double()
    weighed = want * scale.double().repeat_interleave(block, dim=1)[:, :outputs]
    assert float((got - weighed).abs().max()) < 1e-2 * float(want.max())
    assert float(got[0, :block].abs().max()) == 0.0


@pytest.mark.parametrize("batch,rows,outputs,inner", [(4, 8, 96, 128), (1, 1, 40, 64), (3, 16, 2048, 72), (5, 3, 17, 1000)])
def test_several_products_of_one_shape_in_one_launch(batch, rows, outputs, inner):
    from tlie_amd import ops
    generator = torch.Generator().manual_seed(outputs)
    x = torch.randn(batch, rows, inner, generator=generator).bfloat16()
    w = (torch.randn(batch, outputs, inner, generator=generator) / math.sqrt(inner)).bfloat16()
    for index, got in enumerate(ops.gemm_rows_batch(x.to(DEVICE), w.to(DEVICE))):
        want = x[index].double() @ w[index].double().T
        assert float((got.dense().cpu().double() - want).abs().max()) < 1e-4


@pytest.mark.parametrize("tokens,window,context", [(3, 20, 500), (8, 100, 3000), (2, 1024, 5000), (1, 40, 30)])
def test_a_decode_step_over_a_window_shares_the_windows_keys(tokens, window, context):
    """Long sequences and a short window: the parts of the keys lie in the window, wherever it begins, and no key is left
    out or taken twice; one key at the window's edge, just inside or just outside, towers over the rest."""
    from tlie_amd import ops
    generator = torch.Generator().manual_seed(window)
    heads, groups, d, page_size = 4, 2, 32, 16
    blocks = -(-context // page_size)
    lengths = [context - 37 * index for index in range(tokens)] if context > 400 else [context] * tokens
    ctx = SimpleNamespace(max_new=1, num_seqs=tokens, num_tokens=tokens, max_context=context, scratch={}, tile_owner=None, compute_units=256, host={})
    plan = ops.attention_plan(ctx, heads // groups, groups, d, window)
    assert plan[2] == 1 or plan[2] * plan[3] < context or window + 31 >= context
    tiles, col_tiles, nsplit, split_len, waves, shared = plan
    k, v = (torch.randn(tokens, context, groups, d, generator=generator).bfloat16() for _ in range(2))
    q = torch.randn(tokens, heads, d, generator=generator).bfloat16()
    positions = torch.tensor([length - 1 for length in lengths], dtype=torch.int32, device=DEVICE)
    table = torch.randperm(tokens * blocks, generator=generator).to(torch.int32).view(tokens, blocks)
    for back in (window - 1, window, 0):                          # the towering key, so many positions before the token
        keys = k.clone()
        for t, length in enumerate(lengths):
            if length - 1 - back >= 0:
                keys[t, length - 1 - back] = 4.0 * q[t].float().reshape(groups, heads // groups, d).mean(dim=1).bfloat16()
        cache = torch.zeros(tokens * blocks, 2, groups, page_size * d, dtype=torch.bfloat16)
        for t in range(tokens):
            for b in range(blocks):
                rows = slice(b * page_size, min((b + 1) * page_size, context))
                count = rows.stop - rows.start
                page = cache[int(table[t, b])]
                page[0].view(groups, page_size, d)[:, :count] = keys[t, rows].transpose(0, 1)
                page[1].view(groups, d, page_size)[:, :, :count] = v[t, rows].permute(1, 2, 0)
        got = ops.attention_mfma(q.reshape(tokens, -1).to(DEVICE), cache.to(DEVICE), table.to(DEVICE), tiles, positions, heads, groups, d, window, 0.3,
                                 nsplit, split_len, col_tiles, waves, shared).float().cpu().reshape(tokens, heads, d)
        for t, length in enumerate(lengths):
            lo = max(0, length - window)
            for h in range(heads):
                weights = torch.softmax(0.3 * keys[t, lo:length, h // 2].double() @ q[t, h].double(), dim=0)
                want = weights @ v[t, lo:length, h // 2].double()
                assert float((got[t, h].double() - want).abs().max()) < 3e-2, f"token {t}, head {h}, key {back} back"


@pytest.mark.parametrize("width,dtype", [(64, torch.float32), (50, torch.float32), (2056, torch.bfloat16), (30, torch.bfloat16)])
def test_what_a_pass_begins_with(width, dtype):
    from tlie_amd import ops
    generator = torch.Generator().manual_seed(width)
    residual, table = torch.randn(7, width, generator=generator), torch.randn(20, width, generator=generator).to(dtype)
    tokens = torch.tensor([3, 19, 0, 3, 7, 11, 1], dtype=torch.int32)
    got = ops.pass_input(residual.to(DEVICE), tokens.to(DEVICE), table.to(DEVICE), dtype).cpu()
    assert torch.equal(got, torch.cat([residual.to(dtype), table[tokens.long()]], dim=1))


# ---- single layers through the engine: a mixer's result from its input, and inputs made so that a fault shows ---------
def _single_layer(tmp_path, layer, seed, vocab=97, width=48, changes=None, settled=False, **keys):
    raw = {"architecture": "Paluzen", "vocab": vocab, "width": width, "norm": {"eps": 1e-5}, "layers": [layer], **keys}
    folder = make_model(tmp_path, raw, seed=seed, settled=settled)
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


PARALLELS = [
    parallel((4, 2, 16, 24, 0.3), (3, 24), (1.3, 0.5), window=9, rot=(500.0, 8)),
    parallel((6, 6, 32, 32, 0.2), (1, 72), (-0.4, 1.0), window=150, rot=(10000.0, 32)),
    parallel((2, 1, 8, 70, 0.5), (2, 160), (0.6, -1.2), rot=(20.0, 4)),
    parallel((8, 2, 96, 96, 0.1), (5, 8), (1.0, 0.0), window=16, rot=(10000.0, 40)),         # the left side alone
    parallel((2, 2, 16, 16, 0.25), (2, 64), (0.0, 1.0), window=1),                           # the right side alone
]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("mixer", PARALLELS)
def test_windowed_attention_beside_token_shift_mixing(tmp_path, mixer, dtype):
    folder, config, weights = _single_layer(tmp_path, {"type": "parallel", "mixer": mixer, "mlp": None}, seed=9, settled=dtype == "bfloat16",
                                            changes=lambda w: w["l0.mix.left.temp"].mul_(torch.linspace(0.4, 2.5, w["l0.mix.left.temp"].numel(), dtype=F64)))
    tokens = tokens_of(10, 300, 97)             # (long enough for the keys to be cut into parts that are merged)
    for cuts in ([300], [33, 1, 2, 20, 150], [280] + [1] * 20):
        h, got = _traced(folder, tokens, dtype, cuts, ["input_norm", "attention_output"])
        want = plain.parallel(mixer, weights, "l0.mix.", h, torch.arange(len(tokens)), 1e-5)
        assert_rows(got, want, SINGLE_LAYER_TOLERANCE[dtype], f"cuts {cuts[:5]}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("mixer", [lightning(16, 20, [0.9, 0.99, 0.5]), lightning(130, 8, [0.998]), lightning(6, 70, [1.0, 0.0, 0.75, 0.96]),
                                   lightning(64, 128, [0.97, 0.999, 0.3, 0.6, 0.9])])
def test_lightning_attention_alone(tmp_path, mixer, dtype):
    folder, config, weights = _single_layer(tmp_path, {"type": "lightning", "mixer": mixer, "mlp": None}, seed=7)
    tokens = tokens_of(8, 150, 97)
    for cuts in ([150], [30, 1, 2, 9, 100], [1]):
        h, got = _traced(folder, tokens, dtype, cuts, ["input_norm", "attention_output"])
        assert_rows(got, plain.lightning(mixer, weights, "l0.mix.", h, None, 1e-5), SINGLE_LAYER_TOLERANCE[dtype], f"cuts {cuts}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("mlp,width", [(dense(40), 48), (dense(264), 48), (moe(6, 3, 16, groups=(4, 2), identity=2), 48), (moe(5, 1, 13, identity=1), 48),
                                       (moe(4, 4, 24), 48), (moe(9, 3, 64, groups=(4, 3), identity=3), 64), (moe(4, 2, 128), 128)])
def test_feed_forwards_alone(tmp_path, mlp, width, dtype):
    """A layer's second sublayer from its input, and what the mixer reads: the shift's result does not depend on the cut."""
    layer = {"type": "lightning", "mixer": lightning(8, 8, [0.9, 0.5]), "mlp": mlp}
    folder, config, weights = _single_layer(tmp_path, layer, seed=15, width=width)
    tokens = tokens_of(16, 100, 97)
    first = None
    for cuts in ([100], [2], [1], [9, 1, 30]):
        h0, h, got = _traced(folder, tokens, dtype, cuts, ["input_norm", "post_attention_norm", "mlp_output"])
        margins = []
        want = plain.feed_forward(mlp, weights, "l0.mlp.", h, margins)
        # (with the engine's own input, only calls closer than float sums' rounding are open)
        rows = torch.arange(len(tokens)) if not margins else (margins[0] > 1e-5).nonzero().flatten()
        assert len(rows) > 95
        assert_rows(got[rows], want[rows], SINGLE_LAYER_TOLERANCE[dtype], f"cuts {cuts}")
        if first is None:
            first = h0
            x = weights["embed"][torch.tensor(tokens)]
            assert_rows(h0, plain.blend(plain.rms_norm(x, weights["l0.norm1"], 1e-5), weights["l0.shift"]), 1e-5 if dtype == "float32" else 1e-2, "the shift")
        else:
            assert_rows(h0, first, 1e-6 if dtype == "float32" else 1e-2, f"the shift's result, cuts {cuts}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("dim,vdim", [(12, 20), (16, 16)])          # the plain attention kernel, and in bfloat16 the matrix cores'
@pytest.mark.parametrize("window", [37, 64, None])
def test_one_key_decides_the_result_inside_the_window_and_not_outside(tmp_path, dtype, dim, vdim, window):
    """One head is made to look at one position only: token B's key and token A's query are large in a dim that does not
    turn.  B stands just inside or just outside A's window, at a page's first or last row, or hundreds of positions back
    (without a window); A comes last, in a prompt's portion and decoded alone."""
    A, B, length = 95, 96, 300
    mixer = parallel((2, 1, dim, vdim, 0.3), (2, 8), (1.0, 0.2), window=window, rot=(100.0, 8))

    def boost(weights):
        weights["l0.shift"][:] = 0.0                              # a mixer reads the token alone
        h = lambda token: plain.rms_norm(weights["embed"][token], weights["l0.norm1"], 1e-5)        # noqa: E731
        a, b = h(A), h(B)
        weights["l0.mix.left.q"][10] = 16.0 * a / (a @ a)         # head 0, dim 10 (past the rotated 8)
        weights["l0.mix.left.k"][10] = 16.0 * b / (b @ b)
        weights["l0.mix.left.g"][0] = 3.0 * a / (a @ a)           # and its gate is open for A
        weights["l0.mix.left.o"] *= 4.0
    folder, config, weights = _single_layer(tmp_path, {"type": "parallel", "mixer": mixer, "mlp": None}, seed=11, changes=boost)
    from tlie_amd import Engine
    engine = Engine(folder, dtype=dtype, max_tokens=640, page_size=16, max_requests=2)
    last = length - 1
    if window is None:
        places = {far: True for far in (0, 1, 15, 16, 250)}
    else:
        places = {last - window + 1: True, last - window: False, last - 1: True, last - window - 1: False}
    for far, inside in places.items():
        tokens = tokens_of(12, length, 97, avoid=(A, B))
        tokens[far], tokens[-1] = B, A
        other = list(tokens)
        other[far] = next(token for token in range(97) if token not in (A, B, tokens[far + 1] if far + 1 < length else A))
        want, lost = plain.forward(config, weights, tokens)[0], plain.forward(config, weights, other)[0]
        moved = float(row_errors(lost[-1:], want[-1:]))
        assert moved > 0.15 if inside else moved < 0.1, f"B at {far}: {moved}"            # the test shows a key that is lost
        for cuts in ([length], [length - 1, 1], [7, 64, 2]):
            got = run_cut(engine, "a", tokens, cuts)
            assert_rows(got[-1:], want[-1:], SINGLE_LAYER_TOLERANCE[dtype], f"B at {far}, cuts {cuts}")


@pytest.mark.parametrize("dtype", DTYPES)
def test_windows_pass_over_decoded_tokens(tmp_path, dtype):
    """The same head; A asks again and again while B, which came in a decoded step too, leaves its window."""
    A, B, window = 95, 96, 40
    mixer = parallel((2, 1, 16, 16, 0.3), (2, 8), (1.0, 0.2), window=window, rot=(100.0, 8))

    def boost(weights):
        weights["l0.shift"][:] = 0.0
        h = lambda token: plain.rms_norm(weights["embed"][token], weights["l0.norm1"], 1e-5)        # noqa: E731
        a, b = h(A), h(B)
        weights["l0.mix.left.q"][10] = 16.0 * a / (a @ a)
        weights["l0.mix.left.k"][10] = 16.0 * b / (b @ b)
        weights["l0.mix.left.g"][0] = 3.0 * a / (a @ a)
        weights["l0.mix.left.o"] *= 4.0
    folder, config, weights = _single_layer(tmp_path, {"type": "parallel", "mixer": mixer, "mlp": None}, seed=11, changes=boost)
    tokens = tokens_of(31, 160, 97, avoid=(A, B))
    tokens[70] = B
    asks = [71, 95, 108, 109, 110, 111, 150]                    # 109 = 70 + 39 sees B, 110 does not
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
@pytest.mark.parametrize("kind", ["lightning", "parallel"])
def test_what_the_state_took_in_long_ago_is_still_there(tmp_path, dtype, kind):
    """Decays close to 1, and a key and value written at the third token that stand out: token B alone has a large
    channel 0, which its key's dim 10 and its value read, and token A alone a large channel 1, which the query's dim 10
    reads.  A comes last.  A state that is lost or zeroed on the way (between steps, at a slice's edge, in a slot that is
    used again) changes the last tokens' results."""
    A, B, length = 95, 96, 260
    if kind == "lightning":
        mixer = lightning(12, 12, [0.9995, 0.9])
        q, k, v, o = ("l0.mix." + name for name in "qkvo")
    else:
        mixer = parallel((2, 1, 8, 8, 0.3), (2, 12), (0.2, 1.0), window=20, rot=(100.0, 8))
        q, k, v, o = ("l0.mix.right." + name for name in "rkvo")

    def boost(weights):
        weights["l0.shift"][:] = 0.0
        weights["embed"][:, :2] = 0.0
        weights["embed"][B, 0], weights["embed"][A, 1] = 4.0, 4.0
        weights[q][10], weights[k][10] = 0.0, 0.0
        weights[q][10, 1], weights[k][10, 0] = 3.0, 3.0          # head 0, dim 10
        weights[v][:12, 0] = torch.linspace(-2.0, 2.0, 12, dtype=F64)
        weights[o] *= 12.0
        if kind == "parallel":
            weights["l0.mix.right.w0"][:] = -9.0                 # exp(-exp(-9)) a token
            for blend in "rkv":
                weights["l0.mix.right.mu." + blend][:] = 0.0     # they read the token itself
    folder, config, weights = _single_layer(tmp_path, {"type": kind, "mixer": mixer, "mlp": None}, seed=13, changes=boost)
    tokens = tokens_of(14, length, 97, avoid=(A, B))
    tokens[2], tokens[-1] = B, A
    other = list(tokens)
    other[2] = tokens[3]
    want, lost = plain.forward(config, weights, tokens)[0], plain.forward(config, weights, other)[0]
    assert float(row_errors(lost[-1:], want[-1:]).min()) > 0.05                     # the test shows a state that is lost
    from tlie_amd import Engine
    engine = Engine(folder, dtype=dtype, max_tokens=640, page_size=16, max_requests=1)      # one slot: used again by every cut
    for cuts in ([length], [length - 40] + [1] * 40, [5, 64, 2, 1], [3, 96, 33, 97]):
        got = run_cut(engine, "a", tokens, cuts)
        assert_rows(got[-2:], want[-2:], SINGLE_LAYER_TOLERANCE[dtype], f"cuts {cuts[:4]}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("loop", [None, {"start": 0, "stop": 1, "times": 2}])
def test_the_first_tokens_of_a_request_see_nothing_of_the_slots_last_owner(tmp_path, dtype, loop):
    """One slot, two requests after each other: the second's first tokens (whose shifts and states start from zeros) equal
    the plain implementation's, and differ from what a kept state would give."""
    from tlie_amd import Engine
    mixer = parallel((2, 1, 8, 8, 0.3), (2, 12), (0.7, 1.0), window=11, rot=(100.0, 8))
    keys = {"loop": loop} if loop else {}
    folder, config, weights = _single_layer(tmp_path, {"type": "parallel", "mixer": mixer, "mlp": dense(40)}, seed=21, **keys)
    first, second = tokens_of(22, 50, 97), tokens_of(23, 9, 97)
    want = plain.forward(config, weights, second)[0]
    joined = plain.forward(config, weights, first + second)[0][len(first):]
    assert float(row_errors(joined[:1], want[:1])) > 0.02
    engine = Engine(folder, dtype=dtype, max_tokens=64, page_size=16, max_requests=1)
    for cuts in ([9], [1], [2, 1]):
        run_cut(engine, "x", first, [50])
        got = run_cut(engine, "y", second, cuts)
        assert_rows(got, want, SINGLE_LAYER_TOLERANCE[dtype], f"cuts {cuts}")


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
def test_every_layer_run_matches_the_plain_implementation(setups, name):
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
        assert float((got - residuals[index]).abs().max()) < 3e-5 * scale, f"{name}: the residual after layer run {index}"


@pytest.mark.parametrize("name,dtype", CASES)
def test_cuts_agree_with_each_other_and_with_the_plain_implementation(setups, name, dtype):
    """Whole, token by token from the first token, in portions of two, and in portions of changing sizes that end inside
    pages, windows and the scans' slices."""
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
    setup = setups("V")
    prompts = [tokens_of(90 + index, 40, CONFIGS["V"]["vocab"]) for index in range(4)]
    want = [plain_generate_greedy(setup["raw"], setup["weights"], prompt, 20) for prompt in prompts]
    engine = new_engine(setup, "float32", max_tokens=176, max_requests=4)
    assert engine.generate(prompts, max_tokens=20, admit_partial=True) == want
    engine.cache.check()


@pytest.mark.parametrize("name,dtype", [("U", "float32"), ("W", "float32"), ("W", "bfloat16")])
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
    setup = setups("U")
    vocab = CONFIGS["U"]["vocab"]
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
        made = setups("U", dtype)
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
    layers = []
    for _ in range(rng.randint(1, 4)):
        kind = rng.choice(["parallel", "lightning"])
        if kind == "parallel":
            groups = rng.choice([1, 2, 3])
            dim = rng.choice([4, 6, 10, 16, 24, 32, 48, 64, 80])
            left = (groups * rng.choice([1, 2, 4]), groups, dim, rng.choice([dim, dim, 5, 12, 40]), rng.choice([0.1, 0.25, 0.4]) * (16.0 / dim) ** 0.5)
            rot = (rng.choice([10.0, 1000.0, 500000.0]), rng.choice([d for d in (2, 4, dim - dim % 2) if d <= dim])) if rng.random() < 0.8 else None
            mixer = parallel(left, (rng.choice([1, 2, 5]), rng.choice([3, 8, 20, 33, 64])), (rng.choice([-1.0, 0.5, 1.0]), rng.choice([0.3, 1.0, -0.7])),
                             window=rng.choice([None, 1, 2, 5, 16, 17, 33, 64]), rot=rot)
        else:
            mixer = lightning(rng.choice([3, 8, 16, 40, 96]), rng.choice([4, 16, 65, 128]), [rng.choice([0.0, 0.5, 0.9, 0.999, 1.0]) for _ in range(rng.choice([1, 2, 5]))])
        mlp = None
        if rng.random() < 0.85:
            if rng.random() < 0.3:
                mlp = dense(rng.choice([3, 40, 150]))
            else:
                count = rng.choice([1, 2, 3, 4])
                outputs = count * rng.choice([1, 2, 5])
                identity = rng.randint(0, outputs - 1)
                keep = rng.randint(1, count)
                mlp = moe(outputs - identity, rng.randint(1, keep * outputs // count), rng.choice([3, 8, 20, 33]),
                          groups=(count, keep) if count > 1 or rng.random() < 0.5 else None, identity=identity or rng.choice([None, 0]))
        layers.append({"type": kind, "mixer": mixer, "mlp": mlp})
    raw = {"architecture": "Paluzen", "vocab": rng.choice([31, 100, 257]), "width": width, "norm": {"eps": rng.choice([1e-6, 1e-5, 1e-3])}, "layers": layers}
    if rng.random() < 0.6:
        raw["logit_softcap"] = rng.choice([2.0, 15.0, 50.0])
    if rng.random() < 0.7:
        start = rng.randrange(len(layers))
        raw["loop"] = {"start": start, "stop": rng.randint(start + 1, len(layers)), "times": rng.randint(1, 3)}
    return raw


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
    folder = make_model(tmp_path / "model", raw, seed=seed, settled=True)
    config, weights = load_plain(folder)
    setup = {"raw": config, "weights": weights, "dtype": "bfloat16", "plain": {}, "allowed": {}}
    tokens = tokens_of(seed, 90, raw["vocab"])
    engine = Engine(folder, dtype="bfloat16", max_tokens=128, page_size=16, max_requests=2)
    assert_plain(run_cut(engine, "w", tokens, [len(tokens)]), setup, tokens, f"seed {seed} whole: {raw}")
    assert_plain(run_cut(engine, "c", tokens, [70] + [1] * 20), setup, tokens, f"seed {seed} decoded: {raw}")
    engine.cache.check()
