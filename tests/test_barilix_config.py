"""The Barilix decoder on the CPU: config.json to the model as data, the tensors it expects, what is refused, and pieces
of the plain implementation against cases worked out by hand."""
import copy
import math
import re

import pytest
import torch

import plain_barilix as plain
from barilix_helpers import CONFIGS, CONFIG_R, CONFIG_S, CONFIG_T

F64 = torch.float64


def spec_of(raw):
    from tlie_amd.registry import config_from_dict
    return config_from_dict(raw).to_spec()


def test_the_configuration_becomes_the_model_as_data():
    spec = spec_of(CONFIG_R)
    assert (spec.architecture, spec.hidden_size, spec.vocab_size, spec.max_positions) == ("Barilix", 72, 181, None)
    assert spec.embedding["scale"] == 3.5 and not spec.head["tied"]
    assert [run.layer for run in spec.runs] == [0, 1, 2, 3] and all(run.cache_of == index for index, run in enumerate(spec.runs))
    assert all(layer.block == "post_norm" and layer.mixer_norm.kind == "layer_norm" and layer.mixer_norm["bias"] is False for layer in spec.layers)
    first, second, third, fourth = spec.layers
    left, right = first.mixer["left"], first.mixer["right"]
    assert (first.mixer.kind, first.mixer["scale"], first.mixer["result_norm_eps"]) == ("side_by_side", 0.5, 1e-5)
    assert (left.kind, left["window"], left["conv"], left["qk_norm"], left["value_dim"], left["scale"], left["bias"]) == ("attention", 7, 3, "head", 24, 0.3, True)
    position = left["position"]
    assert (position.kind, position["rot_dim"], position["theta"]) == ("rotary", 8, 90.0)
    assert position["wavelength_scaling"] == {"factor": 3.0, "low": 0.5, "high": 2.0, "original": 40.0}
    assert [right[key] for key in ("num_heads", "head_dim", "state_size", "groups", "norm_groups", "taps")] == [6, 10, 12, 3, 2, 5]
    assert (first.feed_forward.kind, first.feed_forward["intermediate_size"]) == ("gated_mlp", 56)
    assert [second.mixer[key] for key in ("num_heads", "num_kv_heads", "head_dim", "value_dim", "taps")] == [6, 2, 24, 40, 2]
    mlp = second.feed_forward
    assert [mlp[key] for key in ("experts", "top", "expert_size", "shared_size", "score", "vocab_size", "weigh")] == [5, 3, 24, 40, "table", 181, "output"]
    assert third.feed_forward is None and third.mixer["left"]["position"].get("wavelength_scaling") is None
    assert fourth.feed_forward["shared_size"] == 0


def test_what_config_json_leaves_out_is_absent():
    spec = spec_of(CONFIG_S)
    assert spec.layers[1].mixer["left"]["window"] is None and spec.layers[1].mixer["left"]["position"].kind == "none"


def test_the_expected_tensors_carry_the_designs_names_and_shapes():
    from tlie_amd.models.builder import expected_tensors
    shapes = {tensor.name: tensor.shape for tensor in expected_tensors(spec_of(CONFIG_R))}
    assert shapes["embed"] == (181, 72) and shapes["head"] == (181, 72) and shapes["final.norm"] == (72,)
    assert shapes["l0.norm1"] == (72,) and shapes["l0.norm2"] == (72,) and "l0.norm1.b" not in shapes
    assert shapes["l0.mix.left.q"] == (64, 72) and shapes["l0.mix.left.k.b"] == (32,) and shapes["l0.mix.left.v"] == (48, 72)
    assert shapes["l0.mix.left.q.conv"] == (64, 3) and shapes["l0.mix.left.v.conv"] == (48, 3) and shapes["l0.mix.left.k.norm"] == (16,)
    assert shapes["l0.mix.left.o"] == (72, 96) and shapes["l0.mix.left.o.b"] == (72,)
    assert shapes["l0.mix.left.out"] == (72,) and shapes["l0.mix.right.out"] == (72,)
    assert shapes["l0.mix.right.in"] == (60 + 60 + 72 + 6, 72) and shapes["l0.mix.right.conv"] == (132, 5) and shapes["l0.mix.right.conv.b"] == (132,)
    assert shapes["l0.mix.right.A_log"] == shapes["l0.mix.right.D"] == shapes["l0.mix.right.dt_bias"] == (6,)
    assert shapes["l0.mix.right.norm"] == (60,) and shapes["l0.mix.right.o"] == (72, 60)
    assert shapes["l0.mlp.gate"] == (56, 72) and shapes["l0.mlp.down"] == (72, 56)
    assert shapes["l1.mix.q"] == (48, 72) and shapes["l1.mix.v.conv"] == (240, 2) and shapes["l1.mix.b"] == (6, 72) and shapes["l1.mix.norm"] == (40,)
    assert shapes["l1.mix.g"] == (240, 72) and shapes["l1.mix.o"] == (72, 240) and "l1.mix.q.b" not in shapes
    assert shapes["l1.mlp.table"] == (181, 3) and shapes["l1.mlp.e4.up"] == (24, 72) and shapes["l1.mlp.shared.down"] == (72, 40)
    assert "l1.mlp.e5.up" not in shapes and "l1.mlp.router" not in shapes and "l3.mlp.shared.up" not in shapes
    assert "l2.norm2" not in shapes                                                     # a layer without a feed-forward
    assert any(re.fullmatch(pattern, "l2.norm2") for pattern in spec_of(CONFIG_R).ignored_tensors)      # (a file may still carry it)
    assert not any(re.fullmatch(pattern, "l1.norm2") for pattern in spec_of(CONFIG_R).ignored_tensors)


def test_random_tables_name_distinct_experts():
    from tlie_amd.models.builder import expected_tensors
    from tlie_amd.weights.random_init import random_tensors
    table = random_tensors(expected_tensors(spec_of(CONFIG_R)), seed=3)["l1.mlp.table"]
    assert table.dtype == torch.int32 and table.shape == (181, 3) and int(table.min()) >= 0 and int(table.max()) < 5
    assert all(len(set(row)) == 3 for row in table.tolist()) and len(set(table[:, 0].tolist())) == 5


@pytest.mark.parametrize("change,message", [
    (lambda raw: raw["layers"][0].update(type="retention"), "not one of"),
    (lambda raw: raw["layers"][0]["mixer"]["left"].update(kv_heads=3), "multiple"),
    (lambda raw: raw["layers"][0]["mixer"]["left"]["rot"].update(dims=7), "even"),
    (lambda raw: raw["layers"][0]["mixer"]["left"]["rot"]["scaling"].update(low=2.5), "low"),
    (lambda raw: raw["layers"][0]["mixer"]["left"]["mask"].update(size=0), "positive"),
    (lambda raw: raw["layers"][0]["mixer"]["left"].pop("conv"), "conv"),
    (lambda raw: raw["layers"][0]["mixer"]["right"].update(groups=4), "groups"),
    (lambda raw: raw["layers"][0]["mixer"]["right"].update(norm_groups=7), "norm_groups"),
    (lambda raw: raw["layers"][1]["mixer"].update(kv_heads=4), "multiple"),
    (lambda raw: raw["layers"][1]["mlp"]["router"].update(top=6), "cannot use"),
    (lambda raw: raw["layers"][1]["mlp"]["shared"].update(ff=0), "positive"),
    (lambda raw: raw["layers"][3]["mlp"].update(kind="gated"), "kind"),
    (lambda raw: raw.pop("embedding"), "scale"),
    (lambda raw: raw["norm"].pop("eps"), "eps"),
])
def test_configurations_that_are_refused(change, message):
    from tlie_amd import EngineError
    raw = copy.deepcopy(CONFIG_R)
    change(raw)
    with pytest.raises(EngineError, match=message):
        spec_of(raw)


def test_a_scaled_embedding_does_not_go_with_runs_that_take_its_rows_again():
    import dataclasses
    from tlie_amd import EngineError
    spec = spec_of(CONFIG_T)
    runs = (dataclasses.replace(spec.runs[0], add_embedding=True), *spec.runs[1:])
    with pytest.raises(EngineError, match="not scaled"):
        dataclasses.replace(spec, runs=runs).validate()


def test_every_configuration_of_the_tests_is_read():
    for raw in CONFIGS.values():
        spec_of(raw)


def test_frequencies_are_kept_slowed_down_and_blended_by_their_wavelengths():
    """Against the plain formula, and that all three cases occur."""
    from tlie_amd.config.spec import PartSpec
    from tlie_amd.registry import lookup
    rot = {"base": 500.0, "dims": 24, "scaling": {"factor": 5.0, "low": 1.0, "high": 3.0, "original": 100}}
    part = lookup("position_encoding", "rotary")(PartSpec("rotary", {"head_dim": 40, "rot_dim": 24, "theta": 500.0, "wavelength_scaling": rot["scaling"]}), torch.float32, "cpu")
    got, dims = part.rotary_table()
    want = torch.tensor(plain.frequencies(rot), dtype=F64)
    unscaled = torch.tensor(plain.frequencies({"base": 500.0, "dims": 24}), dtype=F64)
    assert dims == 24 and torch.equal(got, want.float())
    ratio = (unscaled / want).tolist()
    assert sum(r == 1.0 for r in ratio) > 1 and sum(abs(r - 5.0) < 1e-9 for r in ratio) > 1 and sum(1.001 < r < 4.999 for r in ratio) > 1


# ---- the plain implementation's pieces, by hand ------------------------------------------------------------
def test_plain_convolution_weighs_the_last_inputs():
    u = torch.tensor([[1.0], [10.0], [100.0], [1000.0]], dtype=F64)
    got = plain.channel_conv(u, torch.tensor([[3.0, 2.0, 1.0]], dtype=F64))
    assert got.flatten().tolist() == [1.0, 12.0, 123.0, 1230.0]             # (zeros before the first; the last tap is the token's own)


def test_plain_window():
    mask = plain.window_mask(6, 3)
    assert mask[5].tolist() == [False, False, False, True, True, True] and mask[1].tolist() == [True, True] + [False] * 4
    assert plain.window_mask(4, None)[3].tolist() == [True] * 4 and plain.window_mask(4, 1).tolist() == torch.eye(4, dtype=torch.bool).tolist()


def test_the_plain_state_space_walk_is_the_sum_over_earlier_tokens():
    generator = torch.Generator().manual_seed(1)
    x, B, C = (torch.randn(7, size, generator=generator, dtype=F64) for size in (5, 3, 3))
    dt, A = torch.rand(7, generator=generator, dtype=F64), torch.tensor(-0.8, dtype=F64)
    got = plain.state_space_walk(x, B, C, dt, A, 0.25)
    for t in range(7):
        want = 0.25 * x[t]
        for s in range(t + 1):
            want = want + torch.exp(A * dt[s + 1:t + 1].sum()) * dt[s] * (C[t] @ B[s]) * x[s]
        assert torch.allclose(got[t], want)


def test_the_plain_delta_rule_replaces_what_a_key_holds():
    key, other = torch.tensor([1.0, 0.0], dtype=F64), torch.tensor([0.0, 1.0], dtype=F64)
    k = torch.stack([key, other, key])
    v = torch.tensor([[2.0], [5.0], [7.0]], dtype=F64)
    ones = torch.ones(3, dtype=F64)
    got = plain.delta_walk(torch.stack([key, key, key]), k, v, ones, ones)
    assert got.flatten().tolist() == [2.0, 2.0, 7.0]                        # the third token's value takes the first one's place
    half = plain.delta_walk(torch.stack([key, key, key]), k, v, 0.5 * ones, 0.5 * ones)
    assert half.flatten().tolist() == [1.0, 0.5, 0.25 + 0.5 * (7.0 - 0.25)]     # decayed first, then moved half the way


def test_the_plain_mixture_weighs_the_tables_experts_alike():
    w = {"table": torch.tensor([[0, 1], [1, 2]], dtype=F64)}
    for e, factor in enumerate((1.0, 2.0, 4.0)):
        w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"] = (torch.tensor([[value]], dtype=F64) for value in (1.0, factor, 1.0))
    h = torch.tensor([[3.0], [3.0]], dtype=F64)
    mlp = {"kind": "moe", "expert": {"ff": 1}, "router": {"experts": 3, "top": 2}}
    unit = 3.0 / (1.0 + math.exp(-3.0)) * 3.0
    got = plain.mixture(mlp, w, "", h, torch.tensor([0, 1]))
    assert torch.allclose(got.flatten(), torch.tensor([unit * 1.5, unit * 3.0], dtype=F64))


def test_plain_norms():
    x = torch.tensor([[1.0, 3.0]], dtype=F64)
    assert torch.allclose(plain.centred_norm(x, torch.tensor([2.0, 2.0], dtype=F64), 3.0), torch.tensor([[-1.0, 1.0]], dtype=F64))
    assert torch.allclose(plain.unit_length(torch.tensor([[3.0, 4.0]], dtype=F64)), torch.tensor([[0.6, 0.8]], dtype=F64), atol=1e-7)
