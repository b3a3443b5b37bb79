"""The Paluzen decoder on the CPU: config.json to the model as data, the tensors it expects, what is refused, and pieces
of the plain implementation against cases worked out by hand."""
import copy
import math
import re

import pytest
import torch

import plain_paluzen as plain
from paluzen_helpers import CONFIGS, CONFIG_U, CONFIG_V, CONFIG_W

F64 = torch.float64


def spec_of(raw):
    from tlie_amd.registry import config_from_dict
    return config_from_dict(raw).to_spec()


def test_the_configuration_becomes_the_model_as_data():
    spec = spec_of(CONFIG_U)
    assert (spec.architecture, spec.hidden_size, spec.vocab_size, spec.max_positions) == ("Paluzen", 72, 181, None)
    # layers 1 and 2 run three times in a row, every pass on a cache and state of its own, and begins with the product
    assert [run.layer for run in spec.runs] == [0, 1, 2, 1, 2, 1, 2, 3]
    assert [run.pass_input for run in spec.runs] == [None, "loop.in", None, "loop.in", None, "loop.in", None, None]
    assert all(run.cache_of == index for index, run in enumerate(spec.runs))
    assert all(layer.block == "pre_norm" and layer.sublayer_input.kind == "token_shift" and layer.sublayer_input_of == ("mixer",)
               for layer in spec.layers)
    first, second, third, fourth = spec.layers
    left, right = first.mixer["left"], first.mixer["right"]
    assert (first.mixer.kind, first.mixer["left_scale"], first.mixer["right_scale"]) == ("side_by_side", 1.2, -0.6)
    assert (left.kind, left["window"], left["head_temp"], left["head_gate"], left["value_dim"], left["scale"]) == ("attention", 7, True, True, 24, 0.3)
    assert (left["position"].kind, left["position"]["rot_dim"], left["position"]["theta"]) == ("rotary", 8, 90.0)
    assert (right.kind, right["num_heads"], right["head_dim"]) == ("token_shift_mixing", 3, 20)
    assert (first.feed_forward.kind, first.feed_forward["activation"], first.feed_forward["intermediate_size"]) == ("mlp", "relu_squared", 56)
    assert (second.mixer.kind, second.mixer["decay"], second.mixer["value_dim"]) == ("lightning_attention", (1.0, 0.9, 0.0), 40)
    mlp = second.feed_forward
    assert mlp.kind == "routed_mlp"
    assert [mlp[key] for key in ("experts", "top", "identity", "groups", "keep", "expert_size", "score", "renormalize", "weigh", "activation")] == \
        [5, 3, 3, 4, 2, 24, "softmax_grouped", True, "output", "relu_squared"]
    assert third.feed_forward is None and third.mixer["left"]["window"] == 37
    assert [fourth.feed_forward[key] for key in ("identity", "groups", "keep")] == [0, 1, 1]
    assert spec.head["tied"] and spec.head["tied_to"] == "embed" and spec.head["softcap"] == 14.0


def test_what_config_json_leaves_out_is_absent():
    spec = spec_of(CONFIG_V)
    assert [run.layer for run in spec.runs] == [0, 1, 2] and all(run.pass_input is None for run in spec.runs)
    assert spec.head.get("softcap") is None and not spec.shared_tensors
    assert spec.layers[1].mixer["left"]["window"] is None and spec.layers[1].mixer["left"]["position"].kind == "none"


def test_the_expected_tensors_carry_the_designs_names_and_shapes():
    from tlie_amd.models.builder import expected_tensors
    shapes = {tensor.name: tensor.shape for tensor in expected_tensors(spec_of(CONFIG_U)) if not tensor.optional}
    assert shapes["embed"] == (181, 72) and shapes["final.norm"] == (72,) and shapes["loop.in"] == (72, 144) and "head" not in shapes
    assert shapes["l0.shift"] == (72,) and shapes["l0.norm1"] == (72,) and shapes["l0.norm2"] == (72,)
    assert shapes["l0.mix.left.q"] == (64, 72) and shapes["l0.mix.left.k"] == (16, 72) and shapes["l0.mix.left.v"] == (24, 72)
    assert shapes["l0.mix.left.o"] == (72, 96) and shapes["l0.mix.left.temp"] == (4,) and shapes["l0.mix.left.g"] == (4, 72)
    assert shapes["l0.mix.right.mu.w"] == (72,) and shapes["l0.mix.right.w1"] == (-1, 72) and shapes["l0.mix.right.w2"] == (60, -1)
    assert shapes["l0.mix.right.u"] == (3, 20) and shapes["l0.mix.right.o"] == (72, 60) and shapes["l0.mix.right.r"] == (60, 72)
    assert shapes["l0.mlp.up"] == (56, 72) and shapes["l0.mlp.down"] == (72, 56) and "l0.mlp.act" not in shapes
    assert shapes["l1.mix.q"] == (72, 72) and shapes["l1.mix.v"] == (120, 72) and shapes["l1.mix.norm"] == (120,) and shapes["l1.mix.o"] == (72, 120)
    assert shapes["l1.mlp.router"] == (8, 72) and shapes["l1.mlp.correction"] == (8,)
    assert shapes["l1.mlp.e4.up"] == (24, 72) and "l1.mlp.e5.up" not in shapes and "l1.mlp.e0.gate" not in shapes
    assert "l2.norm2" not in shapes and "l2.mlp.up" not in shapes                       # a layer without a feed-forward
    assert any(re.fullmatch(pattern, "l2.norm2") for pattern in spec_of(CONFIG_U).ignored_tensors)      # (a file may still carry it)
    assert not any(re.fullmatch(pattern, "l1.norm2") for pattern in spec_of(CONFIG_U).ignored_tensors)
    assert "loop.in" not in {tensor.name for tensor in expected_tensors(spec_of(CONFIG_V))}


@pytest.mark.parametrize("change,message", [
    (lambda raw: raw["layers"][0].update(type="retention"), "not one of"),
    (lambda raw: raw["layers"][0]["mixer"]["left"].update(kv_heads=3), "multiple"),
    (lambda raw: raw["layers"][0]["mixer"]["left"]["rot"].update(dims=7), "even"),
    (lambda raw: raw["layers"][0]["mixer"]["left"]["mask"].update(size=0), "positive"),
    (lambda raw: raw["layers"][0]["mixer"].pop("right_scale"), "right_scale"),
    (lambda raw: raw["layers"][1]["mixer"].update(decay=[0.5]), "one number"),
    (lambda raw: raw["layers"][1]["mlp"]["router"].update(top=5), "cannot use"),
    (lambda raw: raw["layers"][1]["mlp"]["router"]["groups"].update(count=3), "groups"),
    (lambda raw: raw["layers"][1]["mlp"]["router"]["groups"].update(keep=5), "groups"),
    (lambda raw: raw["layers"][3]["mlp"].update(kind="gated"), "kind"),
    (lambda raw: raw.update(loop={"start": 2, "stop": 7, "times": 2}), "stretch"),
    (lambda raw: raw["norm"].pop("eps"), "eps"),
])
def test_configurations_that_are_refused(change, message):
    from tlie_amd import EngineError
    raw = copy.deepcopy(CONFIG_U)
    change(raw)
    with pytest.raises(EngineError, match=message):
        spec_of(raw)


def test_a_pass_input_that_is_no_shared_tensor_is_refused():
    import dataclasses
    from tlie_amd import EngineError
    spec = spec_of(CONFIG_W)
    with pytest.raises(EngineError, match="loop.in"):
        dataclasses.replace(spec, shared_tensors=()).validate()


def test_every_configuration_of_the_tests_is_read():
    for raw in CONFIGS.values():
        spec_of(raw)


# ---- the plain implementation's pieces, by hand ------------------------------------------------------------
def test_plain_blend_reads_the_token_before():
    h = torch.tensor([[2.0, 4.0], [6.0, 8.0], [0.0, 1.0]], dtype=F64)
    got = plain.blend(h, torch.tensor([0.0, 0.25], dtype=F64))
    assert got.tolist() == [[2.0, 3.0], [6.0, 7.0], [0.0, 1.0 + 7.0 * 0.25]]        # (zeros before the first)


def test_plain_window():
    mask = plain.window_mask(6, 3)
    assert mask[5].tolist() == [False, False, False, True, True, True] and mask[1].tolist() == [True, True] + [False] * 4
    assert plain.window_mask(4, None)[3].tolist() == [True] * 4 and plain.window_mask(4, 1).tolist() == torch.eye(4, dtype=torch.bool).tolist()


@pytest.mark.parametrize("bonus", [False, True])
def test_the_plain_walk_is_the_sum_over_earlier_tokens(bonus):
    generator = torch.Generator().manual_seed(1)
    q, k, v = (torch.randn(7, size, generator=generator, dtype=F64) for size in (3, 3, 5))
    decay = torch.rand(7, 3, generator=generator, dtype=F64)
    u = torch.randn(3, generator=generator, dtype=F64) if bonus else None
    got = plain.decayed_state_walk(q, k, v, decay, bonus=u)
    for t in range(7):
        want = torch.zeros(5, dtype=F64)
        for s in range(t + 1):
            if bonus and s == t:
                weight = u
            else:           # with a bonus the result is read before token t's own decay is applied
                weight = torch.prod(decay[s + 1:t if bonus else t + 1], dim=0) if s < t else torch.ones(3, dtype=F64)
            want += (q[t] * weight * k[s]).sum() * v[s]
        assert torch.allclose(got[t], want)


def test_the_plain_router_chooses_by_groups_and_weighs_without_the_correction():
    z = torch.log(torch.tensor([[0.30, 0.05, 0.20, 0.10, 0.25, 0.10]], dtype=F64))      # (its softmax is itself)
    correction = torch.tensor([-0.40, 0.00, -0.30, -0.25, -0.50, -0.50], dtype=F64)
    # choice scores: -.10 .05 | -.10 -.15 | -.25 -.40; all but one negative: a closed group counts as minus infinity, not 0
    scores, chosen, weights = plain.router_choice(z, correction, 3, {"count": 3, "keep": 2})
    assert chosen.tolist() == [[1, 0, 2]] or chosen.tolist() == [[1, 2, 0]]
    by_expert = dict(zip(chosen[0].tolist(), weights[0].tolist()))
    assert all(math.isclose(by_expert[e], s / 0.55, rel_tol=1e-12) for e, s in ((1, 0.05), (0, 0.30), (2, 0.20)))
    _, open_choice, _ = plain.router_choice(z, correction, 5, None)
    assert sorted(open_choice[0].tolist()) == [0, 1, 2, 3, 4]
    # two groups' experts are fewer than the third group's would have offered without the groups
    _, chosen, _ = plain.router_choice(z, torch.tensor([0.0, 0.0, 0.0, 0.0, 0.5, 0.5], dtype=F64), 2, {"count": 3, "keep": 1})
    assert sorted(chosen[0].tolist()) == [4, 5]
    margin = plain.router_margin(z, correction, 3, {"count": 3, "keep": 2})
    assert math.isclose(float(margin), 0.05, rel_tol=1e-9)                # the third choice -.10 against -.15; groups: -.10 against -.25


def test_the_plain_mixture_hands_identities_the_input():
    w = {"router": torch.zeros(3, 2, dtype=F64), "correction": torch.tensor([0.0, 1.0, 2.0], dtype=F64),
         "e0.up": torch.tensor([[1.0, 0.0]], dtype=F64), "e0.down": torch.tensor([[1.0], [1.0]], dtype=F64),
         "e1.up": torch.tensor([[0.0, -2.0]], dtype=F64), "e1.down": torch.tensor([[1.0], [0.0]], dtype=F64)}
    h = torch.tensor([[3.0, -1.0]], dtype=F64)
    mlp = {"kind": "moe", "expert": {"ff": 1}, "router": {"experts": 2, "top": 2, "identity": 1}}
    got = plain.mixture(mlp, w, "", h)                                    # expert 1 and the identity, half each
    assert torch.allclose(got, 0.5 * torch.tensor([[4.0, 0.0]], dtype=F64) + 0.5 * h)
    assert plain.relu_squared(torch.tensor([-2.0, 3.0], dtype=F64)).tolist() == [0.0, 9.0]


def test_the_plain_loop_begins_every_pass_with_the_embedding():
    assert plain.run_order(CONFIG_U) == [(0, False), (1, True), (2, False), (1, True), (2, False), (1, True), (2, False), (3, False)]
    assert plain.run_order(CONFIG_W) == [(0, True), (0, True), (1, False), (2, False)]
