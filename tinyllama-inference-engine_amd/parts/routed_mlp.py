"""A routed feed-forward: a router scores the experts for every token, the token uses the `top` best, and an
expert that every token uses may run beside them.

    z = W_router x (float sums),  s = sigmoid(z)
    the `top` experts with the largest s are the token's; each is fed with s_e * x:
    out = sum over them of down_e(silu(gate_e(s_e x)) * up_e(s_e x))  +  shared(x)
(the scores are not renormalized, and weigh the expert's input, not its result).

Other designs of the same shape, as options:
    score "softmax_of_chosen"   the `top` largest logits z (+ a bias) are chosen, and their weights are the softmax over
                                the chosen logits only
    weigh "output"              out = sum of w_e * expert_e(x): the weight multiplies what the expert gives
    activation "clamped_swish"  g = min(gate, limit), u = clamp(up, -limit, limit), g * sigmoid(alpha g) * (u + 1), with a
                                limit for the experts and one for the shared expert
    score "softmax_grouped"     s = softmax(z) over all outputs; the choice goes by s + a correction [outputs], among the
                                experts of the `keep` of `groups` groups of neighbours whose best such number is largest;
                                the weights are the chosen s divided by their sum
    identity                    so many outputs of the router after the experts stand for the identity: their "result" is x
                                itself, times the weight
    activation "relu_squared"   experts without a gate, down_e(max(up_e(x), 0)^2)
    score "table"               no router: a table of integers [vocab, top] names each token id's experts (the entries of a
                                row differ), each of weight 1 / top
    shared_gate                 the shared expert's result is multiplied by sigmoid(w_sg . x), one number a token

All experts' gate and up matrices are one matrix, their rows side by side expert by expert (g0 u0 g1 u1 ...), the
shared expert's last, and all down matrices are one matrix along the inner index: the feed-forward is then two
products around a gate kernel that multiplies an expert's columns by the token's score for it, which is zero for an
expert that the token does not use (silu(0) * 0 adds nothing to the second product, exactly).  Since the products
are linear, s (W x) stands for W (s x); a weight on an expert's result multiplies the columns of the second product's
input in the result's place; and the shared expert's gate is one more row of the router's matrix, which stands outside
the choice.  An expert without a gate has its up rows alone in the first matrix.  With a table, a shared expert whose size
is a multiple of the experts' counts as that many experts more that every token uses with weight 1 (a sum over its inner
columns, cut).  In a step of many tokens the
products of experts without gates, or named by a table, run over the pairs of an expert and a token that uses it (`ops.route_plan`), where that pays.  The
identities' weights together multiply the row x, which whoever adds the feed-forward's result into the residual adds beside it (`ops.ScaledSum`).
"""
from __future__ import annotations

from functools import partial

import torch

from .. import ops
from ..config.spec import PartSpec, TensorSpec
from ..errors import invalid_config
from ..registry import register
from ..weights.arena import keep_in
from .base import FeedForward
from .linear import Linear


@register("feed_forward", "routed_mlp")
class RoutedMLP(FeedForward):
    """spec: hidden_size, experts, top, expert_size, shared_size (0: no shared expert), score ("sigmoid",
    "softmax_of_chosen", "table" (with vocab_size), or "softmax_grouped" with groups, keep and identity), renormalize (the last score's weights are,
    the others' are not), weigh ("input" or "output"), router_bias (False), activation ("silu", "clamped_swish" with alpha,
    limit, shared_limit, or "relu_squared"), shared_gate (False), names (router, router_bias, correction, expert: a pattern
    with {} for the expert's number, shared, shared_gate, table, gate, up, down).
    Tensors: table int32 [vocab, top], or router [experts + identity, hidden] (and its bias [experts], or its correction [experts + identity]); per expert
    and for the shared one gate (if the activation has one), up [size, hidden], down [hidden, size]; the shared expert's
    gate [1, hidden]."""
    graph_safe = True
    NAMES = {"router": "router.weight", "router_bias": "router.bias", "correction": "router.correction", "expert": "experts.{}.", "shared": "shared_expert.",
             "shared_gate": "shared_expert_gate.weight", "table": "table", "gate": "gate_proj.weight", "up": "up_proj.weight", "down": "down_proj.weight"}

    def __init__(self, spec: PartSpec, dtype, device):
        super().__init__(spec, dtype, device)
        self.hidden = int(spec["hidden_size"])
        self.experts, self.top = int(spec["experts"]), int(spec["top"])
        self.expert_size, self.shared_size = int(spec["expert_size"]), int(spec.get("shared_size", 0))
        if min(self.experts, self.top, self.expert_size) <= 0 or self.top > self.experts + int(spec.get("identity", 0)) or self.shared_size < 0:
            raise invalid_config("routed_mlp: experts, top (at most all outputs) and expert_size must be positive")
        self.score, self.weigh = spec.get("score", "sigmoid"), spec.get("weigh", "input")
        self.activation = spec.get("activation", "silu")
        self.alpha, self.limit = float(spec.get("alpha", 1.0)), float(spec.get("limit", 0.0))
        self.shared_limit = float(spec.get("shared_limit", self.limit))
        self.router_bias, self.shared_gate = bool(spec.get("router_bias", False)), bool(spec.get("shared_gate", False))
        self.grouped = self.score == "softmax_grouped"
        self.by_table = self.score == "table"
        self.identity = int(spec.get("identity", 0))
        self.groups, self.keep_groups = int(spec.get("groups", 1)), int(spec.get("keep", 1))
        if self.by_table and (self.weigh != "output" or self.router_bias or self.shared_gate or self.activation != "silu" or int(spec["vocab_size"]) <= 0):
            raise invalid_config("routed_mlp: a table of experts goes with SiLU gates, weights on the results, and no router's options")
        if ((not self.grouped and not self.by_table and self.score not in ops.ROUTER_SCORES) or self.weigh not in ("input", "output")
                or bool(spec.get("renormalize", False)) != self.grouped):
            raise invalid_config("routed_mlp: scores are sigmoids, the softmax over the chosen logits (both not renormalized) or the "
                                 "softmax over all of them with a choice among groups (renormalized), or a table's, and weigh the expert's input "
                                 "or its output")
        if self.identity < 0 or (not self.grouped and (self.identity, self.groups, self.keep_groups) != (0, 1, 1)):
            raise invalid_config("routed_mlp: identities and groups go with the softmax over all logits")
        if self.grouped:
            outputs = self.experts + self.identity
            if self.groups <= 0 or outputs % self.groups != 0 or not 0 < self.keep_groups <= self.groups:
                raise invalid_config(f"routed_mlp: {self.groups} equal groups, of which {self.keep_groups} stay, do not divide {outputs} outputs")
            if self.top > self.keep_groups * (outputs // self.groups):
                raise invalid_config(f"routed_mlp: a token cannot use {self.top} of the outputs of {self.keep_groups} groups")
            if self.activation != "relu_squared" or self.shared_size > 0 or spec.get("router_bias", False):
                raise invalid_config("routed_mlp: a choice among groups goes with experts without gates, no shared expert and no router bias")
        if self.activation == "relu_squared" and (self.weigh != "output" or self.shared_size > 0):
            raise invalid_config("routed_mlp: experts without gates take weights on their results, and have no shared one beside them")
        if (self.activation not in ops.GATES and self.activation != "relu_squared") or (self.weigh == "input" and self.activation != "silu"):
            raise invalid_config("routed_mlp: a score that weighs the expert's input goes with the SiLU gate only")
        if self.activation == "clamped_swish" and not (self.limit > 0.0 and self.shared_limit > 0.0):
            raise invalid_config("routed_mlp: the clamped gate needs positive limits")
        if self.shared_gate and (self.shared_size == 0 or self.weigh != "output"):
            raise invalid_config("routed_mlp: a gate of the shared expert needs a shared expert, and scores that weigh results")
        if self.score == "softmax_of_chosen" and self.top > 64:
            raise invalid_config("routed_mlp: the softmax over the chosen logits takes at most 64 of them")
        self.names = {**self.NAMES, **dict(spec.get("names") or {})}
        # a shared expert as so many experts more that every token uses
        self.always = self.shared_size // self.expert_size if self.by_table and self.shared_size % self.expert_size == 0 else 0
        self.router = self.router_b = self.correction = self.gate_up = self.down = self.table = None

    @classmethod
    def _prefixes(cls, spec, prefix, names):
        places = [prefix + names["expert"].format(e) for e in range(int(spec["experts"]))]
        sizes = [int(spec["expert_size"])] * len(places)
        if int(spec.get("shared_size", 0)) > 0:
            places.append(prefix + names["shared"])
            sizes.append(int(spec["shared_size"]))
        return list(zip(places, sizes))

    @classmethod
    def tensor_specs(cls, spec, prefix):
        names = {**cls.NAMES, **dict(spec.get("names") or {})}
        hidden = int(spec["hidden_size"])
        outputs, gated = int(spec["experts"]) + int(spec.get("identity", 0)), spec.get("activation", "silu") != "relu_squared"
        if spec.get("score", "sigmoid") == "table":
            specs = [TensorSpec(prefix + names["table"], (int(spec["vocab_size"]), int(spec["top"])), init="choice", choices=int(spec["experts"]))]
        else:
            specs = [TensorSpec(prefix + names["router"], (outputs, hidden))]
        if spec.get("score", "sigmoid") == "softmax_grouped":
            specs.append(TensorSpec(prefix + names["correction"], (outputs,), init="offset"))
        if spec.get("router_bias", False):
            specs.append(TensorSpec(prefix + names["router_bias"], (int(spec["experts"]),), init="spread"))
        if spec.get("shared_gate", False):
            specs.append(TensorSpec(prefix + names["shared_gate"], (1, hidden)))
        for place, size in cls._prefixes(spec, prefix, names):
            if gated:
                specs.append(TensorSpec(place + names["gate"], (size, hidden)))
            specs += [TensorSpec(place + names["up"], (size, hidden)), TensorSpec(place + names["down"], (hidden, size))]
        return specs

    def load(self, weights, prefix):
        names, keep = self.names, partial(keep_in, weights)
        if self.by_table:
            table = weights[prefix + names["table"]]
            if table.dtype != torch.int32 or table.numel() == 0 or int(table.min()) < 0 or int(table.max()) >= self.experts:
                raise invalid_config(f"routed_mlp: '{prefix}{names['table']}' must hold integers from 0 to {self.experts - 1}")
            self.table = keep(table.contiguous())
        else:
            self._load_router(weights, prefix, keep)
        rows, columns = [], []
        for place, size in self._prefixes(self.spec, prefix, names):
            up = weights[place + names["up"]]
            if self.activation == "relu_squared":
                rows.append(up)
            else:
                rows.append(torch.stack([weights[place + names["gate"]], up], dim=1).reshape(2 * size, self.hidden))
            columns.append(weights[place + names["down"]])
        self.gate_up = Linear(torch.cat(rows, dim=0).contiguous(), None, self.dtype, keep=keep)
        self.down = Linear(torch.cat(columns, dim=1).contiguous(), None, self.dtype, keep=keep)

    def _load_router(self, weights, prefix, keep):
        names = self.names
        router = weights[prefix + names["router"]]
        bias = weights[prefix + names["router_bias"]].to(router.dtype) if self.router_bias else None
        if self.shared_gate:
            # the gate's row stands after the experts' rows, outside the choice (its bias: none)
            router = torch.cat([router, weights[prefix + names["shared_gate"]].to(router.dtype).reshape(1, self.hidden)], dim=0)
            if bias is not None:
                bias = torch.cat([bias, torch.zeros(1, dtype=bias.dtype, device=bias.device)])
        self.router = keep(router.contiguous())
        self.router_b = keep(bias.contiguous()) if bias is not None else None
        if self.grouped:                                   # (it enters the router's choice, which is float)
            self.correction = keep(weights[prefix + names["correction"]].float().contiguous())

    def forward(self, x, ctx, into=None):
        if self.activation == "relu_squared":
            return self._forward_ungated(x)
        if self.by_table:
            return self._forward_table(x, ctx)
        scale = ops.few_outputs(x, self.router, self.router_b, top=self.top, score=self.score, extra=1 if self.shared_gate else 0)
        hidden = ops.routed_gate(ops.as_product(self.gate_up(x)), scale, self.expert_size, self.dtype, weigh=self.weigh,
                                 shared_scaled=self.shared_gate, gate=self.activation, alpha=self.alpha, limit=self.limit,
                                 shared_limit=self.shared_limit)
        return self.down(hidden)

    def _forward_table(self, x, ctx):
        scale = ops.table_scale(ctx.tokens, self.table, self.experts, self.always)
        experts, most = self.experts + self.always, self.top + self.always
        whole = self.always > 0 or self.shared_size == 0          # (no columns beside the experts')
        if whole and x.dtype == torch.bfloat16 and ops.routed_products_pay(x.shape[0], self.gate_up.weight, self.down.weight, experts, most):
            plan = ops.route_plan(scale, experts, most)
            return ops.routed_sum(ops.routed_down(ops.routed_gated(x, self.gate_up.weight, plan), self.down.weight, plan), plan)
        hidden = ops.routed_gate(ops.as_product(self.gate_up(x)), scale, self.expert_size, self.dtype, weigh="output")
        return self.down(hidden)

    def _forward_ungated(self, x):
        if self.grouped:
            scale = ops.grouped_router(x, self.router, self.correction, self.top, self.identity, self.groups, self.keep_groups)
        else:
            scale = ops.few_outputs(x, self.router, self.router_b, top=self.top, score=self.score)
        most = min(self.top, self.experts)
        if ops.routed_products_pay(x.shape[0], self.gate_up.weight, self.down.weight, self.experts, most) and x.dtype == torch.bfloat16:
            plan = ops.route_plan(scale, self.experts, most)
            out = ops.routed_sum(ops.routed_down(ops.routed_relu_squared(x, self.gate_up.weight, plan), self.down.weight, plan), plan)
        else:
            out = self.down(self.gate_up.relu_squared(x, scale, self.expert_size))
        if self.identity == 0:
            return out
        # the identities' weights together are the scale matrix's last column: x times it joins beside the experts' sum
        return ops.ScaledSum(ops.as_product(out), 1.0, ops.as_product(x), 1.0, row_scale=scale)
