"""Mixers whose heads keep a matrix state that decays by one number a token and head, behind short causal convolutions.

A request's state is, in one row of floats, the heads' S (dim x vdim each, zero when the request is admitted) and after it
the convolutions' last inputs.  The projections are one product; the convolutions' sums, the unit norms, the gates of
the recurrence, S, the scan's sums and the heads' norms are float whatever the activation type (`ops.short_conv`,
`ops.gated_scan`, `ops.head_combine`):

    state_space    with N = state_size, groups of heads that share B and C, inner = num_heads * head_dim:
                       [z | x | B | C | dt] = W_in h;   x, B, C pass a convolution with a bias, then silu
                       dt = softplus(dt + bias_h);   S <- exp(-exp(rate_h) dt) S + dt B x^T;   y = S^T C + skip_h x
                       y * silu(z) RMS-normed in norm_groups equal parts, times a weight, output product
    gated_delta    q and k (num_kv_heads * head_dim), v (num_heads * value_dim), each through a convolution and silu; q and
                   k of unit length a head, q also times head_dim^(-1/2); head h uses q and k of head h // (heads / kv heads)
                       beta = sigmoid(W_b h),   g = exp(-exp(rate_h) softplus(W_a h + bias_h))
                       S <- g S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q
                   each head's o RMS-normed with a weight the heads share, times silu(gate), output product
"""
from __future__ import annotations

from functools import partial

import torch

from .. import ops
from ..config.spec import PartSpec, TensorSpec
from ..errors import invalid_config
from ..registry import register
from ..weights.arena import keep_in
from .base import Binding, Mixer, StateNeed
from .linear import Linear


def _padded(rows: torch.Tensor) -> torch.Tensor:
    """Rows of zeros appended up to a multiple of 8 (a product's rows then start at multiples of 16 bytes)."""
    more = -rows.shape[0] % 8
    return rows.contiguous() if more == 0 else torch.cat([rows, rows.new_zeros(more, rows.shape[1])], dim=0)


def _value_width(value_dim: int) -> int:
    """The values' planes on their way into the scan: a head's columns, or equal pieces of them where the convolution's kernel
    takes no head so wide."""
    pieces = next(count for count in range(1, value_dim + 1) if value_dim % count == 0 and value_dim // count <= ops.SHORT_CONV_MAX_HEAD)
    return value_dim // pieces


def _check_taps(kind, taps):
    if not 1 <= taps <= ops.SHORT_CONV_MAX_TAPS:
        raise invalid_config(f"{kind}: a short convolution has 1 to {ops.SHORT_CONV_MAX_TAPS} taps")


@register("mixer", "state_space")
class StateSpace(Mixer):
    """spec: hidden_size, num_heads, head_dim, state_size, groups, norm_groups, taps, norm_eps, names (the tensors' names
    after the prefix, by role).
    Tensors: in [2 * inner + 2 * groups * state_size + num_heads, hidden]; conv [inner + 2 * groups * state_size, taps] with
    conv_bias; dt_bias, rate, skip [num_heads]; norm [inner]; o [hidden, inner]."""
    graph_safe = True
    NAMES = {"in": "in_proj.weight", "conv": "conv1d.weight", "conv_bias": "conv1d.bias", "dt_bias": "dt_bias", "rate": "A_log", "skip": "D",
             "norm": "norm.weight", "o": "out_proj.weight"}

    def __init__(self, spec: PartSpec, dtype, device):
        super().__init__(spec, dtype, device)
        self.hidden = int(spec["hidden_size"])
        self.heads, self.dv, self.d = int(spec["num_heads"]), int(spec["head_dim"]), int(spec["state_size"])
        self.groups, self.parts, self.taps = int(spec["groups"]), int(spec["norm_groups"]), int(spec["taps"])
        self.eps = float(spec["norm_eps"])
        self.inner = self.heads * self.dv
        if min(self.heads, self.dv, self.d, self.groups, self.parts) <= 0 or self.heads % self.groups != 0 or self.inner % self.parts != 0:
            raise invalid_config("state_space: heads are a positive multiple of groups, and norm_groups divide heads * head_dim")
        if self.d > ops.GATED_SCAN_MAX_DIM:
            raise invalid_config(f"state_space: state_size {self.d} is beyond what the scan keeps in registers ({ops.GATED_SCAN_MAX_DIM})")
        _check_taps("state_space", self.taps)
        self.channels = self.inner + 2 * self.groups * self.d
        # (planes as wide as those of B and C, where they go into the values evenly, leave the convolution no lane without work)
        self.value_width = self.d if self.inner % self.d == 0 else _value_width(self.dv)
        self.scan_floats = ops.gated_scan_state_floats(self.heads, self.d, self.dv)
        self.names = {**self.NAMES, **dict(spec.get("names") or {})}
        self.first = self.o = self.conv = self.conv_bias = self.dt_bias = self.rate = self.skip = self.norm = None

    @classmethod
    def tensor_specs(cls, spec, prefix):
        names = {**cls.NAMES, **dict(spec.get("names") or {})}
        hidden, heads, dv, groups, d = (int(spec[key]) for key in ("hidden_size", "num_heads", "head_dim", "groups", "state_size"))
        inner, channels = heads * dv, heads * dv + 2 * groups * d
        return [TensorSpec(prefix + names["in"], (inner + channels + heads, hidden)),
                TensorSpec(prefix + names["conv"], (channels, int(spec["taps"])), init="taps"),
                TensorSpec(prefix + names["conv_bias"], (channels,), init="offset"),
                TensorSpec(prefix + names["dt_bias"], (heads,), init="step_bias"), TensorSpec(prefix + names["rate"], (heads,), init="log_rate"),
                TensorSpec(prefix + names["skip"], (heads,), init="norm"), TensorSpec(prefix + names["norm"], (inner,), init="norm"),
                TensorSpec(prefix + names["o"], (hidden, inner))]

    def load(self, weights, prefix):
        keep = partial(keep_in, weights)
        get = lambda role: weights[prefix + self.names[role]]        # noqa: E731
        self.first = Linear(_padded(get("in")), None, self.dtype, keep=keep)
        self.conv = keep(get("conv").to(self.first.weight.dtype).contiguous())
        self.conv_bias = keep(get("conv_bias").to(self.first.weight.dtype).contiguous())
        # (what enters the recurrence is float)
        self.dt_bias, self.rate, self.skip = (keep(get(role).float().contiguous()) for role in ("dt_bias", "rate", "skip"))
        self.norm = keep(get("norm").contiguous())
        self.o = Linear(get("o"), None, self.dtype, keep=keep)

    def state_need(self):
        """The heads' S, then the convolution's last taps - 1 inputs."""
        return StateNeed((self.scan_floats + ops.short_conv_state_floats(self.channels, self.taps),), torch.float32)

    def forward(self, x, ctx, binding: Binding, into=None):
        fused = ops.as_product(self.first(x))
        b_first = self.inner
        c_first = b_first + self.groups * self.d
        segments = [ops.ConvSegment(self.inner, self.value_width, target="heads"),
                    ops.ConvSegment(2 * self.groups * self.d, self.d, target="heads", out_col=b_first)]
        mixed = ops.short_conv(fused, self.inner, self.conv, self.conv_bias, binding.state[:, self.scan_floats:], ctx, segments, self.channels,
                               torch.float32, silu=True)
        scanned = ops.gated_scan(mixed, c_first, b_first, 0, fused, self.inner + self.channels, self.rate, self.dt_bias, binding.state, ctx,
                                 self.heads, self.groups, self.d, self.dv, skip=self.skip, value_width=self.value_width)
        normed = ops.head_combine(scanned, self.parts, self.inner // self.parts, self.eps, self.dtype, weight=self.norm, gate=fused, gate_col=0,
                                  gate_kind="silu", gate_first=True)
        return self.o(normed)


@register("mixer", "gated_delta")
class GatedDelta(Mixer):
    """spec: hidden_size, num_heads, num_kv_heads, head_dim, value_dim, taps, norm_eps, names (the tensors' names after the
    prefix, by role).
    Tensors: q and k [num_kv_heads * head_dim, hidden] and v [num_heads * value_dim, hidden], each with a convolution
    ({q,k,v}_conv [rows, taps]); beta and decay [num_heads, hidden]; decay_bias, rate [num_heads]; gate
    [num_heads * value_dim, hidden]; norm [value_dim] (the heads share it); o [hidden, num_heads * value_dim]."""
    graph_safe = True
    UNIT_EPS = 1e-6                # inside the root of a query's or key's length
    NAMES = {"q": "q_proj.weight", "k": "k_proj.weight", "v": "v_proj.weight", "q_conv": "q_conv1d.weight", "k_conv": "k_conv1d.weight",
             "v_conv": "v_conv1d.weight", "beta": "b_proj.weight", "decay": "a_proj.weight", "decay_bias": "dt_bias", "rate": "A_log",
             "gate": "g_proj.weight", "norm": "o_norm.weight", "o": "o_proj.weight"}

    def __init__(self, spec: PartSpec, dtype, device):
        super().__init__(spec, dtype, device)
        self.hidden = int(spec["hidden_size"])
        self.heads, self.groups = int(spec["num_heads"]), int(spec["num_kv_heads"])
        self.d, self.dv, self.taps = int(spec["head_dim"]), int(spec["value_dim"]), int(spec["taps"])
        self.eps = float(spec["norm_eps"])
        if min(self.heads, self.groups, self.d, self.dv) <= 0 or self.heads % self.groups != 0:
            raise invalid_config("gated_delta: num_heads must be a positive multiple of num_kv_heads")
        if self.d > ops.GATED_SCAN_MAX_DIM:
            raise invalid_config(f"gated_delta: head_dim {self.d} is beyond what the scan keeps in registers ({ops.GATED_SCAN_MAX_DIM})")
        _check_taps("gated_delta", self.taps)
        self.keys, self.values = self.groups * self.d, self.heads * self.dv
        self.channels = 2 * self.keys + self.values
        self.value_width = _value_width(self.dv)
        self.scan_floats = ops.gated_scan_state_floats(self.heads, self.d, self.dv)
        self.names = {**self.NAMES, **dict(spec.get("names") or {})}
        self.first = self.o = self.conv = self.decay_bias = self.rate = self.norm = None

    @classmethod
    def tensor_specs(cls, spec, prefix):
        names = {**cls.NAMES, **dict(spec.get("names") or {})}
        hidden, heads, groups, d, dv, taps = (int(spec[key]) for key in ("hidden_size", "num_heads", "num_kv_heads", "head_dim", "value_dim", "taps"))
        rows = {"q": groups * d, "k": groups * d, "v": heads * dv, "beta": heads, "decay": heads, "gate": heads * dv}
        specs = [TensorSpec(prefix + names[role], (count, hidden)) for role, count in rows.items()]
        specs += [TensorSpec(prefix + names[role + "_conv"], (rows[role], taps), init="taps") for role in ("q", "k", "v")]
        specs += [TensorSpec(prefix + names["decay_bias"], (heads,), init="step_bias"), TensorSpec(prefix + names["rate"], (heads,), init="log_rate"),
                  TensorSpec(prefix + names["norm"], (dv,), init="norm"), TensorSpec(prefix + names["o"], (hidden, heads * dv))]
        return specs

    def load(self, weights, prefix):
        keep = partial(keep_in, weights)
        get = lambda role: weights[prefix + self.names[role]]        # noqa: E731
        # one product: q, k and v (the convolutions' inputs), the gate, and the two gates of the recurrence
        self.first = Linear(_padded(torch.cat([get(role) for role in ("q", "k", "v", "gate", "decay", "beta")], dim=0)), None, self.dtype, keep=keep)
        self.conv = keep(torch.cat([get(role + "_conv") for role in ("q", "k", "v")], dim=0).to(self.first.weight.dtype).contiguous())
        self.decay_bias, self.rate = (keep(get(role).float().contiguous()) for role in ("decay_bias", "rate"))
        self.norm = keep(get("norm").repeat(self.heads).contiguous())         # (one entry a head and dim, as the combine kernel reads it)
        self.o = Linear(get("o"), None, self.dtype, keep=keep)

    def state_need(self):
        """The heads' S, then the convolutions' last taps - 1 inputs."""
        return StateNeed((self.scan_floats + ops.short_conv_state_floats(self.channels, self.taps),), torch.float32)

    def forward(self, x, ctx, binding: Binding, into=None):
        fused = ops.as_product(self.first(x))
        segments = [ops.ConvSegment(self.keys, self.d, "length", None, self.UNIT_EPS, float(self.d) ** -0.5, target="heads"),
                    ops.ConvSegment(self.keys, self.d, "length", None, self.UNIT_EPS, target="heads", out_col=self.keys),
                    ops.ConvSegment(self.values, self.value_width, target="heads", out_col=2 * self.keys)]
        mixed = ops.short_conv(fused, 0, self.conv, None, binding.state[:, self.scan_floats:], ctx, segments, self.channels, torch.float32, silu=True)
        gate_col = self.channels
        a_col = gate_col + self.values
        scanned = ops.gated_scan(mixed, 0, self.keys, 2 * self.keys, fused, a_col, self.rate, self.decay_bias, binding.state, ctx,
                                 self.heads, self.groups, self.d, self.dv, b_col=a_col + self.heads, value_width=self.value_width)
        normed = ops.head_combine(scanned, self.heads, self.dv, self.eps, self.dtype, weight=self.norm, gate=fused, gate_col=gate_col,
                                  gate_kind="silu")
        return self.o(normed)
