"""The configuration of the Barilix decoder, read from its own config.json keys.

    architecture       "Barilix"
    vocab, width       sizes of the vocabulary and of the residual stream
    norm.eps           of every norm
    embedding.scale    what the embedding's rows are multiplied by
    layers             one entry a layer: `type` ("parallel", "delta"), `mixer` (that mixer's sizes and constants) and `mlp`
                       (null: no feed-forward; kind "dense" with `ff`; kind "moe" with `expert` (ff), `router` (experts, top)
                       and optionally `shared` (ff))

    parallel    left (heads, kv_heads, dim, vdim, conv, scale, and optionally mask (size: a sliding window) and rot (base, dims,
                and optionally scaling (factor, low, high, original))),
                right (heads, vdim, state, groups, norm_groups, conv)
    delta       heads, kv_heads, dim, vdim, conv

The sublayers read the residual itself; what they give passes a layer norm (a weight, no bias) before it joins.  Every size
and every constant that can differ between two models of the design is read from here; what the design fixes (the
arrangement, rotation of halves, the experts that a table names, the tensors' names) is written down in `to_spec`.  The
design sets no bound on positions.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass
from typing import Any, Mapping

from ..errors import invalid_config
from .fadutar import _number
from .spec import LayerSpec, ModelSpec, PartSpec, Run

LAYER_TYPES = ("parallel", "delta")


@dataclass(frozen=True)
class BarilixConfig:
    raw: Mapping[str, Any]          # config.json as read (validated)
    architecture: str = "Barilix"

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any]) -> "BarilixConfig":
        config = cls(raw=copy.deepcopy(dict(raw)), architecture=str(raw.get("architecture", "Barilix")))
        config.validate()
        return config

    def to_dict(self) -> dict:
        return copy.deepcopy(dict(self.raw))

    # ---- checks -----------------------------------------------------------------------------------
    def validate(self) -> None:
        raw = self.raw
        _number("the model", raw, "vocab")
        _number("the model", raw, "width")
        _number("norm", raw.get("norm"), "eps", float)
        _number("embedding", raw.get("embedding"), "scale", float, positive=False)
        layers = raw.get("layers")
        if not isinstance(layers, list) or not layers:
            raise invalid_config("'layers' must be a list with at least one layer")
        for index, layer in enumerate(layers):
            where = f"layer {index}"
            if not isinstance(layer, Mapping) or layer.get("type") not in LAYER_TYPES:
                kind = layer.get("type") if isinstance(layer, Mapping) else layer
                raise invalid_config(f"{where}: type {kind!r} is not one of {', '.join(LAYER_TYPES)}")
            mixer = layer.get("mixer")
            if not isinstance(mixer, Mapping):
                raise invalid_config(f"{where} lacks 'mixer'")
            getattr(self, "_check_" + layer["type"])(mixer, f"{where}'s mixer")
            if layer.get("mlp") is not None:
                self._check_mlp(layer["mlp"], f"{where}'s mlp")

    @staticmethod
    def _check_heads(where, part):
        heads, kv_heads = _number(where, part, "heads"), _number(where, part, "kv_heads")
        _number(where, part, "dim"), _number(where, part, "vdim"), _number(where, part, "conv")
        if heads % kv_heads != 0:
            raise invalid_config(f"{where}: heads {heads} is not a multiple of kv_heads {kv_heads}")

    def _check_parallel(self, mixer, where):
        left, right = mixer.get("left"), mixer.get("right")
        side = f"{where}'s left"
        self._check_heads(side, left)
        _number(side, left, "scale", float)
        if left.get("mask") is not None:
            _number(f"{side}'s mask", left["mask"], "size")
        rot = left.get("rot")
        if rot is not None:
            _number(f"{side}'s rot", rot, "base", float)
            dims = _number(f"{side}'s rot", rot, "dims")
            if dims > int(left["dim"]) or dims % 2 != 0:
                raise invalid_config(f"{where}: rot.dims must be even and at most dim (the dims past it pass unrotated)")
            scaling = rot.get("scaling")
            if scaling is not None:
                low, high = _number(f"{side}'s scaling", scaling, "low", float), _number(f"{side}'s scaling", scaling, "high", float)
                _number(f"{side}'s scaling", scaling, "factor", float), _number(f"{side}'s scaling", scaling, "original", float)
                if not low < high:
                    raise invalid_config(f"{where}: rot.scaling.low must be below high")
        side = f"{where}'s right"
        heads, vdim, groups = _number(side, right, "heads"), _number(side, right, "vdim"), _number(side, right, "groups")
        _number(side, right, "state"), _number(side, right, "conv")
        if heads % groups != 0 or (heads * vdim) % _number(side, right, "norm_groups") != 0:
            raise invalid_config(f"{side}: groups must divide heads, and norm_groups heads * vdim")

    def _check_delta(self, mixer, where):
        self._check_heads(where, mixer)

    def _check_mlp(self, mlp, where):
        if not isinstance(mlp, Mapping) or mlp.get("kind") not in ("dense", "moe"):
            raise invalid_config(f"{where}: an mlp must be null or of kind 'dense' or 'moe'")
        if mlp["kind"] == "dense":
            _number(where, mlp, "ff")
            return
        _number(f"{where}'s expert", mlp.get("expert"), "ff")
        router = mlp.get("router")
        experts, top = _number(f"{where}'s router", router, "experts"), _number(f"{where}'s router", router, "top")
        if top > experts:
            raise invalid_config(f"{where}: a token cannot use {top} of {experts} experts")
        if mlp.get("shared") is not None:
            _number(f"{where}'s shared expert", mlp["shared"], "ff")

    # ---- the model as data ----------------------------------------------------------------------------
    def to_spec(self) -> ModelSpec:
        raw = self.raw
        width, vocab, eps = int(raw["width"]), int(raw["vocab"]), float(raw["norm"]["eps"])
        norm = PartSpec("layer_norm", {"size": width, "eps": eps, "bias": False, "tensor": ""})      # (the tensor is named by the place alone)
        layers, runs = [], []
        for index, layer in enumerate(raw["layers"]):
            mlp = layer.get("mlp")
            layers.append(LayerSpec(
                prefix=f"l{index}.", block="post_norm", mixer=getattr(self, "_spec_" + layer["type"])(layer["mixer"], width, eps),
                feed_forward=self._spec_mlp(mlp, width, vocab) if mlp is not None else None,
                mixer_norm=norm, feed_forward_norm=norm if mlp is not None else None,
                mixer_norm_place="norm1", mixer_place="mix.", feed_forward_norm_place="norm2", feed_forward_place="mlp."))
            runs.append(Run(layer=index, cache_of=index))
        spec = ModelSpec(
            architecture=self.architecture, hidden_size=width, vocab_size=vocab, max_positions=None,
            embedding=PartSpec("token_embedding", {"vocab_size": vocab, "hidden_size": width, "scale": float(raw["embedding"]["scale"])}),
            layers=tuple(layers), runs=tuple(runs), final_norm=norm,
            head=PartSpec("lm_head", {"vocab_size": vocab, "hidden_size": width, "tied": False}),
            embedding_name="embed", final_norm_prefix="final.norm", head_name="head",
            # a layer without a feed-forward reads no second norm: a file that carries one all the same is taken
            ignored_tensors=tuple(rf"l{index}\.norm2" for index, layer in enumerate(raw["layers"]) if layer.get("mlp") is None))
        spec.validate()
        return spec

    @staticmethod
    def _spec_parallel(mixer, width, eps) -> PartSpec:
        left, right = mixer["left"], mixer["right"]
        rot, mask = left.get("rot"), left.get("mask")
        position = PartSpec("none")
        if rot is not None:
            params = {"head_dim": int(left["dim"]), "rot_dim": int(rot["dims"]), "theta": float(rot["base"])}
            if rot.get("scaling") is not None:
                params["wavelength_scaling"] = {key: float(rot["scaling"][key]) for key in ("factor", "low", "high", "original")}
            position = PartSpec("rotary", params)
        names = {role: role for role in ("q", "k", "v", "o")}
        names.update({f"{role}_bias": f"{role}.b" for role in ("q", "k", "v", "o")})
        names.update({f"{role}_conv": f"{role}.conv" for role in ("q", "k", "v")})
        names.update({"q_norm": "q.norm", "k_norm": "k.norm"})
        attention = PartSpec("attention", {
            "hidden_size": width, "num_heads": int(left["heads"]), "num_kv_heads": int(left["kv_heads"]),
            "head_dim": int(left["dim"]), "value_dim": int(left["vdim"]), "scale": float(left["scale"]), "bias": True,
            "window": int(mask["size"]) if mask is not None else None, "position": position, "conv": int(left["conv"]),
            "qk_norm": "head", "norm_eps": eps, "names": names})
        state_space = PartSpec("state_space", {
            "hidden_size": width, "num_heads": int(right["heads"]), "head_dim": int(right["vdim"]), "state_size": int(right["state"]),
            "groups": int(right["groups"]), "norm_groups": int(right["norm_groups"]), "taps": int(right["conv"]), "norm_eps": eps,
            "names": {"in": "in", "conv": "conv", "conv_bias": "conv.b", "dt_bias": "dt_bias", "rate": "A_log", "skip": "D", "norm": "norm", "o": "o"}})
        return PartSpec("side_by_side", {"left": attention, "right": state_space, "result_norm_eps": eps, "scale": 0.5, "hidden_size": width,
                                         "left_place": "left.", "right_place": "right.", "result_norm": "out"})

    @staticmethod
    def _spec_delta(mixer, width, eps) -> PartSpec:
        names = {role: role for role in ("q", "k", "v", "o", "norm")}
        names.update({f"{role}_conv": f"{role}.conv" for role in ("q", "k", "v")})
        names.update({"beta": "b", "decay": "a", "decay_bias": "dt_bias", "rate": "A_log", "gate": "g"})
        return PartSpec("gated_delta", {
            "hidden_size": width, "num_heads": int(mixer["heads"]), "num_kv_heads": int(mixer["kv_heads"]), "head_dim": int(mixer["dim"]),
            "value_dim": int(mixer["vdim"]), "taps": int(mixer["conv"]), "norm_eps": eps, "names": names})

    @staticmethod
    def _spec_mlp(mlp, width, vocab) -> PartSpec:
        names = {"gate": "gate", "up": "up", "down": "down"}
        if mlp["kind"] == "dense":
            return PartSpec("gated_mlp", {"hidden_size": width, "intermediate_size": int(mlp["ff"]), "activation": "silu", "names": names})
        router, shared = mlp["router"], mlp.get("shared")
        return PartSpec("routed_mlp", {
            "hidden_size": width, "experts": int(router["experts"]), "top": int(router["top"]), "expert_size": int(mlp["expert"]["ff"]),
            "shared_size": int(shared["ff"]) if shared is not None else 0, "score": "table", "vocab_size": vocab, "weigh": "output",
            "names": {"table": "table", "expert": "e{}.", "shared": "shared.", **names}})
