"""The configuration of the Paluzen decoder, read from its own config.json keys.

    architecture    "Paluzen"
    vocab, width    sizes of the vocabulary and of the residual stream
    norm.eps        of every norm
    logit_softcap   c: the logits leave as c tanh(logits / c) (absent: as they are)
    loop            start, stop, times: layers start .. stop - 1 run `times` times in a row with the same weights, each pass
                    on a cache and state of its own, and each pass begins with the product of [residual; embedding output]
                    (absent: every layer runs once)
    layers          one entry a layer: `type` ("parallel", "lightning"), `mixer` (that mixer's sizes and constants) and `mlp`
                    (null: no feed-forward; kind "dense" with `ff`; kind "moe" with `expert` (ff) and `router` (experts, top,
                    and optionally groups (count, keep) and identity))

    parallel    left (heads, kv_heads, dim, vdim, scale, and optionally rot (base, dims) and mask (size: a sliding window)),
                right (heads, dim), left_scale, right_scale
    lightning   heads, dim, vdim, decay (one a head)

A layer is pre-norm with RMS norms; what a mixer reads is its norm's result blended with that of the token before.  Every
size and every constant that can differ between two models of the design is read from here (the rank of the decays'
low-rank product is the stored tensors' own); what the design fixes (the arrangement, rotation of halves, a head tied to
the embedding's table, how the router chooses and weighs, the tensors' names) is written down in `to_spec`.  The design sets
no bound on positions.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass
from typing import Any, Mapping

from ..errors import invalid_config
from .fadutar import _number
from .spec import LayerSpec, ModelSpec, PartSpec, Run, TensorSpec

LAYER_TYPES = ("parallel", "lightning")


@dataclass(frozen=True)
class PaluzenConfig:
    raw: Mapping[str, Any]          # config.json as read (validated)
    architecture: str = "Paluzen"

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any]) -> "PaluzenConfig":
        config = cls(raw=copy.deepcopy(dict(raw)), architecture=str(raw.get("architecture", "Paluzen")))
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
        if raw.get("logit_softcap") is not None:
            _number("the model", raw, "logit_softcap", float)
        layers = raw.get("layers")
        if not isinstance(layers, list) or not layers:
            raise invalid_config("'layers' must be a list with at least one layer")
        loop = raw.get("loop")
        if loop is not None:
            start, stop = _number("loop", loop, "start", positive=False), _number("loop", loop, "stop")
            _number("loop", loop, "times")
            if not 0 <= start < stop <= len(layers):
                raise invalid_config(f"loop: layers {start} .. {stop - 1} are not a stretch of the model's {len(layers)}")
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

    def _check_parallel(self, mixer, where):
        left, right = mixer.get("left"), mixer.get("right")
        side = f"{where}'s left"
        heads, kv_heads, dim = _number(side, left, "heads"), _number(side, left, "kv_heads"), _number(side, left, "dim")
        _number(side, left, "vdim"), _number(side, left, "scale", float)
        if heads % kv_heads != 0:
            raise invalid_config(f"{where}: heads {heads} is not a multiple of kv_heads {kv_heads}")
        if left.get("mask") is not None:
            _number(f"{side}'s mask", left["mask"], "size")
        rot = left.get("rot")
        if rot is not None:
            _number(f"{side}'s rot", rot, "base", float)
            dims = _number(f"{side}'s rot", rot, "dims")
            if dims > dim or dims % 2 != 0:
                raise invalid_config(f"{where}: rot.dims must be even and at most dim (the dims past it pass unrotated)")
        _number(f"{where}'s right", right, "heads"), _number(f"{where}'s right", right, "dim")
        _number(where, mixer, "left_scale", float, positive=False), _number(where, mixer, "right_scale", float, positive=False)

    def _check_lightning(self, mixer, where):
        heads = _number(where, mixer, "heads")
        _number(where, mixer, "dim"), _number(where, mixer, "vdim")
        decay = mixer.get("decay")
        if not isinstance(decay, list) or len(decay) != heads or not all(isinstance(value, (int, float)) and 0 <= value <= 1 for value in decay):
            raise invalid_config(f"{where}: 'decay' must list one number between 0 and 1 a head")

    def _check_mlp(self, mlp, where):
        if not isinstance(mlp, Mapping) or mlp.get("kind") not in ("dense", "moe"):
            raise invalid_config(f"{where}: an mlp must be null or of kind 'dense' or 'moe'")
        if mlp["kind"] == "dense":
            _number(where, mlp, "ff")
            return
        _number(f"{where}'s expert", mlp.get("expert"), "ff")
        router = mlp.get("router")
        experts, top = _number(f"{where}'s router", router, "experts"), _number(f"{where}'s router", router, "top")
        identity = _number(f"{where}'s router", router, "identity", positive=False) if router.get("identity") is not None else 0
        count, keep = self._groups(router, where)
        outputs = experts + identity
        if identity < 0 or outputs % count != 0 or keep > count:
            raise invalid_config(f"{where}: {count} equal groups, of which {keep} stay, do not divide {outputs} experts and identities")
        if top > keep * (outputs // count):
            raise invalid_config(f"{where}: a token cannot use {top} of the {keep * (outputs // count)} it may choose from")

    @staticmethod
    def _groups(router, where):
        groups = router.get("groups")
        if groups is None:
            return 1, 1
        return _number(f"{where}'s router groups", groups, "count"), _number(f"{where}'s router groups", groups, "keep")

    # ---- the model as data ----------------------------------------------------------------------------
    def to_spec(self) -> ModelSpec:
        raw = self.raw
        width, vocab, eps = int(raw["width"]), int(raw["vocab"]), float(raw["norm"]["eps"])
        norm = PartSpec("rms_norm", {"size": width, "eps": eps, "tensor": ""})      # (the tensor is named by the place alone)
        layers = []
        for index, layer in enumerate(raw["layers"]):
            mlp = layer.get("mlp")
            layers.append(LayerSpec(
                prefix=f"l{index}.", block="pre_norm", mixer=getattr(self, "_spec_" + layer["type"])(layer["mixer"], width, eps),
                feed_forward=self._spec_mlp(mlp, width) if mlp is not None else None,
                mixer_norm=norm, feed_forward_norm=norm if mlp is not None else None,
                mixer_norm_place="norm1", mixer_place="mix.", feed_forward_norm_place="norm2", feed_forward_place="mlp.",
                sublayer_input=PartSpec("token_shift", {"size": width, "tensor": ""}), sublayer_input_of=("mixer",),
                mixer_input_place="shift"))
        count = len(layers)
        loop = raw.get("loop")
        order, shared = [(index, None) for index in range(count)], ()
        if loop is not None:
            start, stop, times = int(loop["start"]), int(loop["stop"]), int(loop["times"])
            one_pass = [(index, "loop.in" if index == start else None) for index in range(start, stop)]
            order = order[:start] + one_pass * times + order[stop:]
            shared = (TensorSpec("loop.in", (width, 2 * width)),)
        runs = tuple(Run(layer=layer, cache_of=index, pass_input=enters) for index, (layer, enters) in enumerate(order))
        head = {"vocab_size": vocab, "hidden_size": width, "tied": True, "tied_to": "embed"}
        if raw.get("logit_softcap") is not None:
            head["softcap"] = float(raw["logit_softcap"])
        spec = ModelSpec(
            architecture=self.architecture, hidden_size=width, vocab_size=vocab, max_positions=None,
            embedding=PartSpec("token_embedding", {"vocab_size": vocab, "hidden_size": width}),
            layers=tuple(layers), runs=runs, final_norm=norm, head=PartSpec("lm_head", head),
            embedding_name="embed", final_norm_prefix="final.norm", head_name="head", shared_tensors=shared,
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
            position = PartSpec("rotary", {"head_dim": int(left["dim"]), "rot_dim": int(rot["dims"]), "theta": float(rot["base"])})
        attention = PartSpec("attention", {
            "hidden_size": width, "num_heads": int(left["heads"]), "num_kv_heads": int(left["kv_heads"]),
            "head_dim": int(left["dim"]), "value_dim": int(left["vdim"]), "scale": float(left["scale"]), "bias": False,
            "window": int(mask["size"]) if mask is not None else None, "position": position, "head_temp": True, "head_gate": True,
            "names": {"q": "q", "k": "k", "v": "v", "o": "o", "temp": "temp", "head_gate": "g"}})
        mixing = PartSpec("token_shift_mixing", {
            "hidden_size": width, "num_heads": int(right["heads"]), "head_dim": int(right["dim"]), "norm_eps": eps})
        return PartSpec("side_by_side", {"left": attention, "right": mixing, "left_scale": float(mixer["left_scale"]),
                                         "right_scale": float(mixer["right_scale"]), "left_place": "left.", "right_place": "right."})

    @staticmethod
    def _spec_lightning(mixer, width, eps) -> PartSpec:
        return PartSpec("lightning_attention", {
            "hidden_size": width, "num_heads": int(mixer["heads"]), "head_dim": int(mixer["dim"]), "value_dim": int(mixer["vdim"]),
            "decay": tuple(float(value) for value in mixer["decay"]), "norm_eps": eps,
            "names": {"q": "q", "k": "k", "v": "v", "gate": "g", "o": "o", "norm": "norm"}})

    def _spec_mlp(self, mlp, width) -> PartSpec:
        names = {"up": "up", "down": "down"}
        if mlp["kind"] == "dense":
            return PartSpec("mlp", {"hidden_size": width, "intermediate_size": int(mlp["ff"]), "activation": "relu_squared", "names": names})
        router = mlp["router"]
        count, keep = self._groups(router, "the router")
        return PartSpec("routed_mlp", {
            "hidden_size": width, "experts": int(router["experts"]), "top": int(router["top"]), "identity": int(router.get("identity") or 0),
            "groups": count, "keep": keep, "expert_size": int(mlp["expert"]["ff"]), "score": "softmax_grouped", "renormalize": True,
            "weigh": "output", "activation": "relu_squared",
            "names": {"router": "router", "correction": "correction", "expert": "e{}.", **names}})
