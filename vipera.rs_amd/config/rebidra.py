"""Configuration of the Rebidra decoder, read from its own ``config.json``.

The file lists the layers one by one: ``layers[i]`` has ``type`` (``attention``: softmax attention in a sliding window with
a sink, short convolutions on queries and keys, and values that are the convolved keys), ``mixer`` (its sizes and constants)
and ``mlp`` (``{"kind": "moe", "expert": {"ff"}, "router": {"experts", "top"}, "shared": {"ff"}}``, or null).  Beside the
list stand ``vocab``, ``width``, ``norm.eps``, ``embedding.scale``, ``logit_scale``, ``token_side.dim`` (columns per layer of
the per-token side table) and ``loop`` (``{"start", "stop", "times"}``: layers ``start`` to ``stop - 1`` run ``times`` times
in a row; ahead of every pass the stream and the embedding's output go through ``loop.in`` together).  Layer norms without a
bias stand in front of the sublayers.  Tensor names: ``embed``, ``loop.in``, ``side.embed``, ``l<i>.norm1 | norm2``,
``l<i>.mix.*``, ``l<i>.mlp.*``, ``l<i>.side.*``, ``final.norm``, ``head``.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional, Tuple

from ..errors import InvalidArgumentError, UnsupportedError
from .base import KeyReader, LayerSpec, ModelConfig, PartSpec, ScheduleEntry

MIXER_TYPES = ("attention",)
MLP_KINDS = ("moe",)


def _sub(data: Dict[str, Any], key: str, where: str) -> Dict[str, Any]:
    value = data.get(key)
    if not isinstance(value, dict):
        raise InvalidArgumentError(f"{where}: key \"{key}\" is {value!r}, expected an object")
    return value


def _optional(data: Dict[str, Any], key: str, where: str) -> Optional[Dict[str, Any]]:
    return _sub(data, key, where) if data.get(key) is not None else None


@dataclass
class RebidraConfig(ModelConfig):
    vocab: int
    width: int
    eps: float
    embedding_scale: float
    logit_scale: float
    side_dim: int                      # 0: the model has no per-token side table
    loop: Optional[Tuple[int, int, int]]       # (start, stop, times), or None: every layer runs once
    layers: List[Dict[str, Any]] = field(default_factory=list)
    max_positions: int = 1 << 20       # nothing learned or tabled bounds the context; a file may give "max_positions"
    eos_token_ids: Tuple[int, ...] = ()

    architecture = "Rebidra"

    # --- reading ----------------------------------------------------------------------
    @classmethod
    def from_dict(cls, data: Dict[str, Any]) -> "RebidraConfig":
        r = KeyReader(data)
        layers = data.get("layers")
        if not isinstance(layers, list) or not all(isinstance(layer, dict) for layer in layers):
            raise InvalidArgumentError("config.json: key \"layers\" must be a list of objects, one per layer")
        eos = data.get("eos_token_id")
        eos_ids = () if eos is None else (eos,) if isinstance(eos, int) else tuple(eos)
        embedding = _optional(data, "embedding", "config.json")
        side = _optional(data, "token_side", "config.json")
        loop = _optional(data, "loop", "config.json")
        if loop is not None:
            lr = KeyReader(loop, "config.json: loop")
            loop = (lr.integer("start"), lr.integer("stop", minimum=1), lr.integer("times", minimum=1))
        config = cls(
            vocab=r.integer("vocab", minimum=1), width=r.integer("width", minimum=1),
            eps=KeyReader(_sub(data, "norm", "config.json"), "config.json: norm").number("eps"),
            embedding_scale=KeyReader(embedding, "config.json: embedding").number("scale", default=1.0) if embedding else 1.0,
            logit_scale=r.number("logit_scale", default=1.0),
            side_dim=KeyReader(side, "config.json: token_side").integer("dim", minimum=1) if side else 0, loop=loop,
            layers=copy.deepcopy(layers), max_positions=r.integer("max_positions", default=1 << 20, minimum=1),
            eos_token_ids=eos_ids)
        config.validate()
        return config

    def validate(self) -> None:
        if not self.eps >= 0.0:
            raise InvalidArgumentError(f"config.json: norm: key \"eps\" is {self.eps!r}, expected a number at or above 0")
        if self.loop is not None and not 0 <= self.loop[0] < self.loop[1] <= len(self.layers):
            raise InvalidArgumentError(f"config.json: loop: layers {self.loop[0]} to {self.loop[1]} (exclusive) are not a range "
                                       f"of the {len(self.layers)} layers")
        for index, layer in enumerate(self.layers):
            where = f"config.json: layers[{index}]"
            kind = layer.get("type")
            if kind not in MIXER_TYPES:
                raise UnsupportedError(f"{where}: type {kind!r} is not implemented; known: {', '.join(MIXER_TYPES)}")
            self._check_attention(_sub(layer, "mixer", where), where + ".mixer")
            self._check_mlp(layer.get("mlp"), where)

    @staticmethod
    def _check_attention(m: Dict[str, Any], where: str) -> None:
        r = KeyReader(m, where)
        heads, kv_heads = r.integer("heads", minimum=1), r.integer("kv_heads", minimum=1)
        if heads % kv_heads:
            raise InvalidArgumentError(f"{where}: \"heads\" {heads} is not a multiple of \"kv_heads\" {kv_heads}")
        dim, vdim = r.integer("dim", minimum=1), r.integer("vdim", minimum=1)
        if dim != vdim:
            raise InvalidArgumentError(f"{where}: \"vdim\" is {vdim}; the values are the keys, which are {dim} wide")
        r.integer("conv", default=1, minimum=1)        # absent: no convolution
        r.number("scale")
        mask = _optional(m, "mask", where)
        if mask is not None:
            KeyReader(mask, where + ".mask").integer("size", minimum=1)
        rot = _optional(m, "rot", where)
        if rot is None:
            return
        rr = KeyReader(rot, where + ".rot")
        dims = rr.integer("dims", minimum=0)
        if dims % 2 or dims > dim:
            raise InvalidArgumentError(f"{where}.rot: \"dims\" is {dims}; it must be even and at most \"dim\" {dim}")
        base = rr.number("base") if dims else 2.0
        if not base > 0:
            raise InvalidArgumentError(f"{where}.rot: \"base\" must be above 0")
        scaling = _optional(rot, "scaling", where + ".rot")
        if scaling is not None:
            sr = KeyReader(scaling, where + ".rot.scaling")
            if not all(sr.number(key) > 0 for key in ("factor", "original", "fast", "slow")) or base == 1.0:
                raise InvalidArgumentError(f"{where}.rot.scaling: {scaling!r}; \"factor\", \"original\", \"fast\" and \"slow\" "
                                           "must be above 0, and the base other than 1")

    @staticmethod
    def _check_mlp(mlp: Any, where: str) -> None:
        if mlp is None:
            return
        if not isinstance(mlp, dict) or mlp.get("kind") not in MLP_KINDS:
            raise UnsupportedError(f"{where}: mlp {mlp!r} is not implemented; \"kind\" {' or '.join(MLP_KINDS)}, or null")
        KeyReader(_sub(mlp, "expert", where + ".mlp"), where + ".mlp.expert").integer("ff", minimum=1)
        router = KeyReader(_sub(mlp, "router", where + ".mlp"), where + ".mlp.router")
        experts, top = router.integer("experts", minimum=1), router.integer("top", minimum=1)
        if top > experts:
            raise InvalidArgumentError(f"{where}.mlp.router: \"top\" {top} is above \"experts\" {experts}")
        shared = _optional(mlp, "shared", where + ".mlp")
        if shared is not None:
            KeyReader(shared, where + ".mlp.shared").integer("ff", minimum=1)

    def to_dict(self) -> Dict[str, Any]:
        data: Dict[str, Any] = {"architecture": self.architecture, "embedding": {"scale": self.embedding_scale},
                                "layers": copy.deepcopy(self.layers), "logit_scale": self.logit_scale,
                                "norm": {"eps": self.eps}, "vocab": self.vocab, "width": self.width}
        if self.loop is not None:
            data["loop"] = dict(zip(("start", "stop", "times"), self.loop))
        if self.side_dim:
            data["token_side"] = {"dim": self.side_dim}
        if self.max_positions != 1 << 20:
            data["max_positions"] = self.max_positions
        if self.eos_token_ids:
            data["eos_token_id"] = list(self.eos_token_ids)
        return data

    @property
    def context_limit(self) -> int:
        return int(self.max_positions)

    # --- for callers that ask a configuration for its sizes by the common names ---------------------
    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def hidden_size(self) -> int:
        return self.width

    # --- the description the generic decoder consumes ---------------------------------------
    def _norm(self, name: str) -> PartSpec:
        return PartSpec("layernorm", {"width": self.width, "eps": self.eps, "tensor": name, "bias": False})

    def _attention(self, m: Dict[str, Any]) -> PartSpec:
        return PartSpec("attention", {
            "hidden": self.width, "heads": int(m["heads"]), "kv_heads": int(m["kv_heads"]), "head_dim": int(m["dim"]),
            "scale": float(m["scale"]), "window": int((m.get("mask") or {}).get("size") or 0), "values": "keys",
            "conv": int(m.get("conv") or 0), "qkv_bias": True, "qk_norm": "head", "eps": self.eps, "sink": True,
            "gate": "head_sigmoid", "name": "mix",
            "tensors": {"q": "q", "k": "k", "o": "o", "g": "g", "q_bias": "q.b", "k_bias": "k.b", "q_norm": "q.norm",
                        "k_norm": "k.norm", "q_conv": "q.conv", "k_conv": "k.conv"}})

    @staticmethod
    def _rotation(m: Dict[str, Any]) -> PartSpec:
        rot = m.get("rot") or {}
        dims = int(rot.get("dims") or 0)
        if not dims:
            return PartSpec("none", {})
        params = {"head_dim": int(m["dim"]), "rotary_dim": dims, "base": float(rot["base"]), "wide_table": True}
        if rot.get("scaling"):
            params["ramp"] = {key: float(rot["scaling"][key]) for key in ("factor", "original", "fast", "slow")}
        return PartSpec("rotary_neox", params)

    def _ffn(self, mlp: Optional[Dict[str, Any]]) -> PartSpec:
        if mlp is None:
            return PartSpec("none", {})
        router, shared = mlp["router"], mlp.get("shared")
        return PartSpec("moe", {"hidden": self.width, "intermediate": int(mlp["expert"]["ff"]),
                                "experts": int(router["experts"]), "top": int(router["top"]), "form": "plain",
                                "activation": "relu2", "scores": "chosen", "router_bias": "router.b",
                                "shared": int(shared["ff"]) if shared is not None else None,
                                "shared_gate": "sigmoid" if shared is not None else None, "name": "mlp"})

    def layer_specs(self) -> List[LayerSpec]:
        specs = []
        for index, layer in enumerate(self.layers):
            extras = {}
            if self.side_dim:
                extras["after"] = PartSpec("token_side", {"hidden": self.width, "dim": self.side_dim, "index": index,
                                                          "eps": self.eps, "activation": "gelu_tanh", "name": "side"})
            specs.append(LayerSpec("prenorm", self._attention(layer["mixer"]), self._ffn(layer.get("mlp")),
                                   self._norm("norm1"), self._norm("norm2"), self._rotation(layer["mixer"]), f"l{index}.",
                                   extras))
        return specs

    def schedule(self) -> List[ScheduleEntry]:
        if self.loop is None:
            return [ScheduleEntry(index) for index in range(len(self.layers))]
        start, stop, times = self.loop
        one_pass = [ScheduleEntry(index, rejoins=index == start) for index in range(start, stop)]
        return ([ScheduleEntry(index) for index in range(start)] + one_pass * times
                + [ScheduleEntry(index) for index in range(stop, len(self.layers))])

    def rejoin_spec(self) -> Optional[PartSpec]:
        if self.loop is None:
            return None
        return PartSpec("concat_linear", {"width": self.width, "tensor": "loop.in"})

    def embedding_spec(self) -> PartSpec:
        params = {"vocab": self.vocab, "width": self.width, "name": "embed", "tensor": "embed",
                  "scale": self.embedding_scale}
        if self.side_dim:
            params["side"] = {"tensor": "side.embed", "width": self.side_dim * len(self.layers)}
        return PartSpec("embedding", params)

    def final_norm_spec(self) -> PartSpec:
        return self._norm("final.norm")

    def head_spec(self) -> PartSpec:
        return PartSpec("lm_head", {"vocab": self.vocab, "width": self.width, "name": "head", "tensor": "head",
                                    "tied_to": None, "scale": self.logit_scale})
