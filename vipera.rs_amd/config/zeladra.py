"""Configuration of the Zeladra decoder, read from its own ``config.json``.

The file lists the layers one by one: ``layers[i]`` has ``type`` (``latent_attention``: latent attention with a gate per
head; ``mamba2``: a state-space recurrence; ``attention``: softmax attention in a sliding window that keeps a sequence's
first positions), ``mixer`` (its sizes and constants) and ``mlp`` (``{"kind": "dense", "ff"}`` or null).  Beside the list
stand ``vocab``, ``width``, ``norm.eps``, ``embedding.scale`` and ``streams`` (residual streams per token).  A
latent-attention layer with ``kv_from: j`` keeps no cache of its own and reads layer ``j``'s.  Rotations turn neighbouring
pairs.  Tensor names: ``embed``, ``l<i>.norm1 | norm2`` (``.b``: their biases), ``l<i>.mix.*``, ``l<i>.mlp.*``,
``l<i>.hc1.* | hc2.*``, ``final.norm``, ``head``.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional, Tuple

from ..errors import InvalidArgumentError, UnsupportedError
from .base import KeyReader, LayerSpec, ModelConfig, PartSpec, ScheduleEntry

MIXER_TYPES = ("latent_attention", "mamba2", "attention")
MLP_KINDS = ("dense",)


def _sub(data: Dict[str, Any], key: str, where: str) -> Dict[str, Any]:
    value = data.get(key)
    if not isinstance(value, dict):
        raise InvalidArgumentError(f"{where}: key \"{key}\" is {value!r}, expected an object")
    return value


def _optional(data: Dict[str, Any], key: str, where: str) -> Optional[Dict[str, Any]]:
    return _sub(data, key, where) if data.get(key) is not None else None


@dataclass
class ZeladraConfig(ModelConfig):
    vocab: int
    width: int
    eps: float
    embedding_scale: float
    streams: int
    layers: List[Dict[str, Any]] = field(default_factory=list)
    max_positions: int = 1 << 20       # nothing learned or tabled bounds the context; a file may give "max_positions"
    eos_token_ids: Tuple[int, ...] = ()

    architecture = "Zeladra"

    # --- reading ----------------------------------------------------------------------
    @classmethod
    def from_dict(cls, data: Dict[str, Any]) -> "ZeladraConfig":
        r = KeyReader(data)
        layers = data.get("layers")
        if not isinstance(layers, list) or not all(isinstance(layer, dict) for layer in layers):
            raise InvalidArgumentError("config.json: key \"layers\" must be a list of objects, one per layer")
        eos = data.get("eos_token_id")
        eos_ids = () if eos is None else (eos,) if isinstance(eos, int) else tuple(eos)
        embedding = _optional(data, "embedding", "config.json")
        config = cls(
            vocab=r.integer("vocab", minimum=1), width=r.integer("width", minimum=1),
            eps=KeyReader(_sub(data, "norm", "config.json"), "config.json: norm").number("eps"),
            embedding_scale=KeyReader(embedding, "config.json: embedding").number("scale", default=1.0) if embedding else 1.0,
            streams=r.integer("streams", default=1, minimum=1), layers=copy.deepcopy(layers),
            max_positions=r.integer("max_positions", default=1 << 20, minimum=1), eos_token_ids=eos_ids)
        config.validate()
        return config

    def validate(self) -> None:
        if not self.eps >= 0.0:
            raise InvalidArgumentError(f"config.json: norm: key \"eps\" is {self.eps!r}, expected a number at or above 0")
        for index, layer in enumerate(self.layers):
            where = f"config.json: layers[{index}]"
            kind = layer.get("type")
            if kind not in MIXER_TYPES:
                raise UnsupportedError(f"{where}: type {kind!r} is not implemented; known: {', '.join(MIXER_TYPES)}")
            mixer = _sub(layer, "mixer", where)
            check = {"latent_attention": self._check_latent, "mamba2": self._check_mamba2, "attention": self._check_attention}
            check[kind](index, mixer, where + ".mixer")
            mlp = layer.get("mlp")
            if mlp is not None:
                if not isinstance(mlp, dict) or mlp.get("kind") not in MLP_KINDS:
                    raise UnsupportedError(f"{where}: mlp {mlp!r} is not implemented; \"kind\" {' or '.join(MLP_KINDS)}, or null")
                KeyReader(mlp, where + ".mlp").integer("ff", minimum=1)

    @staticmethod
    def _check_rot(m: Dict[str, Any], dim: int, where: str) -> None:
        rot = _optional(m, "rot", where)
        if rot is None:
            return
        rr = KeyReader(rot, where + ".rot")
        dims = rr.integer("dims", minimum=0)
        if dims % 2 or dims > dim:
            raise InvalidArgumentError(f"{where}.rot: \"dims\" is {dims}; it must be even and at most {dim}")
        base = rr.number("base") if dims else 2.0
        if not base > 0:
            raise InvalidArgumentError(f"{where}.rot: \"base\" must be above 0")
        scaling = _optional(rot, "scaling", where + ".rot")
        if scaling is not None:
            sr = KeyReader(scaling, where + ".rot.scaling")
            if not all(sr.number(key) > 0 for key in ("factor", "original", "fast", "slow")) or base == 1.0:
                raise InvalidArgumentError(f"{where}.rot.scaling: {scaling!r}; \"factor\", \"original\", \"fast\" and \"slow\" "
                                           "must be above 0, and the base other than 1")

    def _check_latent(self, index: int, m: Dict[str, Any], where: str) -> None:
        r = KeyReader(m, where)
        for key in ("heads", "dim", "vdim", "q_rank", "kv_rank"):
            r.integer(key, minimum=1)
        r.number("scale")
        self._check_rot(m, r.integer("rot_dim", minimum=0), where)
        if r.has("kv_from"):
            source = r.integer("kv_from")
            owner = self.layers[source] if source < index else None
            if owner is None or owner.get("type") != "latent_attention" or owner["mixer"].get("kv_from") is not None:
                raise InvalidArgumentError(f"{where}: \"kv_from\" is {source}; it must name an earlier latent-attention layer "
                                           "that has a cache of its own")
            for key in ("kv_rank", "rot_dim", "rot"):
                if owner["mixer"].get(key) != m.get(key):
                    raise InvalidArgumentError(f"{where}: \"{key}\" differs from layer {source}'s, whose cache this layer reads")

    def _check_mamba2(self, index: int, m: Dict[str, Any], where: str) -> None:
        r = KeyReader(m, where)
        heads, vdim = r.integer("heads", minimum=1), r.integer("vdim", minimum=1)
        r.integer("state", minimum=1)
        r.integer("conv", minimum=1)
        groups, parts = r.integer("groups", minimum=1), r.integer("norm_groups", minimum=1)
        if heads % groups:
            raise InvalidArgumentError(f"{where}: \"heads\" {heads} is not a multiple of \"groups\" {groups}")
        if heads * vdim % parts:
            raise InvalidArgumentError(f"{where}: \"norm_groups\" {parts} does not divide the {heads * vdim} inner numbers")

    def _check_attention(self, index: int, m: Dict[str, Any], where: str) -> None:
        r = KeyReader(m, where)
        heads, kv_heads = r.integer("heads", minimum=1), r.integer("kv_heads", minimum=1)
        if heads % kv_heads:
            raise InvalidArgumentError(f"{where}: \"heads\" {heads} is not a multiple of \"kv_heads\" {kv_heads}")
        dim = r.integer("dim", minimum=1)
        r.integer("vdim", minimum=1)
        r.number("scale")
        mask = _optional(m, "mask", where)
        if mask is not None:
            mr = KeyReader(mask, where + ".mask")
            mr.integer("size", minimum=1)
            mr.integer("keep_first", default=0, minimum=0)
        self._check_rot(m, dim, where)

    def to_dict(self) -> Dict[str, Any]:
        data: Dict[str, Any] = {"architecture": self.architecture, "embedding": {"scale": self.embedding_scale},
                                "layers": copy.deepcopy(self.layers), "norm": {"eps": self.eps}, "streams": self.streams,
                                "vocab": self.vocab, "width": self.width}
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
        return PartSpec("layernorm", {"width": self.width, "eps": self.eps, "tensor": name})

    @staticmethod
    def _rotation(m: Dict[str, Any], head_dim: int) -> PartSpec:
        rot = m.get("rot") or {}
        dims = int(rot.get("dims") or 0)
        if not dims:
            return PartSpec("none", {})
        params = {"head_dim": head_dim, "rotary_dim": dims, "base": float(rot["base"]), "wide_table": True}
        if rot.get("scaling"):
            params["ramp"] = {key: float(rot["scaling"][key]) for key in ("factor", "original", "fast", "slow")}
        return PartSpec("rotary_neox", params)

    @staticmethod
    def _pairs(m: Dict[str, Any]) -> Dict[str, Any]:
        dims = int((m.get("rot") or {}).get("dims") or 0)
        return {"pairs": "interleaved", "rotary_dim": dims} if dims else {}

    def _latent(self, m: Dict[str, Any]) -> PartSpec:
        return PartSpec("latent_attention", {
            "hidden": self.width, "heads": int(m["heads"]), "dim": int(m["dim"]), "rot_dim": int(m["rot_dim"]),
            "vdim": int(m["vdim"]), "q_rank": int(m["q_rank"]), "kv_rank": int(m["kv_rank"]), "scale": float(m["scale"]),
            "eps": self.eps, "shares_cache": m.get("kv_from") is not None, "gate": "head_sigmoid", "name": "mix",
            **self._pairs(m)})

    def _mamba2(self, m: Dict[str, Any]) -> PartSpec:
        return PartSpec("state_space", {
            "hidden": self.width, "heads": int(m["heads"]), "vdim": int(m["vdim"]), "state": int(m["state"]),
            "groups": int(m["groups"]), "norm_groups": int(m["norm_groups"]), "conv": int(m["conv"]), "eps": self.eps,
            "name": "mix"})

    def _attention(self, m: Dict[str, Any]) -> PartSpec:
        mask = m.get("mask") or {}
        return PartSpec("attention", {
            "hidden": self.width, "heads": int(m["heads"]), "kv_heads": int(m["kv_heads"]), "head_dim": int(m["dim"]),
            "value_dim": int(m["vdim"]), "scale": float(m["scale"]), "window": int(mask.get("size") or 0),
            "keep_first": int(mask.get("keep_first") or 0), "tensors": {"q": "q", "k": "k", "v": "v", "o": "o"}, "name": "mix",
            **self._pairs(m)})

    def layer_specs(self) -> List[LayerSpec]:
        specs = []
        for index, layer in enumerate(self.layers):
            m, position = layer["mixer"], PartSpec("none", {})
            if layer["type"] == "latent_attention":
                mixer, position = self._latent(m), self._rotation(m, int(m["rot_dim"]))
            elif layer["type"] == "attention":
                mixer, position = self._attention(m), self._rotation(m, int(m["dim"]))
            else:
                mixer = self._mamba2(m)
            mlp = layer.get("mlp")
            ffn = PartSpec("none", {}) if mlp is None else PartSpec("gated_mlp", {
                "hidden": self.width, "intermediate": int(mlp["ff"]), "activation": "silu",
                "tensors": {"gate": "gate", "up": "up", "down": "down"}, "name": "mlp"})
            specs.append(LayerSpec("hyper", mixer, ffn, self._norm("norm1"), self._norm("norm2"), position, f"l{index}.",
                                   params={"streams": self.streams, "names": ("hc1", "hc2")}))
        return specs

    def schedule(self) -> List[ScheduleEntry]:
        return [ScheduleEntry(index, layer["mixer"].get("kv_from") if layer["type"] == "latent_attention" else None)
                for index, layer in enumerate(self.layers)]

    def embedding_spec(self) -> PartSpec:
        return PartSpec("embedding", {"vocab": self.vocab, "width": self.width, "name": "embed", "tensor": "embed",
                                      "scale": self.embedding_scale, "streams": self.streams})

    def final_norm_spec(self) -> PartSpec:
        return PartSpec("summed", {"norm": self._norm("final.norm")})

    def head_spec(self) -> PartSpec:
        return PartSpec("lm_head", {"vocab": self.vocab, "width": self.width, "name": "head", "tensor": "head",
                                    "tied_to": None})
