"""Rebidra: a decoder whose layers are listed one by one in its configuration, a range of which runs several times in a row
(softmax attention in a sliding window with a sink, whose queries and keys pass short convolutions and whose values are the
convolved keys; a mixture of ungated experts with a gated shared one; a per-token side table that every layer reads).

Everything specific to the architecture is in :class:`~vipera_rs_amd.config.RebidraConfig`, which describes the
layers as data; the model itself is the generic decoder.
"""
from __future__ import annotations

from ..config.rebidra import RebidraConfig
from ..config.registry import register_architecture
from .decoder import DecoderModel


def build_rebidra(config: RebidraConfig, runtime) -> DecoderModel:
    return DecoderModel(config, runtime)


register_architecture("Rebidra", RebidraConfig, build_rebidra)
