"""Zeladra: a decoder whose layers are listed one by one in its configuration (latent attention with a gate per head, one
layer reading another's cache; a state-space recurrence with one decay per head and token; attention in a sliding window
that keeps a sequence's first positions), each sublayer behind a layer norm and between several residual streams.

Everything specific to the architecture is in :class:`~vipera_rs_amd.config.ZeladraConfig`, which describes the
layers as data; the model itself is the generic decoder.
"""
from __future__ import annotations

from ..config.registry import register_architecture
from ..config.zeladra import ZeladraConfig
from .decoder import DecoderModel


def build_zeladra(config: ZeladraConfig, runtime) -> DecoderModel:
    return DecoderModel(config, runtime)


register_architecture("Zeladra", ZeladraConfig, build_zeladra)
