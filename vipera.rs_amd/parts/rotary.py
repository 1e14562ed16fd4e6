"""Rotary position encoding, NeoX layout: pairs ``(i, i + rotary_dim / 2)`` of each head.

Reference: crates/vipera-backend-cpu/src/model.rs:4192-4251.  ``inv_i = 1 / base^(2i / head_dim)``
in 32-bit; the angle is ``float(pos) * inv_i`` in 32-bit; ``x[i] = lo*c - hi*s``,
``x[i + half] = lo*s + hi*c``.  The table of ``inv_i`` is computed once on the host with 32-bit
operations (``wide_table``: in 64-bit, rounded once) and kept on the device; the angle and its sine and cosine are computed in the kernel, or for
a step of many tokens once per step into a table that all layers with these frequencies read.
"""
from __future__ import annotations

import math
from typing import List

import numpy as np
import torch

from ..config.base import PartSpec
from ..errors import InvalidArgumentError
from ..ops import kernels
from .base import PositionEncoding, register_position


ANGLE_TABLE_MIN_TOKENS = 128   # steps with at least this many tokens share one table of sines and cosines


def neox_inverse_frequencies(rotary_dim: int, base: float) -> np.ndarray:
    index = np.arange(rotary_dim // 2, dtype=np.float32)
    exponent = (np.float32(2.0) * index) / np.float32(rotary_dim)
    return (np.float32(1.0) / np.power(np.float32(base), exponent, dtype=np.float32)).astype(np.float32)


def stretch_long_waves(table: np.ndarray, factor: float, low: float, high: float, original: float) -> np.ndarray:
    """Frequencies scaled by wavelength, as Llama 3.1 stretches its context: with ``l = 2 pi / f``, a frequency stays
    where ``l < original / high``, is divided by ``factor`` where ``l > original / low``, and in between is blended,
    ``(1 - s) f / factor + s f`` with ``s = (original / l - low) / (high - low)``."""
    f = table.astype(np.float64)
    wave = 2.0 * np.pi / f
    share = (original / wave - low) / (high - low)
    out = np.where(wave < original / high, f, np.where(wave > original / low, f / factor, (1.0 - share) * f / factor + share * f))
    return out.astype(np.float32)


def blend_by_index(table: np.ndarray, rotary_dim: int, base: float, factor: float, original: float, fast: float,
                   slow: float) -> np.ndarray:
    """Frequencies blended by a ramp over the pair's index (YaRN; Peng et al., "YaRN: Efficient Context Window Extension of
    Large Language Models"): pairs that make more than ``fast`` turns within ``original`` positions stay, those that make
    fewer than ``slow`` are divided by ``factor``, and the ramp between the two indices is linear."""
    def index_of(turns: float) -> float:
        return rotary_dim * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    low = max(math.floor(index_of(fast)), 0)
    high = min(math.ceil(index_of(slow)), rotary_dim - 1)
    ramp = np.clip((np.arange(rotary_dim // 2) - low) / max(high - low, 0.001), 0.0, 1.0)
    f = table.astype(np.float64)
    return f / factor * ramp + f * (1.0 - ramp)


def pairs_apart(weight: torch.Tensor, heads: int, dim: int, first: int, rotary_dim: int) -> torch.Tensor:
    """The rows of a projection whose heads (``dim`` rows each) rotate neighbouring pairs ``(2i, 2i + 1)`` of the
    ``rotary_dim`` numbers from ``first`` on, reordered so that the pairs lie ``rotary_dim / 2`` apart, as the kernels rotate
    them.  Done to queries and keys alike it changes no score."""
    if rotary_dim < 4:
        return weight
    order = torch.arange(dim, device=weight.device)
    order[first:first + rotary_dim] = first + torch.arange(rotary_dim, device=weight.device).view(-1, 2).t().reshape(-1)
    return weight.view(heads, dim, -1)[:, order].reshape(weight.shape).contiguous()


class RotaryNeox(PositionEncoding):
    def __init__(self, spec: PartSpec, prefix: str, runtime):
        super().__init__(spec, prefix, runtime)
        self.head_dim = int(spec.params["head_dim"])
        self.rotary_dim = int(spec.params.get("rotary_dim", self.head_dim))
        self.base = float(spec.params["base"])
        # linear scaling: every frequency divided by one factor (positions count as that much closer together)
        self.scaling_factor = float(spec.params.get("scaling_factor") or 1.0)
        if self.rotary_dim % 2 or not 0 <= self.rotary_dim <= self.head_dim:
            raise InvalidArgumentError(
                f"rotary_dim {self.rotary_dim} must be even and at most head_dim {self.head_dim}")
        if spec.params.get("wide_table"):
            table = self.base ** (-2.0 * np.arange(self.rotary_dim // 2, dtype=np.float64) / max(self.rotary_dim, 1))
        else:
            table = neox_inverse_frequencies(self.rotary_dim, self.base)
        if self.scaling_factor != 1.0:
            table = (table / np.float32(self.scaling_factor)).astype(np.float32)
        # ``long_waves``: {"factor", "low", "high", "original"}, see stretch_long_waves
        self.long_waves = spec.params.get("long_waves")
        if self.long_waves and self.rotary_dim:
            w = self.long_waves
            table = stretch_long_waves(table, float(w["factor"]), float(w["low"]), float(w["high"]), float(w["original"]))
        # ``ramp``: {"factor", "original", "fast", "slow"}, see blend_by_index; sines and cosines then grow, too
        self.ramp = spec.params.get("ramp")
        if self.ramp and self.rotary_dim:
            r = {key: float(self.ramp[key]) for key in ("factor", "original", "fast", "slow")}
            table = blend_by_index(table, self.rotary_dim, self.base, **r)
            self.amplitude = 0.1 * math.log(r["factor"]) + 1.0
        self.inv_freq = torch.from_numpy(np.asarray(table, dtype=np.float32)).to(runtime.device)

    def fused_rotary(self):
        return self.inv_freq, self.rotary_dim

    def step_angles(self, batch):
        # a prompt's tokens times all heads times all layers would compute the same few sines again and
        # again; a few decoded tokens are cheaper without the extra launch
        if not self.rotary_dim or (batch.num_tokens < ANGLE_TABLE_MIN_TOKENS and self.amplitude == 1.0):
            return None
        key = ("rope_angles", self.base, self.rotary_dim, self.scaling_factor, bool(self.spec.params.get("wide_table")),
               tuple(sorted(self.long_waves.items())) if self.long_waves else None,
               tuple(sorted(self.ramp.items())) if self.ramp else None)
        table = batch.shared.get(key)
        if table is None:
            table = batch.shared[key] = kernels.rope_angles(batch.positions, self.inv_freq, batch.num_tokens,
                                                                   self.amplitude)
        return table

    def apply(self, qkv, batch, heads, kv_heads, head_dim):
        kernels.rope_kvwrite(qkv, batch.positions, self.inv_freq, self.rotary_dim, None, None,
                             batch.entry_of_token, None, heads, kv_heads, head_dim, self.step_angles(batch))


def prompt_angles(position: PositionEncoding, batch, rotary_dim: int):
    """The table of the step's sines and cosines where the step has enough tokens to share one, else None: the kernel then
    computes them itself (with the position part's amplitude)."""
    return position.step_angles(batch) if rotary_dim and batch.num_tokens >= ANGLE_TABLE_MIN_TOKENS else None


class NoPosition(PositionEncoding):
    """No position encoding: queries and keys stay as projected."""

    def fused_rotary(self):
        return None, 0

    def apply(self, qkv, batch, heads, kv_heads, head_dim):
        return None


register_position("rotary_neox", RotaryNeox)
register_position("none", NoPosition)
