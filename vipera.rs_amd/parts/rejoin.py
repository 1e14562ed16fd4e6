"""Parts that bring the embedding's output back into the stream between layers (``ScheduleEntry.rejoins``).

``concat_linear``: ``x <- W [x; x0]``, ``x0`` being the embedding's output of the same tokens.  The product reads both side
by side in the run's dtype, and its 32-bit sums are the new stream.
"""
from __future__ import annotations

from typing import Dict, List

import torch

from ..config.base import PartSpec
from ..ops import kernels
from ..ops.linear import linear
from ..weights.checkpoint import MATRIX, TensorSpec
from .base import Part, register_rejoin

KEPT_ROWS = "rejoin.rows"      # key in ``batch.shared``: [tokens, 2 width] in the run's dtype, x0 in its right half


class ConcatLinear(Part):
    """``params``: ``width``, ``tensor`` (``[width, 2 width]``, the stream's columns first)."""

    def __init__(self, spec: PartSpec, prefix: str, runtime):
        super().__init__(spec, prefix, runtime)
        self.width = int(spec.params["width"])
        self.weight = None

    @classmethod
    def declare(cls, spec: PartSpec, prefix: str) -> List[TensorSpec]:
        width = int(spec.params["width"])
        return [TensorSpec(f"{prefix}{spec.params['tensor']}", (width, 2 * width), MATRIX)]

    def load(self, tensors: Dict[str, torch.Tensor]) -> None:
        self.weight = tensors[f"{self.prefix}{self.spec.params['tensor']}"]

    def keep(self, x: torch.Tensor, batch) -> None:
        rows = self.runtime.empty((x.shape[0], 2 * self.width))
        kernels.activation(x, "none", rows[:, self.width:])
        batch.shared[KEPT_ROWS] = rows

    def forward(self, x: torch.Tensor, batch) -> None:
        rows = batch.shared[KEPT_ROWS]
        kernels.activation(x, "none", rows[:, :self.width])
        linear(rows, self.weight, None, x)


register_rejoin("concat_linear", ConcatLinear)
