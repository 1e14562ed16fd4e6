"""Several residual streams per token: hyper-connections (Zhu et al., "Hyper-Connections").

Instead of one residual a token has ``streams`` of them, ``x_1 .. x_s``, all equal to the embedding's row at the start.
A sublayer with the learned ``in [s]``, ``out [s]`` and ``mix [s, s]`` reads ``u = sum_s in[s] x_s`` through its norm, gives
``y``, and then all streams at once become ``x_t <- sum_s mix[s, t] x_s + out[t] y``.  Behind the last layer the streams are
added up.

:class:`ResidualStreams` is what travels through the layers in place of the residual tensor.  It holds the streams and
the last sublayer's output that has not joined them yet: whoever reads next (the next sublayer's norm, the final norm)
has it joined, the streams weighed and the norm applied in one launch, so a sublayer costs one pass over the streams.
Block kind ``hyper``; norm kind ``summed`` (the norm behind the last layer, of the streams' sum).
"""
from __future__ import annotations

from typing import Dict, List, Optional

import torch

from ..config.base import LayerSpec, PartSpec
from ..errors import UnsupportedError
from ..ops import kernels
from ..weights.checkpoint import VECTOR, TensorSpec
from .base import Block, Norm, part_class, register_block, register_norm


class ResidualStreams:
    def __init__(self, rows: torch.Tensor, streams: int):
        self.held = rows                # [tokens, width] while all streams are equal, then [tokens, streams, width]
        self.streams = streams
        self.pending = None             # (y, mix, share) of the last sublayer

    @property
    def shape(self):
        return self.held.shape[0], self.held.shape[-1]

    def leave(self, y: torch.Tensor, mix: torch.Tensor, share: torch.Tensor) -> None:
        """A sublayer's output: it joins the streams with the next reading."""
        if self.pending is not None:
            self._pass(None, None, "none", None, None, 0.0)
        self.pending = (y, mix, share)

    def _pass(self, read, out, norm, weight, bias, eps) -> None:
        y, mix, share = self.pending or (None, None, None)
        into = None
        if y is not None:
            into = self.held if self.held.dim() == 3 else torch.empty(
                (self.held.shape[0], self.streams, self.held.shape[1]), dtype=torch.float32, device=self.held.device)
        kernels.streams_step(self.held, self.streams, y, mix, share, into, read, out, norm, weight, bias, eps)
        if into is not None:
            self.held, self.pending = into, None

    def read(self, weights: Optional[torch.Tensor], norm: Norm, runtime) -> torch.Tensor:
        """``norm(sum_s weights[s] x_s)`` in the run's dtype (``weights`` None: the plain sum)."""
        fused = norm.as_kernel()
        if fused is None:
            u = torch.empty(self.shape, dtype=torch.float32, device=self.held.device)
            self._pass(weights, u, "none", None, None, 0.0)
            return norm.forward(u)
        out = runtime.empty(self.shape)
        self._pass(weights, out, *fused)
        return out

    def read_rows(self, norm: Norm, rows: torch.Tensor, runtime) -> torch.Tensor:
        """``norm(sum_s x_s)`` of some tokens; the streams themselves are left as they are."""
        y, mix, share = self.pending or (None, None, None)
        fused = norm.as_kernel()
        shape = (rows.numel(), self.shape[1])
        out = runtime.empty(shape) if fused is not None else torch.empty(shape, dtype=torch.float32, device=self.held.device)
        kernels.streams_step(self.held, self.streams, y, mix, share, None, None, out,
                             *(fused or ("none", None, None, 0.0)), rows=rows)
        return out if fused is not None else norm.forward(out)

    def total(self) -> torch.Tensor:
        """The sum of the streams, 32-bit ``[tokens, width]``."""
        out = torch.empty(self.shape, dtype=torch.float32, device=self.held.device)
        self._pass(None, out, "none", None, None, 0.0)
        return out


class HyperBlock(Block):
    """Two sublayers over :class:`ResidualStreams`.  ``LayerSpec.params``: ``streams``, ``names`` (the tensors' names after
    the layer's prefix, one for each sublayer: ``<name>.in | out | mix``).  A layer whose feed-forward is ``none`` has only
    the first sublayer, and none of the second's tensors."""

    def __init__(self, spec: LayerSpec, runtime):
        super().__init__(spec, runtime)
        self.streams = int(spec.params["streams"])
        self.parts = {role: part_class(family, part.kind)(part, spec.prefix, runtime)
                      for role, family, part in self._roles(spec)}
        self.mixer = self.parts["mixer"]
        self.connections: List[tuple] = []

    @staticmethod
    def _sublayers(spec: LayerSpec) -> int:
        return 1 if spec.ffn.kind == "none" else 2

    @classmethod
    def _roles(cls, spec: LayerSpec):
        roles = [("mixer_norm", "norm", spec.mixer_norm), ("mixer", "mixer", spec.mixer), ("position", "position", spec.position)]
        if cls._sublayers(spec) == 2:
            roles += [("ffn_norm", "norm", spec.ffn_norm), ("ffn", "ffn", spec.ffn)]
        return roles

    @classmethod
    def _connection_specs(cls, spec: LayerSpec, index: int) -> List[TensorSpec]:
        base, s = f"{spec.prefix}{spec.params['names'][index]}.", int(spec.params["streams"])
        return [TensorSpec(base + "in", (s,), VECTOR, "one_plus_normal", std=0.2),
                TensorSpec(base + "out", (s,), VECTOR, "one_plus_normal", std=0.2),
                TensorSpec(base + "mix", (s, s), VECTOR, std=0.3)]

    @classmethod
    def declare(cls, spec: LayerSpec) -> List[TensorSpec]:
        out: List[TensorSpec] = []
        for _, family, part in cls._roles(spec):
            out += part_class(family, part.kind).declare(part, spec.prefix)
        for index in range(cls._sublayers(spec)):
            out += cls._connection_specs(spec, index)
        if cls._sublayers(spec) == 1:
            # nothing reads the second sublayer's norm and connection; a folder that stores them all the same is not
            # refused for it
            unread = part_class("norm", spec.ffn_norm.kind).declare(spec.ffn_norm, spec.prefix) + cls._connection_specs(spec, 1)
            out += [TensorSpec(t.name, t.shape, t.role, t.init, t.std, True) for t in unread]
        return out

    @classmethod
    def check_supported(cls, spec: LayerSpec, dtype: torch.dtype) -> None:
        if not 1 <= int(spec.params["streams"]) <= kernels.STREAMS_MAX:
            raise UnsupportedError(f"{spec.params['streams']} residual streams: 1 to {kernels.STREAMS_MAX} are implemented")
        for _, family, part in cls._roles(spec):
            part_class(family, part.kind).check_supported(part, dtype)

    def load(self, tensors: Dict[str, torch.Tensor]) -> None:
        for part in self.parts.values():
            part.load(tensors)
        for index in range(self._sublayers(self.spec)):
            base = f"{self.spec.prefix}{self.spec.params['names'][index]}."
            self.connections.append(tuple(tensors[base + n] for n in ("in", "out", "mix")))

    def forward(self, x: ResidualStreams, batch, cache, state, reads_only: bool = False) -> None:
        read, write, mix = self.connections[0]
        h = x.read(read, self.parts["mixer_norm"], self.runtime)
        y = self._output(self.mixer, x)
        kwargs = {"accumulate": False} if self.mixer.can_overwrite else {}
        self.mixer.forward(h, batch, cache, state, self.parts["position"], y, reads_only, **kwargs)
        x.leave(y, mix, write)
        if len(self.connections) == 2:
            read, write, mix = self.connections[1]
            ffn = self.parts["ffn"]
            h = x.read(read, self.parts["ffn_norm"], self.runtime)
            y = self._output(ffn, x)
            ffn.forward(h, batch, y, **({"accumulate": False} if ffn.can_overwrite else {}))
            x.leave(y, mix, write)

    @staticmethod
    def _output(part, x: ResidualStreams) -> torch.Tensor:
        make = torch.empty if part.can_overwrite else torch.zeros
        return make(x.shape, dtype=torch.float32, device=x.held.device)


class SummedNorm(Norm):
    """The norm ``params["norm"]`` (a PartSpec) of the sum of the residual streams."""

    def __init__(self, spec: PartSpec, prefix: str, runtime):
        super().__init__(spec, prefix, runtime)
        inner = spec.params["norm"]
        self.norm = part_class("norm", inner.kind)(inner, prefix, runtime)

    @classmethod
    def declare(cls, spec: PartSpec, prefix: str) -> List[TensorSpec]:
        return part_class("norm", spec.params["norm"].kind).declare(spec.params["norm"], prefix)

    @classmethod
    def check_supported(cls, spec: PartSpec, dtype: torch.dtype) -> None:
        part_class("norm", spec.params["norm"].kind).check_supported(spec.params["norm"], dtype)

    def load(self, tensors: Dict[str, torch.Tensor]) -> None:
        self.norm.load(tensors)

    def forward(self, x: ResidualStreams, out=None, rows=None):
        if rows is None:
            return x.read(None, self.norm, self.runtime)
        return x.read_rows(self.norm, rows, self.runtime)


register_block("hyper", HyperBlock)
register_norm("summed", SummedNorm)
