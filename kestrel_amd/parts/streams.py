"""Hyper-connections: how a sublayer reads and writes several copies of the residual stream."""

from __future__ import annotations

from typing import Dict, Optional

import torch

from .base import Norm, Part, register_stream_mix
from .specs import ParamSpec, StreamMixSpec


class StreamMix(Part):
    """The numbers of one sublayer (tensors ``in``, ``out`` ``[S]`` and ``mix`` ``[S, S]``, indexed from and to): it reads
    ``sum_s in[s] x_s``, and with its output ``y`` the streams become, all at once from the old ones,
    ``x_t <- sum_s mix[s, t] x_s + out[t] y``. Held in fp32; ``ops.core.streams_step`` does both."""

    replays_every_step = True

    def __init__(self, spec: StreamMixSpec) -> None:
        super().__init__(spec)
        if spec.streams <= 0:
            raise ValueError("a stream mix needs a positive number of streams")
        self.into: Optional[torch.Tensor] = None
        self.out: Optional[torch.Tensor] = None
        self.matrix: Optional[torch.Tensor] = None

    def params(self) -> Dict[str, ParamSpec]:
        S = self.spec.streams
        return {"in": ParamSpec((S,), "vector", "share"), "out": ParamSpec((S,), "vector", "open"), "mix": ParamSpec((S, S), "matrix", "identity")}

    def bind(self, tensors, dtype, device) -> None:
        f32 = dict(device=device, dtype=torch.float32)
        self.into, self.out, self.matrix = (tensors[name].to(**f32).contiguous() for name in ("in", "out", "mix"))


class StreamReading:
    """What a reader of the streams sees: the norm of ``sum_s in[s] x_s`` (``mix`` ``None``: of the sum of the streams)."""

    def __init__(self, mix: Optional[StreamMix], norm: Norm) -> None:
        self.mix, self.norm = mix, norm

    def operands(self):
        """As ``ops.core.streams_step`` takes them."""
        ln = self.norm.layernorm_operands()
        if ln is not None:
            form = ("layernorm", *ln)
        else:
            rms = self.norm.rms_operands()
            if rms is None:
                raise ValueError("streams are read through a layer norm or a root-mean-square norm")
            form = ("rms", rms[0], None, rms[1])
        return (None if self.mix is None else self.mix.into), form


register_stream_mix("stream_mix", StreamMix)
