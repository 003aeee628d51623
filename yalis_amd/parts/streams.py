"""A residual stream kept as several copies in place of one (Zhu et al., "Hyper-Connections"): every branch reads a weighted
sum of the copies, and its output goes back while all of them are mixed anew:

    u = sum_s in[s] x_s,   y = branch(norm(u)),   x_t <- sum_s mix[s, t] x_s + out[t] y   (all t from the old x_s)

The copies start equal and the model reads their sum at the end.  The stream's tensor is then [N, streams, width]
(float32); one kernel between two branches (``ops.streams_norm``) mixes the copies, adds the branch's output, takes the next
branch's weighted sum and norms it.

params: prefix, streams, names (optional overrides of "in", "out", "mix" below the prefix)."""
from __future__ import annotations

from typing import Dict, Mapping

import torch

from ..weights.loader import TensorSpec
from .base import Runtime, StreamMix, Streams, register_streams


@register_streams("mixed_streams")
class MixedStreams(Streams):
    graph_capturable = True

    def __init__(self, params, rt: Runtime):
        super().__init__(params, rt)
        self.prefix = params["prefix"]
        self.streams = int(params["streams"])
        names = {"in": "in", "out": "out", "mix": "mix"}
        names.update(params.get("names", {}))
        self.names = {k: f"{self.prefix}.{v}" for k, v in names.items()}
        self.read = self.out = self.mix = None

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        s = self.streams
        return {self.names["in"]: TensorSpec((s,), "float", ("normal", 0.5)), self.names["out"]: TensorSpec((s,), "float", ("one_plus_normal", 0.1)),
                self.names["mix"]: TensorSpec((s, s), "float", ("normal", 0.5))}

    def load(self, tensors: Mapping[str, torch.Tensor]) -> None:
        self.read, self.out, self.mix = (tensors[self.names[n]].to(torch.float32).contiguous() for n in ("in", "out", "mix"))

    def write(self, y) -> StreamMix:
        return StreamMix(y, self.mix, self.out)
