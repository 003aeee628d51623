"""Two mixers side by side: both read the same input, and the result is a multiple of the sum of their outputs,
each scaled to a root mean square of one (over the model's width) and multiplied by a weight of its own.

params: left, right (PartSpecs of the two mixers), left_norm, right_norm (names of the weights [hidden]), hidden_size,
eps, scale (0.5).  At most one of the two keeps pages; their states lie one after the other among this mixer's.
What it hands on is a ``NormedSum``, which the block's norm takes apart in the pass that reads it.
"""
from __future__ import annotations

from typing import Dict, Mapping

import torch

from ..weights.loader import TensorSpec
from .base import MIXERS, Mixer, NormedSum, Runtime, StateNeed, register_mixer


class _Share:
    """One mixer's part of the pair's site: its own states, and the pages where they are its own."""

    def __init__(self, site, first: int, count: int, keeps_pages: bool):
        self._site, self._first, self._count = site, first, count
        self.info = site.info
        self.group = site.group if keeps_pages else None
        self.owns_cache = site.owns_cache and keeps_pages

    def kv(self):
        return self._site.kv() if self.group is not None else (None, None)

    def state(self, which: int = 0):
        return self._site.state(self._first + which) if which < self._count else None

    def states(self):
        return self._site.states()[self._first: self._first + self._count]


@register_mixer("side_by_side")
class SideBySide(Mixer):
    def __init__(self, params, rt: Runtime):
        super().__init__(params, rt)
        self.hidden = int(params["hidden_size"])
        self.eps = float(params["eps"])
        self.scale = float(params.get("scale", 0.5))
        self.norm_names = (params["left_norm"], params["right_norm"])
        handed = {"projects_kv": params["projects_kv"]} if "projects_kv" in params else {}
        self.mixers = tuple(MIXERS.get(p.kind)(dict(p.params, **handed), rt) for p in (params["left"], params["right"]))
        self.graph_capturable = all(m.graph_capturable for m in self.mixers)
        self._kv = tuple(m.kv_need() for m in self.mixers)
        if all(need is not None for need in self._kv):
            raise ValueError("of two mixers side by side, at most one keeps pages")
        needs = []
        for m in self.mixers:
            need = m.state_need()
            needs.append(() if need is None else ((need,) if isinstance(need, StateNeed) else tuple(need)))
        self._states = tuple(needs)
        self.weights = None

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        specs = {name: TensorSpec((self.hidden,), "float", ("one_plus_normal", 0.1)) for name in self.norm_names}
        for m in self.mixers:
            specs.update(m.tensor_specs())
        return specs

    def load(self, tensors: Mapping[str, torch.Tensor]) -> None:
        self.weights = tuple(tensors[name].contiguous() for name in self.norm_names)
        for m in self.mixers:
            m.load(tensors)

    def kv_need(self):
        return self._kv[0] if self._kv[0] is not None else self._kv[1]

    def state_need(self):
        return self._states[0] + self._states[1] or None

    def step_inputs(self):
        return {name: fn for m in self.mixers for name, fn in m.step_inputs().items()}

    def products(self):
        return tuple(p for m in self.mixers for p in m.products())

    def forward(self, h: torch.Tensor, ctx, site) -> NormedSum:
        ops = self.rt.ops
        left, right = self.mixers
        a = left.forward(h, ctx, _Share(site, 0, len(self._states[0]), self._kv[0] is not None))
        first = (a, self.weights[0], self.eps)
        if not isinstance(a, torch.Tensor):
            # a product's unreduced slices wait in the library's workspace, which the other mixer's products take:
            # they are summed and normed now
            first = (ops.rmsnorm(a, self.weights[0], self.eps, False, torch.float32), None, 0.0)
        b = right.forward(h, ctx, _Share(site, len(self._states[0]), len(self._states[1]), self._kv[1] is not None))
        return NormedSum(ops, (first, (b, self.weights[1], self.eps)), self.scale)
