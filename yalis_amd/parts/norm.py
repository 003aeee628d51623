"""RMS normalisation (reference: yalis/external/model.py:957-989).

out = x * rsqrt(mean(x^2) + eps) * weight, all in float32 with one rounding at
the end; ``unit_offset`` multiplies by (1 + weight) instead (a flag of the same
class in the reference, :984).  The kernel fuses the residual sum that precedes
every norm of a pre-norm block: the float32 residual stream is updated in place
and normalised in one pass.  ``norm_add`` is the other way round, for blocks that norm a
branch's output instead of its input: residual += norm(branch), again one pass.  ``sum_norm`` is
for blocks that norm the stream itself after the branch has joined it: residual = norm(a * residual +
branch), with an optional weight per element on the branch (a layer scale), one pass too.  ``streams_norm`` is for a
stream kept as several copies: it mixes them, adds the branch, and norms the sum that the next branch reads, one pass again.
"""
from __future__ import annotations

from typing import Dict, Mapping, Optional

import torch

from ..weights.loader import TensorSpec
from .base import ExpertRows, Norm, NormedBranch, NormedSum, PlusRow, Runtime, Settled, StreamMix, register_norm


@register_norm("rmsnorm")
class RMSNorm(Norm):
    """params: name (checkpoint tensor), size, eps, unit_offset, branch_weight (None, or the name of a
    tensor [size]: what ``sum_norm`` multiplies a branch with, element by element, before it joins the
    stream)."""

    graph_capturable = True

    def __init__(self, params, rt: Runtime):
        super().__init__(params, rt)
        self.name = params["name"]
        self.size = int(params["size"])
        self.eps = float(params["eps"])
        self.unit_offset = bool(params.get("unit_offset", False))
        self.weight: Optional[torch.Tensor] = None
        self.branch_weight_name = params.get("branch_weight")
        self.branch_weight: Optional[torch.Tensor] = None
        self.takes_embedded_rows = hasattr(rt.ops, "embedded_rows")

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        # (random weights: around the value that leaves a row as it is, 0 where 1 is added)
        specs = {self.name: TensorSpec((self.size,), "float", ("normal", 0.1) if self.unit_offset else ("one_plus_normal", 0.1))}
        if self.branch_weight_name:
            specs[self.branch_weight_name] = TensorSpec((self.size,), "float", ("one_plus_normal", 0.1))
        return specs

    def load(self, tensors: Mapping[str, torch.Tensor]) -> None:
        self.weight = tensors[self.name]
        if self.branch_weight_name:
            self.branch_weight = tensors[self.branch_weight_name].contiguous()
            if self.branch_weight.dtype != self.weight.dtype:
                self.weight, self.branch_weight = self.weight.float(), self.branch_weight.float()

    def norm(self, x):
        if isinstance(x, NormedSum):
            x = x.combine()
        return self.rt.ops.rmsnorm(x, self.weight, self.eps, self.unit_offset, self.rt.act_dtype)

    def add_norm(self, residual, delta):
        row = None
        if isinstance(delta, PlusRow):  # a vector for every token joins the stream in the same pass
            delta, row = delta.inner, delta.row
        if isinstance(delta, NormedBranch):
            delta = delta.settle(residual)
        if isinstance(delta, Settled):
            delta = None
        if isinstance(delta, NormedSum):
            delta = delta.combine()
        if row is not None:
            return self.rt.ops.add_rmsnorm(residual, delta, self.weight, self.eps, self.unit_offset, self.rt.act_dtype, row=row)
        return self.rt.ops.add_rmsnorm(
            residual, delta, self.weight, self.eps, self.unit_offset, self.rt.act_dtype
        )

    def norm_add(self, residual, branch, expert_rows=None, expert_weight=1.0, scale=1.0):
        if scale != 1.0:
            raise ValueError("this norm adds its branch unscaled")
        if isinstance(branch, NormedSum) or (isinstance(branch, ExpertRows) and branch.row_weights is not None):
            branch = branch.combine()  # (rows with weights of their own are summed first)
        if isinstance(branch, ExpertRows):
            branch, expert_rows, expert_weight = branch.dense, branch.rows, branch.weight
        return self.rt.ops.norm_add(residual, branch, self.weight, self.eps, self.unit_offset, self.rt.act_dtype,
                                    expert_rows=expert_rows, expert_weight=expert_weight)

    def sum_norm(self, residual, branch, residual_scale=1.0):
        if isinstance(branch, ExpertRows):
            branch = branch.combine()
        terms, scale = (branch.terms, branch.scale) if isinstance(branch, NormedSum) else (((branch, None, 0.0),), 1.0)
        return self.rt.ops.sum_norm(residual, terms, scale, self.branch_weight, residual_scale, self.weight, self.eps,
                                    self.unit_offset, self.rt.act_dtype)

    def streams_norm(self, residual, delta, read, rows=None):
        if delta is not None and not isinstance(delta, StreamMix):
            raise TypeError(f"a stream kept as copies takes contributions that say how they mix, got {type(delta).__name__}")
        y, mix, out = (None, None, None) if delta is None else (delta.inner, delta.mix, delta.out)
        experts = None
        if isinstance(y, NormedSum):
            y = y.combine()
        if isinstance(y, ExpertRows):
            y, experts = y.dense, (y.rows, y.top, y.weight, y.row_weights)
        return self.rt.ops.streams_norm(residual, y, experts, mix, out, read, rows, self.weight, self.eps, self.unit_offset, self.rt.act_dtype)

    def gather_add_norm(self, residual, delta, rows):
        if residual.dim() == 3:  # copies of the stream: the final norm reads their sum
            return self.streams_norm(residual, delta, None, rows)
        if isinstance(delta, PlusRow):
            delta = delta.settle(residual)
        if isinstance(delta, NormedBranch):
            delta = delta.settle(residual)
        if isinstance(delta, Settled):
            delta = None
        if isinstance(delta, NormedSum):
            delta = delta.combine()
        return self.rt.ops.gather_add_rmsnorm(
            residual, delta, rows, self.weight, self.eps, self.unit_offset, self.rt.act_dtype
        )


@register_norm("layernorm")
class LayerNorm(Norm):
    """(x - mean) / sqrt(variance + eps) * weight + bias over a row, the variance the mean of the
    squared deviations; float32 arithmetic, one rounding at the end.

    params: name (weight tensor), bias (bias tensor's name, or None: no bias), size, eps, center
    (True; False: no mean is taken off, which makes it an RMS norm with an optional bias).

    One kernel (``ops.sandwich_norm``) serves every place a block may put it: a pending
    contribution, plain or itself normed and scaled (``NormedBranch``), is added into the float32
    residual and the new residual normed in the same pass."""

    graph_capturable = True

    def __init__(self, params, rt: Runtime):
        super().__init__(params, rt)
        self.name = params["name"]
        self.bias_name = params.get("bias")
        self.size = int(params["size"])
        self.eps = float(params["eps"])
        self.center = bool(params.get("center", True))
        self.weight: Optional[torch.Tensor] = None
        self.bias: Optional[torch.Tensor] = None

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        specs = {self.name: TensorSpec((self.size,), "float", ("one_plus_normal", 0.1))}
        if self.bias_name:
            specs[self.bias_name] = TensorSpec((self.size,), "float", ("normal", 0.1))
        return specs

    def load(self, tensors: Mapping[str, torch.Tensor]) -> None:
        self.weight = tensors[self.name].contiguous()
        self.bias = tensors[self.bias_name].contiguous() if self.bias_name else None
        if self.bias is not None and self.bias.dtype != self.weight.dtype:
            self.weight, self.bias = self.weight.float(), self.bias.float()

    def constants(self):
        """What the kernel library needs of a norm: (weight, bias or None, eps, center)."""
        return (self.weight, self.bias, self.eps, self.center)

    def _pending(self, residual, delta):
        """(branch, its norm's constants or None, scale) of a pending contribution."""
        if isinstance(delta, PlusRow):
            delta = delta.settle(residual)
        if isinstance(delta, Settled) or delta is None:
            return None, None, 1.0
        if isinstance(delta, NormedBranch):
            if not isinstance(delta.norm, LayerNorm):
                delta.settle(residual)
                return None, None, 1.0
            return delta.branch, delta.norm.constants(), delta.scale
        return (delta.combine() if isinstance(delta, NormedSum) else delta), None, 1.0

    def norm(self, x):
        return self.rt.ops.sandwich_norm(None, x, None, 1.0, self.constants(), None, self.rt.act_dtype)

    def add_norm(self, residual, delta):
        branch, post, scale = self._pending(residual, delta)
        return self.rt.ops.sandwich_norm(residual, branch, post, scale, self.constants(), None, self.rt.act_dtype)

    def gather_add_norm(self, residual, delta, rows):
        branch, post, scale = self._pending(residual, delta)
        return self.rt.ops.sandwich_norm(residual, branch, post, scale, self.constants(), rows, self.rt.act_dtype)

    def norm_add(self, residual, branch, expert_rows=None, expert_weight=1.0, scale=1.0):
        if isinstance(branch, (ExpertRows, NormedSum)):
            branch = branch.combine()
        elif expert_rows is not None:
            raise ValueError("this norm takes its branch combined")
        self.rt.ops.sandwich_norm(residual, branch, self.constants(), scale, None, None, self.rt.act_dtype)
        return self.rt.ops.round_rows(residual, self.rt.act_dtype)
