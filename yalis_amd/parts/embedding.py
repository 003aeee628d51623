"""Token embedding and output head.

Reference: yalis/external/model.py:137-141 (x = wte[ids], no scaling for Llama) and
:183-189 (logits = lm_head(ln_f(x)), no bias, no softcap), cast to float32 by the
engine (yalis/engine.py:96,136).  A tied head reads the embedding table (the
reference's converter copies it instead, yalis/external/convert_hf_checkpoint.py:856-875).
The head runs on the wanted rows only and writes float32 logits.
"""
from __future__ import annotations

from typing import Dict, Mapping

import torch

from ..weights.loader import TensorSpec
from .base import Part, Runtime, Settled, StateNeed, register_embedding, register_head


@register_embedding("token_embedding")
class TokenEmbedding(Part):
    """params: name, vocab_size, hidden_size, scale (1.0: what a token's row is multiplied with, in float32)."""

    graph_capturable = True

    def __init__(self, params, rt: Runtime):
        super().__init__(params, rt)
        self.name = params["name"]
        self.vocab = int(params["vocab_size"])
        self.hidden = int(params["hidden_size"])
        self.scale = float(params.get("scale", 1.0))
        self.table = None

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        return {self.name: TensorSpec((self.vocab, self.hidden))}

    def load(self, tensors: Mapping[str, torch.Tensor]) -> None:
        self.table = tensors[self.name]

    def forward(self, token_ids: torch.Tensor) -> torch.Tensor:
        """The float32 residual stream [N, hidden]."""
        if self.scale != 1.0:
            return self.rt.ops.embed(token_ids, self.table, scale=self.scale)
        return self.rt.ops.embed(token_ids, self.table)

    def begin(self, token_ids: torch.Tensor, lazily: bool):
        """(residual, delta) with which the first block starts: the gathered rows and nothing
        to add, or, ``lazily`` and where the kernel library can, an unfilled residual and the
        rows as a pending contribution that the first norm's kernel gathers itself (a block says
        through ``takes_embedded_rows`` whether its first norm does)."""
        make = getattr(self.rt.ops, "embedded_rows", None)
        if lazily and make is not None and self.scale == 1.0:
            return make(token_ids, self.table)
        return self.forward(token_ids), None


@register_embedding("token_position_embedding")
class TokenPositionEmbedding(TokenEmbedding):
    """The token's row plus a learned vector for its absolute position (not scaled), summed in float32.

    params: name, position_name (a table [max_positions, hidden]), vocab_size, hidden_size, max_positions."""

    graph_capturable = True
    needs_positions = True

    def __init__(self, params, rt: Runtime):
        super().__init__(params, rt)
        self.position_name = params["position_name"]
        self.max_positions = int(params["max_positions"])
        self.position_table = None

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        return {self.name: TensorSpec((self.vocab, self.hidden)), self.position_name: TensorSpec((self.max_positions, self.hidden))}

    def load(self, tensors: Mapping[str, torch.Tensor]) -> None:
        self.table = tensors[self.name]
        self.position_table = tensors[self.position_name].contiguous()

    def forward(self, token_ids: torch.Tensor, positions: torch.Tensor = None) -> torch.Tensor:
        if positions is None:
            raise ValueError("this embedding adds a vector per position: it needs the tokens' positions")
        return self.rt.ops.embed(token_ids, self.table, positions=positions, position_table=self.position_table)

    def begin(self, token_ids: torch.Tensor, lazily: bool, positions: torch.Tensor = None):
        return self.forward(token_ids, positions), None


@register_embedding("token_pair_embedding")
class TokenPairEmbedding(TokenEmbedding):
    """The token's scaled row plus a row for the pair (token before it, token), summed in float32: row
    (before * mul_prev + token * mul_cur) mod buckets of a second table [buckets + 1, hidden]; a sequence's
    first token, which has none before it, takes the last row.  The token before a step's first one is the
    request's state (one int32, -1 before the first token).

    params: name, vocab_size, hidden_size, scale, pair_name, buckets, mul_prev, mul_cur."""

    graph_capturable = True
    keeps_state = True

    def __init__(self, params, rt: Runtime):
        super().__init__(params, rt)
        self.pair_name = params["pair_name"]
        self.buckets = int(params["buckets"])
        self.mul_prev, self.mul_cur = int(params["mul_prev"]), int(params["mul_cur"])
        # (the row number is an unsigned 64-bit sum on the device)
        if min(self.mul_prev, self.mul_cur) < 0 or max(self.mul_prev, self.mul_cur) * self.vocab >= 1 << 62:
            raise ValueError(f"{self.pair_name}: multipliers {self.mul_prev} and {self.mul_cur} are out of range")
        self.pair_table = None

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        return {self.name: TensorSpec((self.vocab, self.hidden)), self.pair_name: TensorSpec((self.buckets + 1, self.hidden))}

    def load(self, tensors: Mapping[str, torch.Tensor]) -> None:
        self.table, self.pair_table = tensors[self.name].contiguous(), tensors[self.pair_name].contiguous()
        if self.pair_table.dtype != self.table.dtype:
            self.table, self.pair_table = self.table.float(), self.pair_table.float()

    def state_need(self) -> StateNeed:
        return StateNeed((1,), torch.int32, -1)

    def begin(self, ctx, site):
        """(the float32 residual stream, ``Settled`` with its copy in the activation dtype)."""
        residual, rounded = self.rt.ops.embed_pairs(
            ctx.arrays["token_ids"], self.table, self.scale, self.pair_table, self.buckets, self.mul_prev, self.mul_cur,
            site.state(0), ctx, self.rt.act_dtype)
        return residual, Settled(rounded)


@register_embedding("normed_token_embedding")
class NormedTokenEmbedding(TokenEmbedding):
    """The token's row through an RMS norm with a weight, float32: the stream starts normed.  ``streams`` (None: one
    stream, [N, hidden]): the stream is kept as that many copies [N, streams, hidden], all equal at the start.

    params: name, norm_name (the norm's weight), eps, vocab_size, hidden_size, streams."""

    graph_capturable = True

    def __init__(self, params, rt: Runtime):
        super().__init__(params, rt)
        self.norm_name = params["norm_name"]
        self.eps = float(params["eps"])
        self.streams = params.get("streams")
        self.norm_weight = None

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        return {self.name: TensorSpec((self.vocab, self.hidden)), self.norm_name: TensorSpec((self.hidden,), "float", ("one_plus_normal", 0.1))}

    def load(self, tensors: Mapping[str, torch.Tensor]) -> None:
        self.table, self.norm_weight = tensors[self.name].contiguous(), tensors[self.norm_name].contiguous()
        if self.norm_weight.dtype != self.table.dtype:
            self.table, self.norm_weight = self.table.float(), self.norm_weight.float()

    def forward(self, token_ids: torch.Tensor) -> torch.Tensor:
        x = self.rt.ops.embed_norm(token_ids, self.table, self.norm_weight, self.eps, 1 if self.streams is None else int(self.streams))
        return x[:, 0] if self.streams is None else x

    def begin(self, token_ids: torch.Tensor, lazily: bool):
        return self.forward(token_ids), None


@register_head("lm_head")
class LMHead(Part):
    """params: name, tied_to (name of the embedding table, or None), vocab_size,
    hidden_size, scale (1.0: what the logits are multiplied with), softcap (None; c: logits are squashed to
    c tanh(z / c), after the scale)."""

    graph_capturable = True

    def __init__(self, params, rt: Runtime):
        super().__init__(params, rt)
        self.name = params["name"]
        self.tied_to = params.get("tied_to")
        self.vocab = int(params["vocab_size"])
        self.hidden = int(params["hidden_size"])
        self.scale = float(params.get("scale", 1.0))
        self.softcap = float(params.get("softcap") or 0.0)
        self.weight = None

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        if self.tied_to is not None:
            return {self.tied_to: TensorSpec((self.vocab, self.hidden))}
        return {self.name: TensorSpec((self.vocab, self.hidden))}

    def load(self, tensors: Mapping[str, torch.Tensor]) -> None:
        self.weight = tensors[self.tied_to if self.tied_to is not None else self.name]
        if self.tied_to is None:
            # a table of its own: kept the way the kernel library streams it best (a tied table
            # stays as the embedding gathers from it)
            keep = getattr(self.rt.ops, "streamed_matrix", None)
            if keep is not None:
                self.weight = keep(self.weight)

    def products(self):
        return ((self.vocab, self.hidden),)

    def forward(self, h: torch.Tensor) -> torch.Tensor:
        logits = self.rt.ops.linear(h, self.weight, torch.float32)
        if self.softcap:
            self.rt.ops.scale_rows(logits, self.scale, softcap=self.softcap)
        elif self.scale != 1.0:
            self.rt.ops.scale_rows(logits, self.scale)
        return logits
