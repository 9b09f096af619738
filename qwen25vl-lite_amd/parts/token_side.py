"""A layer's own columns of a second table of token rows, gated by what the layer has made of the token."""

from __future__ import annotations

from typing import Dict, Optional

import torch

from ..ops import skinny
from ..ops.linear import linear, linear_into
from .base import FeedForward, ParamSpec, StepContext, register_part

__all__ = ["TokenSideInput"]


class TokenSideInput(FeedForward):
    """``Wproj (gelu(Wgate x) * e)``, ``e`` being columns ``first .. first + dim - 1`` of the token's row of the model's second
    table (``StepContext.token_side``) and gelu its tanh form.

    params: ``hidden_size``, ``dim``, ``first``, ``names`` (local names of the matrices: ``gate``, ``proj``; default these).
    """

    graph_safe = True

    def __init__(self, params, dtype, device):
        super().__init__(dtype, device)
        self.hidden, self.dim, self.first = int(params["hidden_size"]), int(params["dim"]), int(params["first"])
        names = dict(params.get("names") or {})
        self.names = {k: names.get(k, k) for k in ("gate", "proj")}
        self.w_gate: Optional[torch.Tensor] = None
        self.w_proj: Optional[torch.Tensor] = None

    def param_specs(self) -> Dict[str, ParamSpec]:
        return {f"{self.names['gate']}.weight": ParamSpec((self.dim, self.hidden)),
                f"{self.names['proj']}.weight": ParamSpec((self.hidden, self.dim))}

    def load(self, tensors):
        self.w_gate, self.w_proj = tensors[f"{self.names['gate']}.weight"], tensors[f"{self.names['proj']}.weight"]

    def named_weights(self) -> Dict[str, torch.Tensor]:
        return {f"{self.names['gate']}.weight": self.w_gate, f"{self.names['proj']}.weight": self.w_proj}

    def forward(self, x: torch.Tensor, step: StepContext):
        from ..ops.sum_norm import gelu_rows

        if step.token_side is None:
            raise RuntimeError("a layer reads a second table of token rows that the model does not have")
        z = linear(x, self.w_gate, out_dtype=torch.float32 if x.shape[0] <= skinny.ONE_BLOCK_ROWS else None)
        return linear_into(None, gelu_rows(z, step.token_side, self.first, step.token_ids), self.w_proj)


register_part("ffn", "token_side", TokenSideInput)
