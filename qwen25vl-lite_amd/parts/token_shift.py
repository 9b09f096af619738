"""A token's row mixed with the row of the token before it in its sequence."""

from __future__ import annotations

from typing import Dict, Optional, Sequence

import torch

from .base import Filter, LayerSlot, ParamSpec, Part, StateNeed, StepContext, register_part

__all__ = ["TokenShift", "TokenMixes"]


class TokenShift(Filter):
    """``h + (h' - h) w``, element by element, with ``h'`` the row of the token before as it was before this step
    (zeros for a sequence's first token).  A request's last row is its state (float32 ``[channels]``), so that a
    sequence may be cut into steps anywhere.

    params: ``channels``.
    """

    graph_safe = True

    def __init__(self, params, dtype, device):
        super().__init__(dtype, device)
        self.channels = int(params["channels"])
        self.weight: Optional[torch.Tensor] = None

    def state_need(self) -> StateNeed:
        return StateNeed((self.channels,), torch.float32)

    def param_specs(self) -> Dict[str, ParamSpec]:
        return {"weight": ParamSpec((self.channels,), "vector")}

    def load(self, tensors):
        self.weight = tensors["weight"]

    def named_weights(self) -> Dict[str, torch.Tensor]:
        return {"weight": self.weight}

    def forward(self, h: torch.Tensor, step: StepContext, slot: LayerSlot, mixes: Optional["TokenMixes"] = None,
                mixes_slot: Optional[LayerSlot] = None) -> torch.Tensor:
        """The shifted rows; with ``mixes`` the rows' mixes with the previous ones, ``[mixes, N, channels]``, formed
        in the same kernel."""
        from ..ops.previous_token import token_mix
        if slot is None or slot.state is None:
            raise RuntimeError("a step towards the previous token needs a state slot")
        more = {} if mixes is None else {"mu": mixes.mu, "prev_mixed": mixes_slot.state}
        return token_mix(h, step.cu_q, step.req_slots, step.token_req, self.dtype, shift=self.weight, prev=slot.state, **more)


class TokenMixes(Part):
    """Several mixes ``h + (h' - h) mu_name`` of a row with the row of the token before, one per name, each read by
    another projection.  A request's last row is its state.

    params: ``channels``, ``names`` (the local names of the weights, in the order the mixes come out).
    """

    graph_safe = True

    def __init__(self, params, dtype, device):
        super().__init__(dtype, device)
        self.channels = int(params["channels"])
        self.names: Sequence[str] = tuple(params["names"])
        self.mu: Optional[torch.Tensor] = None         # float32 [names, channels]

    def state_need(self) -> StateNeed:
        return StateNeed((self.channels,), torch.float32)

    def param_specs(self) -> Dict[str, ParamSpec]:
        return {f"{name}.weight": ParamSpec((self.channels,), "vector") for name in self.names}

    def load(self, tensors):
        self.mu = torch.stack([tensors[f"{name}.weight"] for name in self.names]).contiguous()

    def named_weights(self) -> Dict[str, torch.Tensor]:
        return {f"{name}.weight": self.mu[i] for i, name in enumerate(self.names)}

    def forward(self, h: torch.Tensor, step: StepContext, slot: LayerSlot) -> torch.Tensor:
        """``[N, channels]`` -> ``[names, N, channels]`` in the run dtype."""
        from ..ops.previous_token import token_mix
        if slot is None or slot.state is None:
            raise RuntimeError("mixes with the previous token need a state slot")
        return token_mix(h, step.cu_q, step.req_slots, step.token_req, self.dtype, mu=self.mu, prev_mixed=slot.state)


register_part("filter", "token_shift", TokenShift)
