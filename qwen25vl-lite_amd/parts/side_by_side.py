"""Two mixers that read the same input."""

from __future__ import annotations

from typing import Dict, Optional

import torch

from .base import LayerSlot, Mixer, NormedMean, ParamSpec, ScaledSum, Part, StepContext, build_part, register_part

__all__ = ["SideBySide"]


class SideBySide(Mixer):
    """``factor * (rmsnorm(left(x)) w_left + rmsnorm(right(x)) w_right)``, the norms over the model width with plain
    weights.  What it returns is a :class:`~qwen25vl_lite_amd.parts.base.NormedMean`, which the kernel that adds it to
    the residual forms on the way: the block it stands in must take one.  With ``norm`` False the two results join as
    they are, under a factor each (a :class:`~qwen25vl_lite_amd.parts.base.ScaledSum`).

    params: ``hidden_size``, ``eps``, ``left``, ``right`` (:class:`PartSpec` of a mixer each), ``factor`` (default 1/2),
    ``norm`` (default True), ``factors`` (left's and right's, without norms), ``names`` (local names of the two mixers and of the two weights: ``left``, ``right``, ``left_norm``, ``right_norm``).
    """

    graph_safe = True

    def __init__(self, params, dtype, device):
        super().__init__(dtype, device)
        self.hidden, self.eps = int(params["hidden_size"]), float(params["eps"])
        self.factor = float(params.get("factor", 0.5))
        self.norm = bool(params.get("norm", True))
        self.factors = tuple(float(f) for f in params.get("factors") or (1.0, 1.0))
        if len(self.factors) != 2:
            raise ValueError("two mixers have a factor each")
        names = dict(params.get("names") or {})
        self.names = {k: names.get(k, k) for k in ("left", "right", "left_norm", "right_norm")}
        self.left = build_part("mixer", params["left"], dtype, device)
        self.right = build_part("mixer", params["right"], dtype, device)
        for mixer in (self.left, self.right):
            if mixer.token_mixes is not None:
                raise ValueError("a mixer that stands beside another reads the input itself")
        self.w_left: Optional[torch.Tensor] = None
        self.w_right: Optional[torch.Tensor] = None

    def sub_parts(self) -> Dict[str, Part]:
        return {self.names["left"]: self.left, self.names["right"]: self.right}

    def param_specs(self) -> Dict[str, ParamSpec]:
        if not self.norm:
            return {}
        return {f"{self.names[k]}.weight": ParamSpec((self.hidden,), "vector", init="around_one")
                for k in ("left_norm", "right_norm")}

    def load(self, tensors):
        self.w_left = tensors[f"{self.names['left_norm']}.weight"]
        self.w_right = tensors[f"{self.names['right_norm']}.weight"]

    def named_weights(self) -> Dict[str, torch.Tensor]:
        return {} if not self.norm else {f"{self.names['left_norm']}.weight": self.w_left, f"{self.names['right_norm']}.weight": self.w_right}

    def forward(self, x: torch.Tensor, step: StepContext, slot: LayerSlot):
        residual, step.residual = step.residual, None     # the two results are normed before they join the sum
        left = self.left.forward(x, step, slot.of(self.names["left"]))
        right = self.right.forward(x, step, slot.of(self.names["right"]))
        step.residual = residual
        if not self.norm:
            return ScaledSum(left, right, *self.factors)
        return NormedMean(left, right, self.w_left, self.w_right, self.eps, self.factor)


register_part("mixer", "side_by_side", SideBySide)
