"""A recurrence over outer products by the delta rule, with one decay and one gate of writing per head and token.

``q = Wq h``, ``k = Wk h`` (groups of ``key_dim``), ``v = Wv h`` (heads of ``value_dim``) each pass a short causal
convolution per channel and silu; q and k become unit vectors, q times ``key_dim^(-1/2)``; ``beta = sigmoid(Wb h)``, decay
``a = exp(-exp(A_log) softplus(Wa h + b))``; per head ``S <- a S``, ``u = beta (v - S^T k)``, ``S <- S + k u^T``, ``o = S^T q``;
each head's ``o`` divided by its root mean square, times a shared weight, times ``silu(Wg h)``; then ``Wo``.
"""

from __future__ import annotations

from typing import Dict, Optional

import torch

from ..ops.linear import linear_into
from .base import LayerSlot, Mixer, ParamSpec, Part, StateNeed, StepContext, register_part
from .state_space import ConvolvedInput, chunk_plan, split_projection

__all__ = ["GatedDelta"]

UNIT_FLOOR = 1e-6       # under the root of a unit vector's sum of squares


class GatedDelta(Mixer):
    """params: ``hidden_size``, ``num_heads``, ``num_kv_heads`` (groups of queries and keys), ``key_dim``, ``value_dim``,
    ``conv_taps``, ``eps`` (of the heads' norm), ``unit_floor`` (default 1e-6), ``names`` (local names of the tensors'
    owners: ``q``, ``k``, ``v``, ``g``, ``b``, ``a``, ``q_conv``, ``k_conv``, ``v_conv``, ``a_log``, ``dt_bias``, ``norm``,
    ``o``; default these).

    q, k, v and the gate are projected (and convolved) in the run dtype, the inputs of beta and the decay in float32;
    unit lengths, decays, the state (float32 ``[heads, key_dim, value_dim]`` per request), outputs and their norm are
    float32.
    """

    graph_safe = True

    def __init__(self, params, dtype, device):
        super().__init__(dtype, device)
        self.hidden, self.heads, self.groups = int(params["hidden_size"]), int(params["num_heads"]), int(params["num_kv_heads"])
        self.dim, self.vdim, self.eps = int(params["key_dim"]), int(params["value_dim"]), float(params["eps"])
        self.unit_floor = float(params.get("unit_floor", UNIT_FLOOR))
        if self.heads % self.groups:
            raise ValueError(f"{self.heads} heads are not a multiple of {self.groups} query/key groups")
        names = dict(params.get("names") or {})
        self.names = {k: names.get(k, k) for k in ("q", "k", "v", "g", "b", "a", "q_conv", "k_conv", "v_conv", "a_log",
                                                   "dt_bias", "norm", "o")}
        self.taps = int(params["conv_taps"])
        self.conv = ConvolvedInput(2 * self.groups * self.dim + self.heads * self.vdim, self.taps, dtype, device, bias=False,
                                   own_tensors=False)
        self.w_in: Optional[torch.Tensor] = None
        self.dt_bias: Optional[torch.Tensor] = None
        self.a_log: Optional[torch.Tensor] = None
        self.a_neg: Optional[torch.Tensor] = None       # float32 [heads]: -exp(a_log)
        self.w_norm: Optional[torch.Tensor] = None
        self.w_out: Optional[torch.Tensor] = None

    def sub_parts(self) -> Dict[str, Part]:
        return {"conv": self.conv}

    def state_need(self) -> StateNeed:
        return StateNeed((self.heads, self.dim, self.vdim), torch.float32)

    def _stacked(self):
        """``(role, rows)`` of the matrices of the input product, in order; b and a last."""
        gd, hv = self.groups * self.dim, self.heads * self.vdim
        return [("q", gd), ("k", gd), ("v", hv), ("g", hv), ("b", self.heads), ("a", self.heads)]

    def param_specs(self) -> Dict[str, ParamSpec]:
        n, rows = self.names, dict(self._stacked())
        specs = {f"{n[role]}.weight": ParamSpec((r, self.hidden)) for role, r in rows.items()}
        specs.update({f"{n[s + '_conv']}.weight": ParamSpec((rows[s], self.taps), "vector") for s in "qkv"})
        specs.update({f"{n['a_log']}.weight": ParamSpec((self.heads,), "vector"),
                      f"{n['dt_bias']}.weight": ParamSpec((self.heads,), "vector"),
                      f"{n['norm']}.weight": ParamSpec((self.vdim,), "vector", init="around_one"),
                      f"{n['o']}.weight": ParamSpec((self.hidden, self.heads * self.vdim))})
        return specs

    def load(self, tensors):
        n = self.names
        self.w_in = torch.cat([tensors[f"{n[role]}.weight"] for role, _ in self._stacked()], dim=0).contiguous()
        self.conv.take(torch.cat([tensors[f"{n[s + '_conv']}.weight"] for s in "qkv"], dim=0))
        self.a_log, self.dt_bias = tensors[f"{n['a_log']}.weight"], tensors[f"{n['dt_bias']}.weight"]
        self.a_neg = (-torch.exp(self.a_log.double())).float().contiguous()
        self.w_norm, self.w_out = tensors[f"{n['norm']}.weight"], tensors[f"{n['o']}.weight"]

    def named_weights(self) -> Dict[str, torch.Tensor]:
        n, at, out = self.names, 0, {}
        taps = self.conv.weight.t()
        for role, rows in self._stacked():
            out[f"{n[role]}.weight"] = self.w_in[at:at + rows]
            if role in "qkv":
                out[f"{n[role + '_conv']}.weight"] = taps[at:at + rows]
            at += rows
        out.update({f"{n['a_log']}.weight": self.a_log, f"{n['dt_bias']}.weight": self.dt_bias,
                    f"{n['norm']}.weight": self.w_norm, f"{n['o']}.weight": self.w_out})
        return out

    def forward(self, x: torch.Tensor, step: StepContext, slot: LayerSlot):
        from ..ops.gated import group_norm_gate
        from ..ops.head_scan import head_scan

        if slot.state is None:
            raise RuntimeError("a recurrence by the delta rule needs a state slot")
        gd, hv = self.groups * self.dim, self.heads * self.vdim
        cols = 2 * gd + hv
        main, raw, at = split_projection(x, self.w_in, cols + hv)
        u = self.conv.forward(main[:, :cols], step, slot.of("conv"))
        o = head_scan(u, 0, gd, 2 * gd, self.heads, self.groups, self.dim, self.vdim, raw, at + self.heads, self.dt_bias,
                      self.a_neg, slot.state, step.cu_q, step.req_slots, beta_off=at, unit_eps=self.unit_floor,
                      q_scale=self.dim ** -0.5, plan=chunk_plan(step, self.dim, self.device))
        y = group_norm_gate(o, self.w_norm, self.vdim, self.eps, self.dtype, gate=main[:, cols:cols + hv], gate_act="silu")
        return linear_into(step.residual, y, self.w_out)


register_part("mixer", "gated_delta", GatedDelta)
