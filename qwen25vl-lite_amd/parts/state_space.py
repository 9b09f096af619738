"""State-space mixers.

The selective one (decays per channel and state): a short convolution, step sizes and projections that depend on the token, and a
diagonal recurrence per channel.

``[x; z] = Win h``; ``x`` passes a causal convolution per channel with a bias and silu; ``[dt; B; C] = Wx x``; step
sizes ``softplus(Wdt dt + b)``, one per channel; per channel c and state n ``S <- exp(step_c A[c, n]) S + step_c x_c B_n``,
``y_c = sum_n S[c, n] C_n + D_c x_c``; then ``Wo (y silu(z))``.  The dual one has one decay per head and token
(:class:`StateSpaceDual`).
"""

from __future__ import annotations

from typing import Dict, Optional

import torch

from ..ops import skinny
from ..ops.linear import linear, linear_into
from .base import LayerSlot, Mixer, ParamSpec, Part, StateNeed, StepContext, register_part

__all__ = ["SelectiveStateSpace", "StateSpaceDual", "ConvolvedInput"]


class ConvolvedInput(Part):
    """``silu([b +] sum_j w[:, j] x_(t - taps + 1 + j))`` per channel, zeros before a sequence's first token.  The last
    ``taps - 1`` rows a request has brought are its state (float32, oldest first).  The weight is ``[channels, taps]``
    in a checkpoint and kept tap-major in float32.  ``own_tensors`` False: the mixer it belongs to holds the tensors
    (several of them, say) and hands them over with :meth:`take`."""

    graph_safe = True

    def __init__(self, channels: int, taps: int, dtype, device, bias: bool = True, own_tensors: bool = True):
        super().__init__(dtype, device)
        self.channels, self.taps = int(channels), int(taps)
        self.has_bias, self.own_tensors = bool(bias), bool(own_tensors)
        if self.taps < 1:
            raise ValueError("a convolution has at least one tap")
        self.weight: Optional[torch.Tensor] = None
        self.bias: Optional[torch.Tensor] = None

    def state_need(self) -> Optional[StateNeed]:
        return StateNeed((self.taps - 1, self.channels), torch.float32) if self.taps > 1 else None

    def param_specs(self) -> Dict[str, ParamSpec]:
        if not self.own_tensors:
            return {}
        specs = {"weight": ParamSpec((self.channels, self.taps), "vector")}
        if self.has_bias:
            specs["bias"] = ParamSpec((self.channels,), "vector")
        return specs

    def load(self, tensors):
        self.take(tensors["weight"], tensors.get("bias"))

    def take(self, weight: torch.Tensor, bias: Optional[torch.Tensor] = None) -> None:
        """``weight [channels, taps]`` and the bias, if any, in float32."""
        self.weight, self.bias = weight.t().contiguous(), bias

    def named_weights(self) -> Dict[str, torch.Tensor]:
        out = {"weight": self.weight.t()} if self.own_tensors else {}
        if self.own_tensors and self.has_bias:
            out["bias"] = self.bias
        return out

    def forward(self, x: torch.Tensor, step: StepContext, slot: LayerSlot) -> torch.Tensor:
        from ..ops.short_conv import short_conv
        if self.taps > 1 and slot.state is None:
            raise RuntimeError("a convolution with more than one tap needs a state slot")
        return short_conv(x, self.weight, slot.state if self.taps > 1 else None, step.cu_q, step.req_slots,
                          step.token_req, self.dtype, bias=self.bias, silu=True)


class SelectiveStateSpace(Mixer):
    """params: ``hidden_size``, ``inner_size``, ``state_size``, ``dt_rank``, ``conv_taps``, ``names`` (local names of the
    tensors' owners: ``in``, ``conv``, ``x``, ``dt``, ``a_log``, ``d``, ``o``; default these).

    The input projection and what the convolution gives are in the run dtype; step sizes, decays, B, C and the state
    (float32 ``[state_size, inner_size]`` per request) are float32.
    """

    graph_safe = True

    def __init__(self, params, dtype, device):
        super().__init__(dtype, device)
        self.hidden, self.inner = int(params["hidden_size"]), int(params["inner_size"])
        self.states, self.rank = int(params["state_size"]), int(params["dt_rank"])
        names = dict(params.get("names") or {})
        self.names = {k: names.get(k, k) for k in ("in", "conv", "x", "dt", "a_log", "d", "o")}
        self.conv = ConvolvedInput(self.inner, int(params["conv_taps"]), dtype, device)
        self.w_in: Optional[torch.Tensor] = None
        self.w_x: Optional[torch.Tensor] = None
        self.w_dt: Optional[torch.Tensor] = None
        self.b_dt: Optional[torch.Tensor] = None
        self.a_log: Optional[torch.Tensor] = None
        self.a2: Optional[torch.Tensor] = None          # float32 [states, inner]: -exp(a_log) log2(e)
        self.skip: Optional[torch.Tensor] = None
        self.w_out: Optional[torch.Tensor] = None

    def sub_parts(self) -> Dict[str, Part]:
        return {self.names["conv"]: self.conv}

    def state_need(self) -> StateNeed:
        return StateNeed((self.states, self.inner), torch.float32)

    def param_specs(self) -> Dict[str, ParamSpec]:
        n, c = self.names, self.inner
        return {f"{n['in']}.weight": ParamSpec((2 * c, self.hidden)),
                f"{n['x']}.weight": ParamSpec((self.rank + 2 * self.states, c)),
                f"{n['dt']}.weight": ParamSpec((c, self.rank)),
                f"{n['dt']}.bias": ParamSpec((c,), "vector"),
                f"{n['a_log']}.weight": ParamSpec((c, self.states), "vector"),
                f"{n['d']}.weight": ParamSpec((c,), "vector", init="around_one"),
                f"{n['o']}.weight": ParamSpec((self.hidden, c))}

    def load(self, tensors):
        from ..ops.selective_scan import LOG2_E
        n = self.names
        self.w_in, self.w_x = tensors[f"{n['in']}.weight"], tensors[f"{n['x']}.weight"]
        self.w_dt, self.b_dt = tensors[f"{n['dt']}.weight"], tensors[f"{n['dt']}.bias"]
        self.a_log, self.skip = tensors[f"{n['a_log']}.weight"], tensors[f"{n['d']}.weight"]
        self.a2 = (-torch.exp(self.a_log.t().double()) * LOG2_E).float().contiguous()
        self.w_out = tensors[f"{n['o']}.weight"]

    def named_weights(self) -> Dict[str, torch.Tensor]:
        n = self.names
        return {f"{n['in']}.weight": self.w_in, f"{n['x']}.weight": self.w_x, f"{n['dt']}.weight": self.w_dt,
                f"{n['dt']}.bias": self.b_dt, f"{n['a_log']}.weight": self.a_log, f"{n['d']}.weight": self.skip,
                f"{n['o']}.weight": self.w_out}

    def forward(self, x: torch.Tensor, step: StepContext, slot: LayerSlot):
        from ..ops.linear_attention import plan_chunks
        from ..ops.selective_scan import CHUNKED_FROM, selective_scan

        if slot.state is None:
            raise RuntimeError("a state-space mixer needs a state slot")
        both = linear(x, self.w_in)                                     # [N, x | z] in the run dtype
        u = self.conv.forward(both[:, :self.inner], step, slot.of(self.names["conv"]))
        low = linear(u, self.w_x, out_dtype=torch.float32)              # [N, dt | B | C]
        dt = linear(low[:, :self.rank].to(self.dtype).contiguous(), self.w_dt, out_dtype=torch.float32)
        plan = None
        if step.max_q_len >= CHUNKED_FROM and len(step.cu_q_host) == step.num_reqs + 1:
            plan = step.derived.get("la_chunks")
            if plan is None:
                plan = step.derived["la_chunks"] = plan_chunks(step.cu_q_host, self.device)
        y = selective_scan(u, dt, self.b_dt, self.a2, low, self.rank, self.rank + self.states, self.skip,
                           both[:, self.inner:], slot.state, step.cu_q, step.req_slots, plan)
        return linear_into(step.residual, y, self.w_out)


class StateSpaceDual(Mixer):
    """A state space with one decay per head and token: ``[z; x; B; C; dt] = Win h``; ``x``, ``B`` and ``C`` pass a causal
    convolution per channel with a bias and silu; ``t = softplus(dt + b)``; per head ``S <- exp(-exp(A_log) t) S + t B x^T``,
    ``y = S^T C + D x``, heads sharing B and C by groups; then ``y silu(z)``, divided in ``norm_groups`` equal parts by each
    part's root mean square, times a weight, and ``Wo``.

    params: ``hidden_size``, ``num_heads``, ``value_dim``, ``state_size``, ``groups``, ``norm_groups``, ``conv_taps``,
    ``eps``, ``names`` (local names of the tensors' owners: ``in``, ``conv``, ``dt_bias``, ``a_log``, ``d``, ``norm``, ``o``;
    default these).  The projections and what the convolution gives are in the run dtype; ``dt`` from its projection on,
    decays, the state (float32 ``[heads, state_size, value_dim]`` per request), outputs and the norm are float32.
    """

    graph_safe = True

    def __init__(self, params, dtype, device):
        super().__init__(dtype, device)
        self.hidden, self.heads, self.vdim = int(params["hidden_size"]), int(params["num_heads"]), int(params["value_dim"])
        self.states, self.groups = int(params["state_size"]), int(params["groups"])
        self.norm_groups, self.eps = int(params["norm_groups"]), float(params["eps"])
        self.inner = self.heads * self.vdim
        if self.heads % self.groups:
            raise ValueError(f"{self.heads} heads are not a multiple of {self.groups} groups")
        if self.inner % self.norm_groups:
            raise ValueError(f"{self.inner} channels do not divide into {self.norm_groups} equal parts")
        names = dict(params.get("names") or {})
        self.names = {k: names.get(k, k) for k in ("in", "conv", "dt_bias", "a_log", "d", "norm", "o")}
        self.conv_channels = self.inner + 2 * self.groups * self.states
        self.conv = ConvolvedInput(self.conv_channels, int(params["conv_taps"]), dtype, device)
        self.w_in: Optional[torch.Tensor] = None
        self.dt_bias: Optional[torch.Tensor] = None
        self.a_log: Optional[torch.Tensor] = None
        self.a_neg: Optional[torch.Tensor] = None       # float32 [heads]: -exp(a_log)
        self.skip: Optional[torch.Tensor] = None
        self.w_norm: Optional[torch.Tensor] = None
        self.w_out: Optional[torch.Tensor] = None

    def sub_parts(self) -> Dict[str, Part]:
        return {self.names["conv"]: self.conv}

    def state_need(self) -> StateNeed:
        return StateNeed((self.heads, self.states, self.vdim), torch.float32)

    def param_specs(self) -> Dict[str, ParamSpec]:
        n, h = self.names, self.heads
        return {f"{n['in']}.weight": ParamSpec((self.inner + self.conv_channels + h, self.hidden)),
                f"{n['dt_bias']}.weight": ParamSpec((h,), "vector"),
                f"{n['a_log']}.weight": ParamSpec((h,), "vector"),
                f"{n['d']}.weight": ParamSpec((h,), "vector", init="around_one"),
                f"{n['norm']}.weight": ParamSpec((self.inner,), "vector", init="around_one"),
                f"{n['o']}.weight": ParamSpec((self.hidden, self.inner))}

    def load(self, tensors):
        n = self.names
        self.w_in, self.w_out = tensors[f"{n['in']}.weight"], tensors[f"{n['o']}.weight"]
        self.dt_bias, self.a_log = tensors[f"{n['dt_bias']}.weight"], tensors[f"{n['a_log']}.weight"]
        self.a_neg = (-torch.exp(self.a_log.double())).float().contiguous()
        self.skip, self.w_norm = tensors[f"{n['d']}.weight"], tensors[f"{n['norm']}.weight"]

    def named_weights(self) -> Dict[str, torch.Tensor]:
        n = self.names
        return {f"{n['in']}.weight": self.w_in, f"{n['dt_bias']}.weight": self.dt_bias, f"{n['a_log']}.weight": self.a_log,
                f"{n['d']}.weight": self.skip, f"{n['norm']}.weight": self.w_norm, f"{n['o']}.weight": self.w_out}

    def forward(self, x: torch.Tensor, step: StepContext, slot: LayerSlot):
        from ..ops.gated import group_norm_gate
        from ..ops.head_scan import head_scan

        if slot.state is None:
            raise RuntimeError("a state-space mixer needs a state slot")
        c, gn = self.inner, self.groups * self.states
        main, raw, raw_at = split_projection(x, self.w_in, c + self.conv_channels)
        u = self.conv.forward(main[:, c:c + self.conv_channels], step, slot.of(self.names["conv"]))
        o = head_scan(u, c + gn, c, 0, self.heads, self.groups, self.states, self.vdim, raw, raw_at, self.dt_bias, self.a_neg,
                      slot.state, step.cu_q, step.req_slots, skip=self.skip, plan=chunk_plan(step, self.states, self.device))
        y = group_norm_gate(o, self.w_norm, c // self.norm_groups, self.eps, self.dtype, gate=main[:, :c], gate_act="silu",
                            gate_first=True)
        return linear_into(step.residual, y, self.w_out)


def split_projection(x: torch.Tensor, weight: torch.Tensor, main_rows: int):
    """``x @ weight.T`` whose columns from ``main_rows`` on are wanted unrounded: ``(main, raw, where raw's columns start)``.
    Few rows, or a float32 run: one product in float32; else the main columns in the run dtype and the others in
    float32 by a product of their own."""
    if weight.dtype == torch.float32 or x.shape[0] <= skinny.ONE_BLOCK_ROWS:
        both = linear(x, weight, out_dtype=torch.float32)
        return both, both, main_rows
    return linear(x, weight[:main_rows]), linear(x, weight[main_rows:], out_dtype=torch.float32), 0


def chunk_plan(step: StepContext, dim: int, device):
    """The step's runs in chunks, if it is scanned that way (the plan is the step's, shared by layers)."""
    from ..ops.head_scan import takes_chunks
    from ..ops.linear_attention import plan_chunks

    if not takes_chunks(dim, step.max_q_len) or len(step.cu_q_host) != step.num_reqs + 1:
        return None
    plan = step.derived.get("la_chunks")
    if plan is None:
        plan = step.derived["la_chunks"] = plan_chunks(step.cu_q_host, device)
    return plan


register_part("mixer", "selective_state_space", SelectiveStateSpace)
register_part("mixer", "state_space_dual", StateSpaceDual)
