"""A recurrence over outer products whose projections each read a mix of their own of the token with the one before
it, with a decay per token and key channel and a bonus for the current token.

``x_s = h + (h' - h) mu_s`` for s in r, k, v, g, w; ``r, k, v = Wr x_r, Wk x_k, Wv x_v`` (heads of ``dim``); decay
``a = exp(-exp(W2 tanh(W1 x_w) + w0))``; per head ``o_t = (S_(t-1) + diag(u) k_t v_t^T)^T r_t``, then
``S_t = diag(a_t) S_(t-1) + k_t v_t^T``; each head's ``o`` divided by its root mean square, the joined heads times a
weight, times ``silu(Wg x_g)``, then ``Wo``.
"""

from __future__ import annotations

from typing import Dict, Optional

import torch

from ..ops import gated
from ..ops.linear import linear, linear_into, linear_stack
from ..ops.linear_attention import CHUNKED_FROM, chunked_scan, decayed_scan, plan_chunks, scan_groups
from .base import LayerSlot, Mixer, ParamSpec, Part, StateNeed, StepContext, register_part
from .token_shift import TokenMixes

__all__ = ["TimeMix"]

DEFAULT_RANK = 64     # of the decay's projection where a checkpoint does not say


class TimeMix(Mixer):
    """params: ``hidden_size``, ``num_heads``, ``head_dim``, ``eps`` (of the heads' norm), ``decay_rank`` (what random
    weights draw; a checkpoint's own size is taken), ``names`` (local names of the tensors' owners: ``mu``, ``r``, ``k``,
    ``v``, ``g``, ``w1``, ``w2``, ``w0``, ``u``, ``norm``, ``o``; default these).

    Takes its input ``[N, hidden]`` and mixes it, or the mixes ``[5, N, hidden]`` made before.  The projections are in the
    run dtype; the decay from its logarithm's projection on, the state (float32 ``[heads, dim, dim]`` per request), the
    outputs and their norm are float32.
    """

    graph_safe = True
    MIXES = ("r", "k", "v", "g", "w")

    def __init__(self, params, dtype, device):
        super().__init__(dtype, device)
        self.hidden, self.heads, self.dim = int(params["hidden_size"]), int(params["num_heads"]), int(params["head_dim"])
        self.eps = float(params["eps"])
        self.rank = int(params.get("decay_rank") or DEFAULT_RANK)
        names = dict(params.get("names") or {})
        self.names = {k: names.get(k, k) for k in ("mu", "r", "k", "v", "g", "w1", "w2", "w0", "u", "norm", "o")}
        self.token_mixes = TokenMixes({"channels": self.hidden, "names": self.MIXES}, dtype, device)
        self.w_in: Optional[torch.Tensor] = None        # [4, heads dim, hidden]: r, k, v, g
        self.w1: Optional[torch.Tensor] = None
        self.w2: Optional[torch.Tensor] = None
        self.w0: Optional[torch.Tensor] = None
        self.bonus: Optional[torch.Tensor] = None
        self.w_norm: Optional[torch.Tensor] = None
        self.w_out: Optional[torch.Tensor] = None

    def sub_parts(self) -> Dict[str, Part]:
        return {self.names["mu"]: self.token_mixes}

    def state_need(self) -> StateNeed:
        return StateNeed((self.heads, self.dim, self.dim), torch.float32)

    def param_specs(self) -> Dict[str, ParamSpec]:
        n, hd = self.names, self.heads * self.dim
        specs = {f"{n[s]}.weight": ParamSpec((hd, self.hidden)) for s in "rkvg"}
        specs.update({f"{n['w1']}.weight": ParamSpec((self.rank, self.hidden), free=(0,)),
                      f"{n['w2']}.weight": ParamSpec((hd, self.rank), free=(1,)),
                      f"{n['w0']}.weight": ParamSpec((hd,), "vector"),
                      f"{n['u']}.weight": ParamSpec((self.heads, self.dim), "vector"),
                      f"{n['norm']}.weight": ParamSpec((hd,), "vector", init="around_one"),
                      f"{n['o']}.weight": ParamSpec((self.hidden, hd))})
        return specs

    def load(self, tensors):
        n = self.names
        self.w_in = torch.stack([tensors[f"{n[s]}.weight"] for s in "rkvg"]).contiguous()
        self.w1, self.w2, self.w0 = tensors[f"{n['w1']}.weight"], tensors[f"{n['w2']}.weight"], tensors[f"{n['w0']}.weight"]
        if self.w1.shape[0] != self.w2.shape[1]:
            raise ValueError(f"the decay's projections do not meet: {tuple(self.w1.shape)} and {tuple(self.w2.shape)}")
        self.rank = self.w1.shape[0]
        self.bonus = tensors[f"{n['u']}.weight"].reshape(-1).contiguous()
        self.w_norm, self.w_out = tensors[f"{n['norm']}.weight"], tensors[f"{n['o']}.weight"]

    def named_weights(self) -> Dict[str, torch.Tensor]:
        n = self.names
        out = {f"{n[s]}.weight": self.w_in[i] for i, s in enumerate("rkvg")}
        out.update({f"{n['w1']}.weight": self.w1, f"{n['w2']}.weight": self.w2, f"{n['w0']}.weight": self.w0,
                    f"{n['u']}.weight": self.bonus.view(self.heads, self.dim), f"{n['norm']}.weight": self.w_norm,
                    f"{n['o']}.weight": self.w_out})
        return out

    def forward(self, x: torch.Tensor, step: StepContext, slot: LayerSlot):
        if slot.state is None:
            raise RuntimeError("a recurrence over outer products needs a state slot")
        if x.dim() == 2:
            x = self.token_mixes.forward(x, step, slot.of(self.names["mu"]))
        hd = self.heads * self.dim
        proj = linear_stack(x[:4], self.w_in)                               # [r | k | v | g, N, heads dim] in the run dtype
        low = gated.tanh_to(linear(x[4], self.w1, out_dtype=torch.float32), self.dtype)
        z = linear(low, self.w2, out_dtype=torch.float32)
        how = dict(z=z, z_bias=self.w0, exp_decay=True, bonus=self.bonus)
        if step.max_q_len >= CHUNKED_FROM and len(step.cu_q_host) == step.num_reqs + 1:
            plan = step.derived.get("la_chunks")
            if plan is None:
                plan = step.derived["la_chunks"] = plan_chunks(step.cu_q_host, self.device)
            o = chunked_scan(proj, 0, hd, 2 * hd, self.heads, self.dim, self.dim, slot.state, plan, step.req_slots, **how)
        else:
            o = decayed_scan(proj, 0, hd, 2 * hd, self.heads, self.dim, self.dim, slot.state, step.cu_q, step.req_slots,
                             groups=scan_groups(step.num_reqs, step.max_q_len, self.heads, self.dim, self.dim, self.device),
                             **how)
        y = gated.group_norm_gate(o, self.w_norm, self.dim, self.eps, self.dtype, gate=proj[3], gate_act="silu")
        return linear_into(step.residual, y, self.w_out)


register_part("mixer", "time_mix", TimeMix)
