"""Python entry point of the selective scan (``csrc/selective_scan.hip``, compiled per state size)."""

from __future__ import annotations

import ctypes
from typing import Optional

import torch

from .kernels import _check, _dev, _fn, _need, _ptr, _stream, dtype_code
from .linear_attention import ChunkPlan

__all__ = ["selective_scan", "MAX_STATE", "CHUNKED_FROM", "LOG2_E"]

_c_int, _c_ptr, _c_ll = ctypes.c_int, ctypes.c_void_p, ctypes.c_longlong
MAX_STATE = 256
CHUNKED_FROM = 128    # a step whose longest run has this many tokens or more is scanned in chunks side by side
LOG2_E = 1.4426950408889634
WHOLE, LAST_STATE, FROM_STATE = 0, 1, 2


def selective_scan(x: torch.Tensor, dt: torch.Tensor, dt_bias: torch.Tensor, a2: torch.Tensor, bc: torch.Tensor, b_off: int,
                   c_off: int, d: torch.Tensor, z: torch.Tensor, state: torch.Tensor, cu_q: torch.Tensor,
                   req_slots: torch.Tensor, plan: Optional[ChunkPlan] = None) -> torch.Tensor:
    """Every request's tokens of the step through ``S[n, c] <- exp(t A[n, c]) S[n, c] + t x_c B_n`` with
    ``t = softplus(dt + dt_bias)`` per token and channel, ``y_c = sum_n S[n, c] C_n + d_c x_c``; returns ``y silu(z)``
    as ``[N, C]`` in ``x``'s dtype.

    ``x [N, C]`` and ``z`` (``[N, C]``, rows any distance apart) are float32 or bfloat16; ``dt`` float32 ``[N, C]``;
    ``a2`` float32 ``[states, C]``, ``A log2(e)``; ``bc`` float32 ``[N, cols]`` with B's ``states`` columns from
    ``b_off`` and C's from ``c_off``; ``state`` float32 ``[slots, states, C]``, read and replaced in the requests' rows.
    ``plan`` (:func:`~qwen25vl_lite_amd.ops.linear_attention.plan_chunks` of the step): long runs are cut into chunks
    that are scanned side by side, the states carried between them."""
    _dev(x, dt, dt_bias, a2, bc, d, z, state, cu_q, req_slots)
    n, c = x.shape
    states = a2.shape[0]
    _need(1 <= states <= MAX_STATE, f"state sizes up to {MAX_STATE} are built")
    _need(x.is_contiguous() and z.shape == (n, c) and z.dtype == x.dtype and z.stride(1) == 1, "x and z must be [N, C] of one dtype")
    for t, shape in ((dt, (n, c)), (dt_bias, (c,)), (a2, (states, c)), (d, (c,))):
        _need(t.dtype == torch.float32 and tuple(t.shape) == shape and t.is_contiguous(),
              "dt, dt_bias, a2 and d must be contiguous float32 [N, C], [C], [states, C] and [C]")
    _need(bc.dtype == torch.float32 and bc.dim() == 2 and bc.shape[0] == n and bc.stride(1) == 1
          and 0 <= b_off and b_off + states <= bc.shape[1] and 0 <= c_off and c_off + states <= bc.shape[1],
          "bc must be float32 [N, cols] with B's and C's columns")
    _need(state.dtype == torch.float32 and state.dim() == 3 and tuple(state.shape[1:]) == (states, c) and state.is_contiguous(),
          "state must be contiguous float32 [slots, states, C]")
    for t in (cu_q, req_slots):
        _need(t.dtype == torch.int32 and t.dim() == 1 and t.is_contiguous(), "cu_q and req_slots must be int32")
    r = req_slots.shape[0]
    _need(cu_q.shape[0] == r + 1, "cu_q must have one more entry than there are requests")
    out = torch.empty_like(x)
    defines = {"SSM_STATE": states}
    fn = _fn("selective_scan", "qvl_selective_scan",
             [_c_int, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ll, _c_int, _c_int, _c_ptr, _c_ptr, _c_ll, _c_ptr, _c_ptr,
              _c_ptr, _c_ptr, _c_ptr, _c_int, _c_int, _c_int, _c_int, _c_ptr], defines)

    def scan(mode, target, sums, bounds, row_of, runs):
        _check(fn(mode, _ptr(x), _ptr(dt), _ptr(dt_bias), _ptr(a2), _ptr(bc), bc.stride(0) if n > 1 else bc.shape[1],
                  int(b_off), int(c_off), _ptr(d), _ptr(z), z.stride(0) if n > 1 else c, _ptr(out), _ptr(target),
                  _ptr(sums), _ptr(bounds), _ptr(row_of), runs, c, states, dtype_code(x.dtype), _stream()), "selective_scan")

    if plan is None:
        scan(WHOLE, state, None, cu_q, req_slots, r)
        return out
    _need(plan.req_first.shape[0] == r + 1, "the chunk plan belongs to another step")
    scratch = torch.empty((plan.chunks, states, c), dtype=torch.float32, device=x.device)
    sums = torch.empty((plan.chunks, c), dtype=torch.float32, device=x.device)
    scan(LAST_STATE, scratch, sums, plan.chunk_cu, None, plan.chunks)
    carry = _fn("selective_scan", "qvl_selective_carry", [_c_ptr] * 6 + [_c_int, _c_int, _c_int, _c_ptr], defines)
    _check(carry(_ptr(scratch), _ptr(sums), _ptr(a2), _ptr(state), _ptr(plan.req_first), _ptr(req_slots), r, c, states,
                 _stream()), "selective carry")
    scan(FROM_STATE, scratch, None, plan.chunk_cu, None, plan.chunks)
    return out
