"""Python entry point of the recurrences with one decay per head and token (``csrc/head_scan.hip``, compiled per key
size): decayed outer products, plain or by the delta rule."""

from __future__ import annotations

import ctypes
from typing import Optional

import torch

from .kernels import _check, _dev, _fn, _need, _ptr, _stream, dtype_code
from .linear_attention import ChunkPlan

__all__ = ["head_scan", "takes_chunks", "MAX_KEY_SIZE", "CHUNKED_FROM"]

_c_int, _c_float, _c_ptr, _c_ll = ctypes.c_int, ctypes.c_float, ctypes.c_void_p, ctypes.c_longlong
MAX_KEY_SIZE = 512
MAX_CHUNKED_KEY_SIZE = 256
CHUNK = 64
CHUNKED_FROM = 40     # a step whose longest run has this many tokens or more is scanned in chunks side by side (one run of
                      # 7B-sized heads: 39 us token after token at 32 tokens, 41 in chunks up to 64; eight runs: 42 and 70)


def takes_chunks(dim: int, max_run: int) -> bool:
    """Whether a step with runs of up to ``max_run`` tokens is scanned in chunks (:func:`head_scan` with a plan)."""
    return max_run >= CHUNKED_FROM and dim <= MAX_CHUNKED_KEY_SIZE


def head_scan(x: torch.Tensor, q_off: int, k_off: int, v_off: int, num_heads: int, num_groups: int, dim: int, vdim: int,
              raw: torch.Tensor, step_off: int, step_bias: torch.Tensor, a_neg: torch.Tensor, state: torch.Tensor,
              cu_q: torch.Tensor, req_slots: torch.Tensor, *, beta_off: Optional[int] = None,
              unit_eps: Optional[float] = None, q_scale: float = 1.0, skip: Optional[torch.Tensor] = None,
              plan: Optional[ChunkPlan] = None) -> torch.Tensor:
    """Every request's tokens of the step through a recurrence per head with the decay ``a = exp(a_neg t)``,
    ``t = softplus(raw[step_off + h] + step_bias)``:

    * ``beta_off`` None: ``S <- a S + t k v^T``, ``o = S^T q``;
    * else the delta rule with ``beta = sigmoid(raw[beta_off + h])``: ``S <- a S``, ``u = beta (v - S^T k)``,
      ``S <- S + k u^T``, ``o = S^T q``.

    ``x [N, cols]`` (float32 or bfloat16, rows any distance apart) holds ``groups * dim`` query columns from ``q_off``,
    as many key columns from ``k_off`` and ``heads * vdim`` value columns from ``v_off``; head h reads group
    ``h // (heads / groups)``.  ``unit_eps``: queries and keys become ``x / sqrt(sum x^2 + unit_eps)`` first; queries
    are multiplied by ``q_scale``; ``skip`` float32 ``[heads]`` adds ``skip v`` to the output.  ``raw`` float32
    ``[N, cols]``; ``state`` float32 ``[slots, heads, dim, vdim]``, read and replaced in the requests' rows.  Returns
    float32 ``[N, heads * vdim]``.

    ``plan`` (:func:`~qwen25vl_lite_amd.ops.linear_attention.plan_chunks` of the step, chunks of 64): chunks side by
    side, the states carried between them."""
    _dev(x, raw, step_bias, a_neg, state, cu_q, req_slots, skip)
    h, g, d, v = int(num_heads), int(num_groups), int(dim), int(vdim)
    _need(1 <= d <= MAX_KEY_SIZE, f"key sizes up to {MAX_KEY_SIZE} are built")
    _need(g > 0 and h % g == 0, "the heads must be a multiple of the groups")
    _need(x.dim() == 2 and x.stride(1) == 1 and raw.dim() == 2 and raw.stride(1) == 1 and raw.dtype == torch.float32
          and raw.shape[0] == x.shape[0], "x [N, cols] and raw float32 [N, cols] with contiguous rows")
    n = x.shape[0]
    for off, width, t in ((q_off, g * d, x), (k_off, g * d, x), (v_off, h * v, x), (step_off, h, raw),
                          (step_off if beta_off is None else beta_off, h, raw)):
        _need(0 <= off and off + width <= t.shape[1], "columns outside x or raw")
    for t in (step_bias, a_neg, skip):
        _need(t is None or (t.dtype == torch.float32 and t.shape == (h,) and t.is_contiguous()),
              "step_bias, a_neg and skip must be float32 [heads]")
    _need(state.dtype == torch.float32 and state.dim() == 4 and tuple(state.shape[1:]) == (h, d, v)
          and state.is_contiguous(), "state must be contiguous float32 [slots, heads, dim, vdim]")
    for t in (cu_q, req_slots):
        _need(t.dtype == torch.int32 and t.dim() == 1 and t.is_contiguous(), "cu_q and req_slots must be int32")
    r = req_slots.shape[0]
    _need(cu_q.shape[0] == r + 1, "cu_q must have one more entry than there are requests")
    _need(unit_eps is None or unit_eps > 0, "the floor of a unit vector must be positive")
    out = torch.empty((n, h * v), dtype=torch.float32, device=x.device)
    defines = {"HS_DIM": d}
    common = [_c_ptr, _c_ll, _c_int, _c_int, _c_int, _c_ptr, _c_ll, _c_int, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_float,
              _c_float, _c_ptr]
    args = (_ptr(x), x.stride(0) if n > 1 else x.shape[1], int(q_off), int(k_off), int(v_off), _ptr(raw),
            raw.stride(0) if n > 1 else raw.shape[1], int(step_off), -1 if beta_off is None else int(beta_off),
            _ptr(step_bias), _ptr(a_neg), _ptr(skip), float(q_scale), -1.0 if unit_eps is None else float(unit_eps),
            _ptr(state))
    if plan is None:
        fn = _fn("head_scan", "qvl_head_scan", common + [_c_ptr] * 3 + [_c_int] * 6 + [_c_ptr], defines)
        _check(fn(*args, _ptr(cu_q), _ptr(req_slots), _ptr(out), r, h, g, d, v, dtype_code(x.dtype), _stream()), "head_scan")
        return out
    _need(d <= MAX_CHUNKED_KEY_SIZE and plan.chunk_len == CHUNK and plan.req_first.shape[0] == r + 1,
          "the chunk plan belongs to another step or size")
    floats = _fn("head_scan", "qvl_head_scan_scratch", [_c_int] * 5, defines)
    floats.restype = _c_ll
    scratch = torch.empty(int(floats(plan.chunks, h, g, v, int(beta_off is not None))), dtype=torch.float32, device=x.device)
    fn = _fn("head_scan", "qvl_head_scan_chunks", common + [_c_ptr] * 5 + [_c_int] * 7 + [_c_ptr], defines)
    _check(fn(*args, _ptr(plan.chunk_cu), _ptr(plan.req_first), _ptr(req_slots), _ptr(out), _ptr(scratch), plan.chunks, r,
              h, g, d, v, dtype_code(x.dtype), _stream()), "head_scan in chunks")
    return out
