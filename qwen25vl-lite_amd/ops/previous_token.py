"""Python entry points of what a token takes from the one before it (``csrc/previous_token.hip``)."""

from __future__ import annotations

import ctypes
from typing import Optional

import torch

from .kernels import _check, _dev, _fn, _need, _ptr, _stream, dtype_code

__all__ = ["bigram_gather", "token_mix"]

_c_int, _c_ptr, _c_ll = ctypes.c_int, ctypes.c_void_p, ctypes.c_longlong


def _runs(cu_q, req_slots, token_req, n: int) -> int:
    for t in (cu_q, req_slots, token_req):
        _need(t.dtype == torch.int32 and t.dim() == 1 and t.is_contiguous(), "cu_q, req_slots and token_req must be int32")
    r = req_slots.shape[0]
    _need(cu_q.shape[0] == r + 1 and token_req.shape[0] == n, "cu_q has one entry more than requests, token_req one per token")
    return r


def bigram_gather(ids: torch.Tensor, table: torch.Tensor, pairs: torch.Tensor, last_id: torch.Tensor, cu_q: torch.Tensor,
                  req_slots: torch.Tensor, token_req: torch.Tensor, mul_prev: int, mul_cur: int) -> torch.Tensor:
    """float32 ``[N, H]``: ``table[id]`` plus row ``(previous id * mul_prev + id * mul_cur) mod buckets`` of ``pairs``
    (``[buckets + 1, H]``; the last row for a sequence's first token).  ``last_id`` (int32 ``[slots, 1]``) holds every
    request's last id plus one, zero before its first token; the runs' last ids replace it."""
    _dev(ids, table, pairs, last_id, cu_q, req_slots, token_req)
    _need(ids.dtype == torch.int32 and ids.dim() == 1 and ids.is_contiguous(), "ids must be contiguous int32 [N]")
    _need(table.dim() == 2 and table.is_contiguous() and pairs.dim() == 2 and pairs.is_contiguous()
          and pairs.dtype == table.dtype and pairs.shape[1] == table.shape[1] and pairs.shape[0] >= 2,
          "the tables must be contiguous [V, H] and [buckets + 1, H] of one dtype")
    _need(last_id.dtype == torch.int32 and last_id.is_contiguous() and last_id.numel() == last_id.shape[0],
          "last_id must be int32, one per slot")
    n = ids.shape[0]
    r = _runs(cu_q, req_slots, token_req, n)
    v, h = table.shape
    out = torch.empty((n, h), dtype=torch.float32, device=table.device)
    fn = _fn("previous_token", "qvl_bigram_gather", [_c_ptr] * 8 + [_c_int] * 5 + [_c_ll, _c_ll, _c_int, _c_ptr])
    _check(fn(_ptr(ids), _ptr(table), _ptr(pairs), _ptr(last_id), _ptr(cu_q), _ptr(req_slots), _ptr(token_req), _ptr(out),
              n, r, h, v, pairs.shape[0] - 1, int(mul_prev), int(mul_cur), dtype_code(table.dtype), _stream()), "bigram_gather")
    return out


def token_mix(h: torch.Tensor, cu_q: torch.Tensor, req_slots: torch.Tensor, token_req: torch.Tensor, out_dtype: torch.dtype,
              *, shift: Optional[torch.Tensor] = None, prev: Optional[torch.Tensor] = None,
              mu: Optional[torch.Tensor] = None, prev_mixed: Optional[torch.Tensor] = None) -> torch.Tensor:
    """With ``h'`` the row of the token before in its sequence (zeros before the first): ``g = h + (h' - h) shift``
    (``shift`` float32 ``[W]``; None: ``g = h``); then, with ``mu`` (float32 ``[mixes, W]``), ``g + (g' - g) mu_m`` as
    ``[mixes, N, W]``, else ``g`` as ``[N, W]``, in ``out_dtype``.  ``prev`` and ``prev_mixed`` (float32 ``[slots, W]``)
    hold every request's last ``h`` and ``g`` (zeros for a new request); the runs' last ones replace them."""
    _dev(h, cu_q, req_slots, token_req, shift, prev, mu, prev_mixed)
    _need(h.dim() == 2 and h.is_contiguous() and h.dtype in (torch.float32, out_dtype),
          "h must be contiguous [N, W], float32 or of the output's dtype")
    n, w = h.shape
    r = _runs(cu_q, req_slots, token_req, n)
    _need(shift is not None or mu is not None, "a step towards the previous row, or mixes with it, are needed")
    for vec, state in ((shift, prev), (mu, prev_mixed)):
        _need(vec is None or (vec.dtype == torch.float32 and vec.is_contiguous() and vec.shape[-1] == w and state is not None
                              and state.dtype == torch.float32 and state.dim() == 2 and state.shape[1] == w
                              and state.is_contiguous()), "weights must be float32 rows of W with a float32 state [slots, W]")
    _need(shift is None or shift.dim() == 1, "the step towards the previous row has one weight per channel")
    _need(mu is None or mu.dim() == 2, "mu must be [mixes, W]")
    mixes = mu.shape[0] if mu is not None else 0
    out = torch.empty((mixes, n, w) if mixes else (n, w), dtype=out_dtype, device=h.device)
    fn = _fn("previous_token", "qvl_token_mix",
             [_c_ptr, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_ll, _c_int,
              _c_int, _c_int, _c_ptr])
    _check(fn(_ptr(h), dtype_code(h.dtype), _ptr(shift), _ptr(prev), _ptr(mu), mixes, _ptr(prev_mixed), _ptr(cu_q),
              _ptr(req_slots), _ptr(token_req), _ptr(out), dtype_code(out_dtype), n * w, n, r, w, _stream()), "token_mix")
    return out
