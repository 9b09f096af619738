"""Python entry point of a residual stream of several copies (``csrc/hyper.hip``, compiled per number of copies)."""

from __future__ import annotations

import ctypes
from typing import NamedTuple, Optional, Tuple, Union

import torch

from ..parts.base import NormedMean
from .kernels import _check, _dev, _fn, _need, _ptr, _stream, dtype_code

__all__ = ["join_norm", "SingleTokens", "MAX_COPIES"]

_c_int, _c_float, _c_ptr, _c_ll = ctypes.c_int, ctypes.c_float, ctypes.c_void_p, ctypes.c_longlong
MAX_COPIES = 32


class SingleTokens(NamedTuple):
    """What :func:`join_norm` does behind the norm in a step of single tokens, one per request: the step towards the
    request's previous row (``shift [W]`` with its state ``prev [slots, W]``) and the mixes of the result with the
    previous one (``mu [mixes, W]`` with ``prev_mixed``); either may be None.  ``slots`` int32 ``[N]``: each token's
    state row.  All vectors and states float32."""

    slots: torch.Tensor
    shift: Optional[torch.Tensor] = None
    prev: Optional[torch.Tensor] = None
    mu: Optional[torch.Tensor] = None
    prev_mixed: Optional[torch.Tensor] = None


def _addend(y: torch.Tensor, n: int, width: int) -> Tuple[int, int]:
    """``(dtype code, slabs)`` of an addend ``[N, W]`` (float32 or bfloat16) or float32 slabs ``[slabs, N, W]``."""
    if y.dim() == 3:
        _need(y.dtype == torch.float32 and tuple(y.shape[1:]) == (n, width) and y.is_contiguous(),
              "slabs of an addend must be contiguous float32 [slabs, N, W]")
        return 0, y.shape[0]
    _need(tuple(y.shape) == (n, width) and y.is_contiguous(), "an addend must be contiguous [N, W]")
    return dtype_code(y.dtype), 1


def join_norm(h: torch.Tensor, copies: Optional[torch.Tensor], join: Optional[Tuple[torch.Tensor, torch.Tensor]],
              pending: Union[None, torch.Tensor, NormedMean], read: Optional[torch.Tensor], weight: torch.Tensor,
              groups: int, eps: float, out_dtype: torch.dtype, *, num_copies: int, rows: Optional[torch.Tensor] = None,
              single: Optional[SingleTokens] = None) -> Tuple[torch.Tensor, Optional[torch.Tensor]]:
    """``(normed rows, copies)``.  The copies are ``copies`` (float32 ``[N, S, W]``), or all equal to ``h`` (float32
    ``[N, W]``) while ``copies`` is None.  With ``join = (mix [S, S], out [S])`` they first become
    ``sum_s mix[s, t] x_s + out[t] y``, ``y`` being ``pending`` (written in place, or to a new tensor if ``copies`` is
    None; not at all with ``rows``).  What is normed is ``sum_t read[t] x_t`` (``read`` None: the sum of the copies), in
    ``groups`` equal parts of the row with a root mean square each, times ``weight``; with ``rows`` (int32) for those
    rows only; with ``single`` it is taken on as :class:`SingleTokens` says and comes as ``[N, W]`` or ``[mixes, N, W]``."""
    s = int(num_copies)
    n, width = h.shape
    _need(1 <= s <= MAX_COPIES, f"1 to {MAX_COPIES} copies are built")
    _need(h.dtype == torch.float32 and h.is_contiguous(), "h must be contiguous float32 [N, W]")
    _need(copies is None or (copies.dtype == torch.float32 and tuple(copies.shape) == (n, s, width) and copies.is_contiguous()),
          "copies must be contiguous float32 [N, S, W]")
    _need(weight.dtype == torch.float32 and weight.shape == (width,) and weight.is_contiguous() and groups > 0
          and width % groups == 0, "the norm's weight must be float32 [W], W in whole groups")
    _need((join is None) == (pending is None), "what is pending joins the copies by a mix and shares, and nothing else does")
    for t, shape in (((read, (s,)),) if join is None else ((read, (s,)), (join[0], (s, s)), (join[1], (s,)))):
        _need(t is None or (t.dtype == torch.float32 and tuple(t.shape) == shape and t.is_contiguous()),
              "a layer's mix, shares and reading weights must be float32 [S, S], [S] and [S]")
    mix, shares = join if join is not None else (None, None)
    y1 = y2 = g1 = g2 = None
    eps_pair, factor, dt1, dt2, slabs1, slabs2 = 0.0, 1.0, 0, 0, 1, 1
    if isinstance(pending, NormedMean):
        y1, y2, g1, g2 = pending.first, pending.second, pending.gain_first, pending.gain_second
        eps_pair, factor = float(pending.eps), float(pending.factor)
        dt1, slabs1 = _addend(y1, n, width)
        dt2, slabs2 = _addend(y2, n, width)
        for g in (g1, g2):
            _need(g.dtype == torch.float32 and g.shape == (width,) and g.is_contiguous(), "gains must be float32 [W]")
    elif pending is not None:
        y1 = pending
        dt1, slabs1 = _addend(y1, n, width)
    m = n
    if rows is not None:
        _need(rows.dtype == torch.int32 and rows.dim() == 1 and rows.is_contiguous(), "rows must be int32 [M]")
        m = rows.shape[0]
    shift = prev = mu = prev_mixed = slots = None
    mixes = 0
    shape = (m, width)
    if single is not None:
        slots, shift, prev, mu, prev_mixed = single
        _need(rows is None and slots.dtype == torch.int32 and slots.shape == (n,) and slots.is_contiguous(),
              "slots must be int32 [N]")
        _need(shift is not None or mu is not None, "a step towards the previous row, or mixes with it, are needed")
        for vec, state in ((shift, prev), (mu, prev_mixed)):
            _need(vec is None or (vec.dtype == torch.float32 and vec.is_contiguous() and vec.shape[-1] == width
                                  and state is not None and state.dtype == torch.float32 and state.dim() == 2
                                  and state.shape[1] == width and state.is_contiguous()),
                  "weights must be float32 rows of W with a float32 state [slots, W]")
        _need(shift is None or shift.dim() == 1, "the step towards the previous row has one weight per channel")
        if mu is not None:
            _need(mu.dim() == 2, "mu must be [mixes, W]")
            mixes = mu.shape[0]
            shape = (mixes, m, width)
    _dev(h, copies, mix, shares, y1, y2, g1, g2, read, weight, rows, slots, shift, prev, mu, prev_mixed)
    new = copies
    if join is not None and copies is None and rows is None:
        new = torch.empty((n, s, width), dtype=torch.float32, device=h.device)
    src = h if copies is None else copies
    out = torch.empty(shape, dtype=out_dtype, device=h.device)
    fn = _fn("hyper", "qvl_hyper_join_norm",
             [_c_ptr, _c_ll, _c_ll, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_int, _c_ptr, _c_int, _c_int, _c_ll, _c_ptr,
              _c_ptr, _c_float, _c_float, _c_ptr, _c_ptr, _c_int, _c_float, _c_ptr, _c_int, _c_ptr, _c_int, _c_int, _c_ptr,
              _c_ptr, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_ll, _c_ptr], {"HC_S": s})
    _check(fn(_ptr(src), width if copies is None else s * width, 0 if copies is None else width,
              _ptr(new) if join is not None and rows is None else None, _ptr(mix), _ptr(shares), _ptr(y1), dt1, slabs1,
              _ptr(y2), dt2, slabs2, n * width, _ptr(g1), _ptr(g2), eps_pair, factor, _ptr(read), _ptr(weight),
              int(groups), float(eps), _ptr(out), dtype_code(out_dtype), _ptr(rows), m, width, _ptr(shift), _ptr(prev),
              _ptr(mu), mixes, _ptr(prev_mixed), _ptr(slots), m * width, _stream()), "hyper join and norm")
    return out, new
