"""Python entry points of ``csrc/sum_norm.hip``: a residual sum joined by one or two terms with the layer norm behind the
sum, and rows of a table gated by an activation."""

from __future__ import annotations

import ctypes
from typing import Optional, Sequence

import torch

from ..parts.base import SumTerm
from .kernels import _check, _dev, _fn, _need, _ptr, _stream, dtype_code

__all__ = ["sum_norm_", "gelu_rows"]

_c_int, _c_float, _c_ptr, _c_ll = ctypes.c_int, ctypes.c_float, ctypes.c_void_p, ctypes.c_longlong


def _slabs(y: torch.Tensor, n: int, width: int) -> int:
    _need(y.is_contiguous() and tuple(y.shape[-2:]) == (n, width) and y.dtype in (torch.float32, torch.bfloat16)
          and (y.dim() == 2 or (y.dim() == 3 and y.dtype == torch.float32)),
          "a term must be contiguous [N, H], float32 or bfloat16, or float32 slabs [slabs, N, H]")
    return y.shape[0] if y.dim() == 3 else 1


def sum_norm_(h: torch.Tensor, alpha: float, terms: Sequence[SumTerm], weight: Optional[torch.Tensor] = None,
              bias: Optional[torch.Tensor] = None, eps: float = 0.0,
              copy_dtype: Optional[torch.dtype] = None) -> Optional[torch.Tensor]:
    """``h = norm(alpha h + sum of the terms)`` in float32, in place; ``norm`` is the layer norm with ``weight`` and
    ``bias``, or nothing without them.  A term contributes ``factor * value``, or with a gain
    ``factor * value / sqrt(mean(value^2) + eps) * gain``.  With ``copy_dtype`` the new rows are also returned in it."""
    _need(1 <= len(terms) <= 2, "one or two terms join the sum")
    _dev(h, weight, bias, *(t.value for t in terms), *(t.gain for t in terms))
    _need(h.dtype == torch.float32 and h.dim() == 2 and h.is_contiguous(), "h must be contiguous float32 [N, H]")
    n, width = h.shape
    _need((weight is None) == (bias is None), "the norm's weight and bias come together")
    for v in (weight, bias, *(t.gain for t in terms)):
        _need(v is None or (v.dtype == torch.float32 and v.shape == (width,) and v.is_contiguous()),
              "weights, biases and gains must be float32 [H]")
    out = None if copy_dtype is None else torch.empty((n, width), dtype=copy_dtype, device=h.device)
    each = []
    for t in (*terms, None)[:2]:
        each += ([None, 0, 1, None, 0.0, 0.0] if t is None else
                 [_ptr(t.value), dtype_code(t.value.dtype), _slabs(t.value, n, width), _ptr(t.gain), float(t.eps),
                  float(t.factor)])
    term = [_c_ptr, _c_int, _c_int, _c_ptr, _c_float, _c_float]
    fn = _fn("sum_norm", "qvl_sum_norm", [_c_ptr, _c_float, *term, *term, _c_ptr, _c_ptr, _c_float, _c_ptr, _c_int, _c_int,
                                          _c_int, _c_ptr])
    _check(fn(_ptr(h), float(alpha), *each, _ptr(weight), _ptr(bias), float(eps), _ptr(out),
              0 if copy_dtype is None else dtype_code(copy_dtype), n, width, _stream()), "sum_norm")
    return out


def gelu_rows(z: torch.Tensor, table: torch.Tensor, first: int, ids: torch.Tensor) -> torch.Tensor:
    """``gelu(z) * table[ids, first : first + C]`` for ``z [N, C]`` (gelu in its tanh form), in the table's dtype."""
    _dev(z, table, ids)
    _need(z.dim() == 2 and z.stride(1) == 1 and table.dim() == 2 and table.stride(1) == 1, "z [N, C] and a table of rows")
    n, c = z.shape
    _need(z.dtype in (torch.float32, table.dtype), "z is float32 or of the table's dtype")
    _need(0 <= first and first + c <= table.shape[1], "columns outside the table")
    _need(ids.dtype == torch.int32 and ids.shape == (n,) and ids.is_contiguous(), "ids must be int32 [N]")
    out = torch.empty((n, c), dtype=table.dtype, device=z.device)
    fn = _fn("sum_norm", "qvl_gelu_rows", [_c_ptr, _c_int, _c_ll, _c_ptr, _c_int, _c_ll, _c_int, _c_ptr, _c_ptr, _c_int,
                                           _c_int, _c_ptr])
    _check(fn(_ptr(z), dtype_code(z.dtype), z.stride(0) if n > 1 else c, _ptr(table), dtype_code(table.dtype),
              table.stride(0) if table.shape[0] > 1 else table.shape[1], int(first), _ptr(ids), _ptr(out), n, c, _stream()),
           "gelu_rows")
    return out
