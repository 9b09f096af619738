"""Choice of the attention kernel for a step."""

from __future__ import annotations

from typing import Optional

import torch

from . import kernels

__all__ = ["paged_attention"]


def paged_attention(q: torch.Tensor, k_cache: torch.Tensor, v_cache: torch.Tensor, block_table: torch.Tensor,
                    step, num_q_heads: int, window: Optional[int], scale: float, keep_first: int = 0,
                    sinks: Optional[torch.Tensor] = None, chunk: Optional[int] = None,
                    turn: Optional[torch.Tensor] = None, turn_pairs: bool = False,
                    gate: Optional[torch.Tensor] = None) -> torch.Tensor:
    """Attention of the step's tokens over their requests' pages.

    bfloat16 with a head size in steps of 16 runs on the matrix cores, with ``sinks`` (float32 ``[heads]``: one more term
    ``exp(sink)`` in each head's softmax denominator) or without;
    bfloat16 with a window that keeps the first keys, values of another width than the keys, sinks with a head size in
    steps of 8, chunks of positions
    that see only themselves (``chunk``) or values turned by their positions (``turn``: the angles by which each
    token's output is turned back) has a matrix-core kernel of its own; everything else (float32, other head sizes) runs through the
    float32-arithmetic kernel.  ``gate`` (float32 ``[N, heads]``): each head's output times the sigmoid of its number, in
    the first of these kernels' last lines or by a kernel behind the others.
    """
    def gated(out):
        if gate is None:
            return out
        from .gated import head_gate_
        return head_gate_(out, gate, num_q_heads)

    plain = not (window and keep_first) and v_cache.shape[2] == k_cache.shape[3] and chunk is None and turn is None
    if q.dtype == torch.bfloat16 and plain:
        from . import attention_mfma
        out = attention_mfma.try_attention(q, k_cache, v_cache, block_table, step, num_q_heads, window, scale, sinks=sinks,
                                           gate=gate)
        if out is not None:
            return out
    if q.dtype == torch.bfloat16 and (not plain or sinks is not None):
        from . import attention_window
        out = attention_window.try_attention(q, k_cache, v_cache, block_table, step, num_q_heads, window, keep_first,
                                             scale, sinks=sinks, chunk=chunk, turn=turn, turn_pairs=turn_pairs)
        if out is not None:
            return gated(out)
    return gated(kernels.paged_attention_generic(q, k_cache, v_cache, block_table, step.token_req, step.token_seqpos,
                                                 num_q_heads, window, scale, keep_first=keep_first, sinks=sinks, chunk=chunk,
                                                 turn=turn, turn_pairs=turn_pairs))
