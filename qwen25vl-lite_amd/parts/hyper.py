"""A layer over several copies of the residual sum that every sublayer mixes anew (hyper-connections).

With copies ``x_1 .. x_s`` (all equal to the embedding's output at the start) a sublayer reads
``u = sum_s in[s] x_s``, and with its result ``y`` copy t becomes ``sum_s mix[s, t] x_s + out[t] y``, the ``x_s`` being
the copies as the sublayer found them.  What a sublayer gave stays pending, with the weights by which it joins, until the kernel
of the next norm in line joins it, forms the next sublayer's ``u`` and norms it in one pass over the copies.
"""

from __future__ import annotations

from typing import Dict, Optional, Tuple

import torch

from .base import Block, LayerSlot, Norm, ParamSpec, Part, ResidualStream, StepContext, build_part, register_part

__all__ = ["CopiesConnection", "CopiesNorm", "CopiesBlock"]


class CopiesConnection(Part):
    """The weights of one sublayer's connection: ``in [s]``, ``out [s]`` and ``mix [s, s]`` (from, to)."""

    graph_safe = True

    def __init__(self, copies: int, dtype, device):
        super().__init__(dtype, device)
        self.copies = int(copies)
        self.w_in: Optional[torch.Tensor] = None
        self.w_out: Optional[torch.Tensor] = None
        self.mix: Optional[torch.Tensor] = None

    def param_specs(self) -> Dict[str, ParamSpec]:
        s = self.copies
        return {"in.weight": ParamSpec((s,), "vector", init="around_one"),
                "out.weight": ParamSpec((s,), "vector", init="around_one"),
                "mix.weight": ParamSpec((s, s), "vector", init="identity")}

    def load(self, tensors):
        self.w_in, self.w_out, self.mix = tensors["in.weight"], tensors["out.weight"], tensors["mix.weight"]

    def named_weights(self) -> Dict[str, torch.Tensor]:
        return {"in.weight": self.w_in, "out.weight": self.w_out, "mix.weight": self.mix}

    @property
    def join(self) -> Tuple[torch.Tensor, torch.Tensor]:
        return self.mix, self.w_out


class CopiesNorm(Norm):
    """The norm of a stream of copies: RMS norm in ``groups`` consecutive equal parts of the row, each divided by its
    own root mean square (``eps`` inside the root), times one weight over the whole row.

    params: ``size``, ``eps``, ``copies``, ``groups`` (default 1: one root mean square for the row).
    """

    graph_safe = True

    def __init__(self, params, dtype, device):
        super().__init__(dtype, device)
        self.size, self.copies = int(params["size"]), int(params["copies"])
        self.groups = int(params.get("groups", 1))
        self.eps = float(params["eps"])
        if self.groups < 1 or self.size % self.groups:
            raise ValueError(f"a row of {self.size} does not divide into {self.groups} equal parts")
        self.weight: Optional[torch.Tensor] = None

    def param_specs(self) -> Dict[str, ParamSpec]:
        return {"weight": ParamSpec((self.size,), "vector", init="around_one")}

    def load(self, tensors):
        self.weight = tensors["weight"]

    def named_weights(self) -> Dict[str, torch.Tensor]:
        return {"weight": self.weight}

    def forward(self, stream: ResidualStream, rows: Optional[torch.Tensor] = None, lazy: bool = False,
                read: Optional[torch.Tensor] = None, out_dtype: Optional[torch.dtype] = None, single=None):
        """Join what is pending to the copies and norm ``sum_t read[t] x_t`` (``read`` None: the sum of the copies, what
        the model's last norm reads).  ``single``: the steps of :class:`~qwen25vl_lite_amd.ops.hyper.SingleTokens`
        behind the norm."""
        from ..ops.hyper import join_norm
        if stream.pending_norm is not None or stream.row_addend is not None:
            raise RuntimeError("a stream of copies takes plain addends and normed means only")
        if stream.pending is not None and stream.pending_join is None:
            raise RuntimeError("an addend is pending that says nothing of how it joins the copies")
        out, copies = join_norm(stream.h, stream.copies, stream.pending_join, stream.pending, read, self.weight,
                                self.groups, self.eps, out_dtype or self.dtype, num_copies=self.copies, rows=rows,
                                single=single)
        if rows is None:
            stream.copies, stream.pending, stream.pending_join = copies, None, None
        return out


class CopiesBlock(Block):
    """A layer of pre-normed sublayers over a stream of copies; a filter may stand between the first norm and the mixer.

    params: ``copies``, ``norm1``, ``mixer``, ``norm2``, ``ffn`` (:class:`PartSpec` each; the norms of kind
    ``copies``; ``ffn`` None for a layer without a feed-forward, whose ``norm2`` is then not built), ``filter`` (a
    :class:`PartSpec` of kind ``token_shift``, or None) and ``names``, the checkpoint sub-name of each part and of
    the two connections (``join1``, ``join2``).

    In a step of single tokens the step towards the previous token and the mixer's own mixes with it, if it has
    any, are made by the norm's kernel; else by one kernel behind it, from the norm's rows in float32.
    """

    graph_safe = True

    def __init__(self, params, dtype, device):
        super().__init__(dtype, device)
        self.names: Dict[str, str] = dict(params["names"])
        copies = int(params["copies"])
        self.norm1 = build_part("norm", params["norm1"], dtype, device)
        self.join1 = CopiesConnection(copies, dtype, device)
        self.mixer = build_part("mixer", params["mixer"], dtype, device)
        self.filter: Optional[Part] = None
        if params.get("filter") is not None:
            self.filter = build_part("filter", params["filter"], dtype, device)
        self.ffn: Optional[Part] = None
        if params.get("ffn") is not None:
            self.norm2 = build_part("norm", params["norm2"], dtype, device)
            self.join2 = CopiesConnection(copies, dtype, device)
            self.ffn = build_part("ffn", params["ffn"], dtype, device)
        for norm in (self.norm1, getattr(self, "norm2", None)):
            if norm is not None and not (isinstance(norm, CopiesNorm) and norm.copies == copies):
                raise ValueError("the norms of a layer over copies are of kind 'copies' and have as many")
        from .token_shift import TokenShift
        if self.filter is not None and not isinstance(self.filter, TokenShift):
            raise ValueError("the filter of a layer over copies is a step towards the previous token")

    def sub_parts(self) -> Dict[str, Part]:
        parts = {self.names["mixer"]: self.mixer, self.names["norm1"]: self.norm1, self.names["join1"]: self.join1}
        if self.filter is not None:
            parts[self.names["filter"]] = self.filter
        if self.ffn is not None:
            parts.update({self.names["ffn"]: self.ffn, self.names["norm2"]: self.norm2, self.names["join2"]: self.join2})
        return parts

    def _mixer_input(self, stream: ResidualStream, step: StepContext, slot: LayerSlot) -> torch.Tensor:
        """``[N, hidden]``, or the mixer's mixes ``[mixes, N, hidden]`` where it takes them."""
        from ..ops.hyper import SingleTokens

        mixes: Optional[Part] = self.mixer.token_mixes
        mixes_slot = None
        if mixes is not None:
            mixer_slot = slot.of(self.names["mixer"])
            mixes_slot = next(mixer_slot.of(name) for name, part in self.mixer.sub_parts().items() if part is mixes)
        if self.filter is None and mixes is None:
            return self.norm1.forward(stream, read=self.join1.w_in)
        filter_slot = slot.of(self.names["filter"]) if self.filter is not None else None
        if step.max_q_len == 1:
            single = SingleTokens(step.req_slots, self.filter.weight if self.filter is not None else None,
                                  filter_slot.state if filter_slot is not None else None,
                                  mixes.mu if mixes is not None else None,
                                  mixes_slot.state if mixes_slot is not None else None)
            return self.norm1.forward(stream, read=self.join1.w_in, single=single)
        h = self.norm1.forward(stream, read=self.join1.w_in, out_dtype=torch.float32)
        if self.filter is not None:
            return self.filter.forward(h, step, filter_slot, mixes, mixes_slot)
        return mixes.forward(h, step, mixes_slot)

    def forward(self, stream: ResidualStream, step: StepContext, slot: LayerSlot) -> ResidualStream:
        step.residual = None                 # a sublayer's result joins the copies in the next norm's kernel
        x = self._mixer_input(stream, step, slot)
        stream.pending = self.mixer.forward(x, step, slot.of(self.names["mixer"]))
        stream.pending_join = self.join1.join
        if self.ffn is not None:
            x = self.norm2.forward(stream, read=self.join2.w_in)
            stream.pending = self.ffn.forward(x, step)
            stream.pending_join = self.join2.join
        return stream


register_part("norm", "copies", CopiesNorm)
register_part("block", "copies", CopiesBlock)
