"""What is added to the residual stream in front of a run of layers that is run several times in a row.

In front of pass t of such a run (t = 0, 1, ...): x <- x + [t > 0] e + step[t], with e the embedding's output for the
token and ``step`` [times, width] stored vectors. The embedding's rows are read from its table again, so nothing is
kept between the passes; the pending delta, both additions and the norm of the run's first layer are one kernel.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, Optional

import torch

from .base import HiddenStream, Part, PartSpec, Runtime, TensorDecl, register_stream_entry


@dataclass(frozen=True)
class PassEntrySpec(PartSpec):
    kind = "pass_entry"
    hidden_size: int = 0
    times: int = 1


@register_stream_entry(PassEntrySpec.kind)
class PassEntry(Part):
    spec_class = PassEntrySpec

    @classmethod
    def tensors(cls, spec: PassEntrySpec) -> Dict[str, TensorDecl]:
        return {"step": TensorDecl((spec.times, spec.hidden_size), init="zeros_normal")}

    def __init__(self, spec: PassEntrySpec, tensors: Dict[str, torch.Tensor], rt: Runtime, embedding):
        if spec.times < 1:
            raise ValueError(f"a run of layers is run at least once, got {spec.times} times")
        if spec.times > 1 and not hasattr(embedding, "row_table"):
            raise NotImplementedError("a later pass adds the embedding's output again: the embedding must offer row_table()")
        self.spec, self.rt, self.embedding = spec, rt, embedding
        self.steps = [row.contiguous() for row in tensors["step"]]

    def forward(self, stream: HiddenStream, ctx, number: int, norm=None) -> None:
        """Enters pass ``number``; the rows of ``norm`` (the norm that comes next) are left in the stream when it is a
        plain scaled RMS norm."""
        if stream.lanes is not None or stream.weighted is not None:
            raise RuntimeError("a run of layers is entered with a plain residual stream")
        delta = stream.delta
        if delta is not None and not isinstance(delta, torch.Tensor):
            delta = delta.materialize()
        rows = None
        if number > 0:
            table, scale = self.embedding.row_table()
            rows = (ctx.token_ids, table, scale)
        form = norm.as_scaled_rms() if norm is not None else None
        out = self.rt.workspace.get("normed", tuple(stream.resid.shape), self.rt.dtype) if form is not None else None
        self.rt.ops.stream_entry(stream.resid, delta, rows, self.steps[number], form, out)
        stream.delta = None
        stream.normed = (norm, out) if out is not None else None
