"""Two mixers side by side on the same input.

y = (rms(left(h)) * w_left + rms(right(h)) * w_right) / 2 with rms(z) = z / sqrt(mean(z^2) + eps) over the model's
width: softmax attention on the left (``parts/attention.py``, a spec with ``row_norm``), a matrix state with a
constant decay per head on the right (``parts/matrix_state.py: ConstantDecay``). All projections of the input are one
packed product. The two output rows are left as a ``NormedPair``: the kernel of the next residual add and norm joins
them. In a step of single tokens the left side's norm and cache write run in the right side's launch.

The parts' tensors are named ``left.<name>`` and ``right.<name>``, the two weights ``left_out`` and ``right_out``.
The left side brings the cache, the right side the state.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, Optional

import torch

from ..kernels.ops import NormedPair
from .attention import Attention, AttentionSpec
from .base import CacheNeed, Mixer, PartSpec, Runtime, TensorDecl, register_mixer
from .matrix_state import ConstantDecay, ConstantDecaySpec


@dataclass(frozen=True)
class ParallelMixerSpec(PartSpec):
    kind = "parallel"
    hidden_size: int = 0
    left: Optional[AttentionSpec] = None
    right: Optional[ConstantDecaySpec] = None
    out_norm_eps: float = 1e-6


@register_mixer(ParallelMixerSpec.kind)
class ParallelMixer(Mixer):
    spec_class = ParallelMixerSpec
    accepts_pending_norm = True         # the input is used by one packed product only

    @classmethod
    def tensors(cls, spec: ParallelMixerSpec) -> Dict[str, TensorDecl]:
        t = {f"left.{name}": decl for name, decl in Attention.tensors(spec.left).items()}
        t.update({f"right.{name}": decl for name, decl in ConstantDecay.tensors(spec.right).items()})
        for side in ("left_out", "right_out"):
            t[side] = TensorDecl((spec.hidden_size,), init="ones_normal")
        return t

    @classmethod
    def cache_need(cls, spec: ParallelMixerSpec) -> Optional[CacheNeed]:
        return Attention.cache_need(spec.left)

    @classmethod
    def state_shapes(cls, spec: ParallelMixerSpec):
        return ConstantDecay.state_shapes(spec.right)

    def __init__(self, spec: ParallelMixerSpec, tensors: Dict[str, torch.Tensor], rt: Runtime, position: Optional[object] = None):
        if not isinstance(spec.left, AttentionSpec) or not isinstance(spec.right, ConstantDecaySpec) or not spec.left.scored:
            raise ValueError("two mixers side by side: softmax attention behind a whole-row norm and a constant decay")
        if spec.left.hidden_size != spec.hidden_size or spec.right.hidden_size != spec.hidden_size:
            raise ValueError("two mixers side by side read and write rows of the model's width")
        self.spec, self.rt = spec, rt

        def side(prefix: str) -> Dict[str, torch.Tensor]:
            return {name[len(prefix):]: t for name, t in tensors.items() if name.startswith(prefix)}

        self.left = Attention(spec.left, side("left."), rt)
        self.right = ConstantDecay(spec.right, side("right."), rt)
        if self.left.w_qkv.dtype != self.right.w_packed.dtype:
            raise ValueError("the two sides' projections are stored in different dtypes; cannot pack them")
        # both sides' rows are multiples of 8 columns already
        self.right_base = self.left.width
        self.w_packed = torch.cat([self.left.w_qkv, self.right.w_packed], dim=0).contiguous()
        self.left.w_qkv = self.right.w_packed = None
        self.width = self.w_packed.shape[0]
        self.w_left, self.w_right = tensors["left_out"].contiguous(), tensors["right_out"].to(tensors["left_out"].dtype).contiguous()

    def first_product(self):
        return self.w_packed.shape[0], self.w_packed.shape[1], False

    def forward(self, x: torch.Tensor, ctx, call: int):
        spec, rt, ops, ws = self.spec, self.rt, self.rt.ops, self.rt.workspace
        n, left, right = x.shape[0], self.left, self.right
        packed = ws.get("parallel.packed", (n, self.width), rt.dtype)
        ops.gemm(x, self.w_packed, packed)
        offsets = left.offsets(0)
        rows, sums, stored = right.recur(packed, self.right_base, ctx, call, beside=left.norm_store_args(packed, offsets, ctx, call))
        if not stored:
            left.norm_store(packed, offsets, ctx, call)
        attn = left.attend_scored(packed, offsets[0], ctx, call)
        y_left = ws.get("parallel.left", (n, spec.hidden_size), rt.dtype)
        y_right = ws.get("parallel.right", (n, spec.hidden_size), rt.dtype)
        ops.gemm(attn, left.w_o, y_left)
        ops.gemm(rows, right.w_o, y_right)
        y = ws.get("mixer.out", (n, spec.hidden_size), rt.dtype)
        return NormedPair(ops, (y_left, y_right), (self.w_left, self.w_right), spec.out_norm_eps, (None, sums), y)
