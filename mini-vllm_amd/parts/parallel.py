"""Two mixers side by side on the same input, with one packed product for all their projections. The parts' tensors are
named ``left.<name>`` and ``right.<name>``. The left side (softmax attention) brings the cache, both sides their states.
In a step of single tokens the left side's cache write runs in the right side's launch.

* ``parallel``: y = (rms(left(h)) * w_left + rms(right(h)) * w_right) / 2 with rms(z) = z / sqrt(mean(z^2) + eps) over the
  model's width: attention behind a whole-row norm (``parts/attention.py``, a spec with ``row_norm``), a matrix state with a
  constant decay per head on the right (``parts/matrix_state.py: ConstantDecay``). The two output rows are left as a
  ``NormedPair``: the kernel of the next residual add and norm joins them. The two weights are ``left_out`` and ``right_out``.
* ``parallel_sum``: y = left(h) + right(h): attention on convolved projections (a spec with ``conv_taps``), gated linear
  attention on the right (``GatedLinear``); constants on the two sides are the specs' ``out_scale``. The heads' outputs of both
  sides lie in one row, so the two output projections and their sum are one product.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, Optional

import torch

from ..kernels.ops import NormedPair
from .attention import Attention, AttentionSpec
from .base import CacheNeed, Mixer, PartSpec, Runtime, TensorDecl, register_mixer
from .matrix_state import ConstantDecay, ConstantDecaySpec, GatedLinear, GatedLinearSpec


def _side(tensors: Dict[str, torch.Tensor], prefix: str) -> Dict[str, torch.Tensor]:
    return {name[len(prefix):]: t for name, t in tensors.items() if name.startswith(prefix)}


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
        self.left = Attention(spec.left, _side(tensors, "left."), rt)
        self.right = ConstantDecay(spec.right, _side(tensors, "right."), rt)
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


@dataclass(frozen=True)
class ParallelSumSpec(PartSpec):
    kind = "parallel_sum"
    hidden_size: int = 0
    left: Optional[AttentionSpec] = None
    right: Optional[GatedLinearSpec] = None

    @property
    def position(self) -> Optional[PartSpec]:
        return self.left.position


@register_mixer(ParallelSumSpec.kind)
class ParallelSum(Mixer):
    spec_class = ParallelSumSpec
    accepts_pending_norm = True         # the input is used by one packed product only
    accepts_fold = True                 # the output comes from one product

    @classmethod
    def tensors(cls, spec: ParallelSumSpec) -> Dict[str, TensorDecl]:
        t = {f"left.{name}": decl for name, decl in Attention.tensors(spec.left).items()}
        t.update({f"right.{name}": decl for name, decl in GatedLinear.tensors(spec.right).items()})
        return t

    @classmethod
    def cache_need(cls, spec: ParallelSumSpec) -> Optional[CacheNeed]:
        return Attention.cache_need(spec.left)

    @classmethod
    def state_shapes(cls, spec: ParallelSumSpec):
        return {**Attention.state_shapes(spec.left), **GatedLinear.state_shapes(spec.right)}

    def __init__(self, spec: ParallelSumSpec, tensors: Dict[str, torch.Tensor], rt: Runtime, position: Optional[object] = None):
        if not isinstance(spec.left, AttentionSpec) or not isinstance(spec.right, GatedLinearSpec) or not spec.left.convolved:
            raise ValueError("the sum of two mixers: softmax attention on convolved projections and gated linear attention")
        if spec.left.hidden_size != spec.hidden_size or spec.right.hidden_size != spec.hidden_size:
            raise ValueError("two mixers side by side read and write rows of the model's width")
        self.spec, self.rt = spec, rt
        self.left = Attention(spec.left, _side(tensors, "left."), rt, position=position)
        self.right = GatedLinear(spec.right, _side(tensors, "right."), rt)
        if self.left.w_qkv.dtype != self.right.w_packed.dtype or self.left.w_o.dtype != self.right.w_o.dtype:
            raise ValueError("the two sides' projections are stored in different dtypes; cannot pack them")
        # both sides' rows are multiples of 8 columns already
        self.right_base = self.left.width
        self.w_packed = torch.cat([self.left.w_qkv, self.right.w_packed], dim=0).contiguous()
        self.width = self.w_packed.shape[0]
        # the right side's columns of the joined row start at a multiple of 8, and the row's length is a multiple of 32: the
        # columns between have zero weights, and the row's buffer holds zeros there
        out_l, out_r, wide = spec.left.out_dim, spec.right.inner, self.left.w_o
        self.right_column = out_l + (-out_l) % 8
        self.inner = self.right_column + out_r + (-(self.right_column + out_r)) % 32
        self.w_o = torch.zeros((spec.hidden_size, self.inner), dtype=wide.dtype, device=wide.device)
        self.w_o[:, :out_l] = self.left.w_o
        self.w_o[:, self.right_column:self.right_column + out_r] = self.right.w_o
        self.left.w_qkv = self.left.w_o = self.right.w_packed = self.right.w_o = None
        self.gaps = [(a, b) for a, b in ((out_l, self.right_column), (self.right_column + out_r, self.inner)) if b > a]

    def first_product(self):
        return self.w_packed.shape[0], self.w_packed.shape[1], False

    def forward(self, x: torch.Tensor, ctx, call: int, fold=None):
        spec, rt, ops, ws = self.spec, self.rt, self.rt.ops, self.rt.workspace
        n, left, right = x.shape[0], self.left, self.right
        packed = ws.get("parallel.packed", (n, self.width), rt.dtype)
        ops.gemm(x, self.w_packed, packed)
        heads = ws.get("parallel.heads", (n, self.inner), rt.dtype)
        for a, b in self.gaps:
            heads[:, a:b].zero_()
        beside = left.conv_store_args(packed, 0, ctx, call)
        rows = heads[:, self.right_column:self.right_column + spec.right.inner]
        if not right.recur(packed, self.right_base, ctx, call, rows, beside=beside):
            left.conv_store(packed, 0, ctx, call)
        left.attend_scored(beside["out"], 0, ctx, call, out=heads[:, :spec.left.out_dim])
        y = ws.get("mixer.out", (n, spec.hidden_size), rt.dtype)
        return ops.gemm(heads, self.w_o, y, defer_sum=True, fold=fold) or y
