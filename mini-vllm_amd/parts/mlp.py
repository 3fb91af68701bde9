"""Gated feed-forward: y = (silu(x Wg^T) * (x Wu^T)) Wd^T.

Reference: minivllm/models/models/qwen3.py:104-121 — three bias-free projections, SiLU on the
gate. Gate and up are packed into one matrix product here; the activation and the product
are computed in float32.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict

import torch

from .base import FeedForward, PartSpec, Runtime, TensorDecl, register_feed_forward


@dataclass(frozen=True)
class SwiGLUSpec(PartSpec):
    kind = "swiglu"
    hidden_size: int = 0
    intermediate_size: int = 0


@register_feed_forward(SwiGLUSpec.kind)
class SwiGLU(FeedForward):
    spec_class = SwiGLUSpec
    accepts_pending_norm = True      # the input is used by one packed product only
    accepts_fold = True              # the output comes from one product

    @classmethod
    def tensors(cls, spec: SwiGLUSpec) -> Dict[str, TensorDecl]:
        return {"gate": TensorDecl((spec.intermediate_size, spec.hidden_size)),
                "up": TensorDecl((spec.intermediate_size, spec.hidden_size)),
                "down": TensorDecl((spec.hidden_size, spec.intermediate_size))}

    def __init__(self, spec: SwiGLUSpec, tensors: Dict[str, torch.Tensor], rt: Runtime):
        self.spec = spec
        self.rt = rt
        if tensors["gate"].dtype != tensors["up"].dtype:
            raise ValueError("gate and up projections are stored in different dtypes; cannot pack them")
        self.w_gate_up = torch.cat([tensors["gate"], tensors["up"]], dim=0).contiguous()
        self.w_down = tensors["down"]

    def first_product(self):
        return self.w_gate_up.shape[0], self.w_gate_up.shape[1], True

    def forward(self, x: torch.Tensor, ctx, fold=None) -> torch.Tensor:
        spec, rt, ops = self.spec, self.rt, self.rt.ops
        n = x.shape[0]
        act = rt.workspace.get("ffn.act", (n, spec.intermediate_size), rt.dtype)
        if not ops.gemm_swiglu(x, self.w_gate_up, act):      # one pass over the weight for few rows
            gu = rt.workspace.get("ffn.gate_up", (n, 2 * spec.intermediate_size), rt.dtype)
            if not isinstance(x, torch.Tensor):
                x = x.materialize()
            ops.gemm(x, self.w_gate_up, gu)
            ops.swiglu(gu, act)
        y = rt.workspace.get("ffn.out", (n, spec.hidden_size), rt.dtype)
        # (the sums of a product whose K was split may be left to the next norm, or the residual add and
        # that norm folded into the product)
        return ops.gemm(act, self.w_down, y, defer_sum=True, fold=fold) or y


@dataclass(frozen=True)
class XIELUSpec(PartSpec):
    """Two projections with the xIELU activation between them: y = Wd act(Wu x), where
    act(z) = a_pos z^2 + z / 2 for z > 0 and a_neg (exp(z) - 1 - z) + z / 2 for z <= 0, with
    a_pos = softplus(p) and a_neg = 1/2 + softplus(q) from the layer's two stored numbers (p, q)."""
    kind = "xielu_mlp"
    hidden_size: int = 0
    intermediate_size: int = 0


@register_feed_forward(XIELUSpec.kind)
class XIELUFeedForward(FeedForward):
    spec_class = XIELUSpec

    @classmethod
    def tensors(cls, spec: XIELUSpec) -> Dict[str, TensorDecl]:
        return {"up": TensorDecl((spec.intermediate_size, spec.hidden_size)),
                "down": TensorDecl((spec.hidden_size, spec.intermediate_size)),
                "act": TensorDecl((2,), init="zeros_normal")}

    def __init__(self, spec: XIELUSpec, tensors: Dict[str, torch.Tensor], rt: Runtime):
        self.spec, self.rt = spec, rt
        self.w_up, self.w_down = tensors["up"], tensors["down"]
        # the two constants of the activation, once, in float32 (they belong to the weights, not to a step)
        pq = torch.nn.functional.softplus(tensors["act"].to(torch.float32)).tolist()
        self.a_pos, self.a_neg = float(pq[0]), 0.5 + float(pq[1])

    def forward(self, x: torch.Tensor, ctx) -> torch.Tensor:
        spec, rt, ops = self.spec, self.rt, self.rt.ops
        if not isinstance(x, torch.Tensor):
            x = x.materialize()
        n = x.shape[0]
        act = rt.workspace.get("ffn.act", (n, spec.intermediate_size), rt.dtype)
        ops.gemm(x, self.w_up, act)
        ops.xielu(act, self.a_pos, self.a_neg, act)
        y = rt.workspace.get("ffn.out", (n, spec.hidden_size), rt.dtype)
        return ops.gemm(act, self.w_down, y, defer_sum=True) or y


@dataclass(frozen=True)
class SquaredReLUSpec(PartSpec):
    """Two projections with the square of ReLU between them: y = Wd max(Wu x + bu, 0)^2 + bd; ``bias`` False leaves both
    biases out."""
    kind = "squared_relu_mlp"
    hidden_size: int = 0
    intermediate_size: int = 0
    bias: bool = True


@register_feed_forward(SquaredReLUSpec.kind)
class SquaredReLU(FeedForward):
    spec_class = SquaredReLUSpec

    @classmethod
    def tensors(cls, spec: SquaredReLUSpec) -> Dict[str, TensorDecl]:
        t = {"up": TensorDecl((spec.intermediate_size, spec.hidden_size)),
             "down": TensorDecl((spec.hidden_size, spec.intermediate_size))}
        if spec.bias:
            t.update(up_bias=TensorDecl((spec.intermediate_size,), init="zeros_normal"),
                     down_bias=TensorDecl((spec.hidden_size,), init="zeros_normal"))
        return t

    def __init__(self, spec: SquaredReLUSpec, tensors: Dict[str, torch.Tensor], rt: Runtime):
        self.spec, self.rt = spec, rt
        self.w_up, self.w_down = tensors["up"], tensors["down"]
        self.b_up = self.b_down = None
        if spec.bias:
            self.b_up = tensors["up_bias"].to(self.w_up.dtype).contiguous()
            self.b_down = tensors["down_bias"].to(self.w_down.dtype).contiguous()

    def forward(self, x: torch.Tensor, ctx) -> torch.Tensor:
        spec, rt, ops = self.spec, self.rt, self.rt.ops
        if not isinstance(x, torch.Tensor):
            x = x.materialize()
        n = x.shape[0]
        act = rt.workspace.get("ffn.act", (n, spec.intermediate_size), rt.dtype)
        ops.gemm_squared_relu(x, self.w_up, act, self.b_up)
        y = rt.workspace.get("ffn.out", (n, spec.hidden_size), rt.dtype)
        return ops.gemm(act, self.w_down, y, self.b_down, defer_sum=True) or y


@dataclass(frozen=True)
class ClampedGLUSpec(PartSpec):
    """A gated pair with clamped halves: g = min(Wg x + bg, limit), u = clamp(Wu x + bu, -limit, limit),
    y = Wd (g * sigmoid(slope * g) * (u + 1)) + bd; ``bias`` False leaves the three biases out."""
    kind = "clamped_glu"
    hidden_size: int = 0
    intermediate_size: int = 0
    limit: float = 0.0
    slope: float = 1.702
    bias: bool = True


@register_feed_forward(ClampedGLUSpec.kind)
class ClampedGLU(FeedForward):
    spec_class = ClampedGLUSpec
    accepts_pending_norm = True      # the input is used by one packed product only
    accepts_fold = True              # the output comes from one product

    @classmethod
    def tensors(cls, spec: ClampedGLUSpec) -> Dict[str, TensorDecl]:
        hid, ff = spec.hidden_size, spec.intermediate_size
        t = {"gate": TensorDecl((ff, hid)), "up": TensorDecl((ff, hid)), "down": TensorDecl((hid, ff))}
        if spec.bias:
            t.update(gate_bias=TensorDecl((ff,), init="zeros_normal"), up_bias=TensorDecl((ff,), init="zeros_normal"),
                     down_bias=TensorDecl((hid,), init="zeros_normal"))
        return t

    def __init__(self, spec: ClampedGLUSpec, tensors: Dict[str, torch.Tensor], rt: Runtime):
        if not spec.limit > 0:
            raise ValueError(f"a clamped pair needs a positive limit, got {spec.limit}")
        self.spec, self.rt = spec, rt
        if tensors["gate"].dtype != tensors["up"].dtype:
            raise ValueError("gate and up projections are stored in different dtypes; cannot pack them")
        self.w_gate_up = torch.cat([tensors["gate"], tensors["up"]], dim=0).contiguous()
        self.w_down = tensors["down"]
        self.b_gate_up = self.b_down = None
        if spec.bias:
            self.b_gate_up = torch.cat([tensors["gate_bias"], tensors["up_bias"]], dim=0).to(self.w_gate_up.dtype).contiguous()
            self.b_down = tensors["down_bias"].to(self.w_down.dtype).contiguous()

    def first_product(self):
        return self.w_gate_up.shape[0], self.w_gate_up.shape[1], True

    def forward(self, x: torch.Tensor, ctx, fold=None) -> torch.Tensor:
        spec, rt, ops = self.spec, self.rt, self.rt.ops
        n = x.shape[0]
        act = rt.workspace.get("ffn.act", (n, spec.intermediate_size), rt.dtype)
        if not ops.gemm_swiglu(x, self.w_gate_up, act, self.b_gate_up, limit=spec.limit, slope=spec.slope):
            gu = rt.workspace.get("ffn.gate_up", (n, 2 * spec.intermediate_size), rt.dtype)
            if not isinstance(x, torch.Tensor):
                x = x.materialize()
            ops.gemm(x, self.w_gate_up, gu, self.b_gate_up)
            ops.swiglu(gu, act, limit=spec.limit, slope=spec.slope)
        y = rt.workspace.get("ffn.out", (n, spec.hidden_size), rt.dtype)
        return ops.gemm(act, self.w_down, y, self.b_down, defer_sum=True, fold=fold) or y
