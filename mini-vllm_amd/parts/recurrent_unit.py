"""The real-gated linear recurrent unit (Griffin's recurrent block): a state of one number per channel.

Two branches of ``width`` channels from the mixer's input h: y = gelu_tanh(W_y h + b_y) and u = conv(W_x h + b_x) + b_c, a
causal convolution over time per channel with ``conv_taps`` taps (the last one the current token's, zeros before the start,
no activation). u is cut into ``blocks`` equal parts; part b passes two square matrices,

    r = sigmoid(ra[b] u_b + ra_bias[b]),   i = sigmoid(ri[b] u_b + ri_bias[b])

and per channel, from S = 0,

    log a = -GATE_POWER * r * softplus(lam),   S <- a S + sqrt(1 - a^2) * i * u,   out = W_o (S * y).

S is float32 [width] per request; the convolution's last ``conv_taps - 1`` inputs (activation type) are state too. Gates,
decays and the recurrence are float32 whatever the activation type. Both projections are one packed product. Prompt portions
run as convolution, one product per part for both gates (float32 rows), and a scan cut into chunks of tokens that run side by
side; a step of single tokens runs everything between the two products as one kernel beside the move of the kept inputs.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, Optional

import torch

from .base import Mixer, PartSpec, Runtime, TensorDecl, register_mixer

GATE_POWER = 8.0


@dataclass(frozen=True)
class RecurrentUnitSpec(PartSpec):
    kind = "recurrent_unit"
    hidden_size: int = 0
    width: int = 0
    blocks: int = 1
    conv_taps: int = 1

    @property
    def block_size(self) -> int:
        return self.width // self.blocks


@register_mixer(RecurrentUnitSpec.kind)
class RecurrentUnit(Mixer):
    spec_class = RecurrentUnitSpec
    accepts_pending_norm = True         # the input is used by one packed product only
    accepts_fold = True                 # the output comes from one product

    @classmethod
    def tensors(cls, spec: RecurrentUnitSpec) -> Dict[str, TensorDecl]:
        hid, W, B, b = spec.hidden_size, spec.width, spec.blocks, spec.block_size
        return {"y": TensorDecl((W, hid)), "y_bias": TensorDecl((W,), init="zeros_normal"),
                "x": TensorDecl((W, hid)), "x_bias": TensorDecl((W,), init="zeros_normal"),
                "conv": TensorDecl((W, spec.conv_taps)), "conv_bias": TensorDecl((W,), init="zeros_normal"),
                "ra": TensorDecl((B, b, b)), "ra_bias": TensorDecl((B, b), init="zeros_normal"),
                "ri": TensorDecl((B, b, b)), "ri_bias": TensorDecl((B, b), init="zeros_normal"),
                "lam": TensorDecl((W,), init="zeros_normal"), "o": TensorDecl((hid, W))}

    @classmethod
    def state_shapes(cls, spec: RecurrentUnitSpec):
        shapes = {"state": ((spec.width,), torch.float32)}
        if spec.conv_taps > 1:
            shapes["conv"] = ((spec.conv_taps - 1, spec.width), None)      # the activation type
        return shapes

    def __init__(self, spec: RecurrentUnitSpec, tensors: Dict[str, torch.Tensor], rt: Runtime, position: Optional[object] = None):
        if min(spec.width, spec.blocks, spec.conv_taps) < 1 or spec.width % spec.blocks:
            raise ValueError(f"recurrent unit: bad sizes {spec}")
        if tensors["y"].dtype != tensors["x"].dtype or tensors["ra"].dtype != tensors["ri"].dtype:
            raise ValueError("recurrent unit: the branches' projections or the gates' matrices are stored in different dtypes")
        self.spec, self.rt = spec, rt
        # packed rows [x | y], each padded to a multiple of 8 columns
        pad = (-spec.width) % 8
        self.y_offset = spec.width + pad

        def padded(t: torch.Tensor) -> torch.Tensor:
            return t if not pad else torch.cat([t, torch.zeros((pad,) + tuple(t.shape[1:]), dtype=t.dtype, device=t.device)], dim=0)

        self.w_packed = torch.cat([padded(tensors["x"]), padded(tensors["y"])], dim=0).contiguous()
        self.b_packed = torch.cat([padded(tensors["x_bias"]), padded(tensors["y_bias"])], dim=0).to(self.w_packed.dtype).contiguous()
        self.packed_width = self.w_packed.shape[0]
        f32 = torch.float32
        self.conv_t = tensors["conv"].to(f32).t().contiguous()             # tap by tap, [taps, width]
        self.conv_bias = tensors["conv_bias"].to(f32).contiguous()
        # both gates of a part in one matrix, [blocks, 2 * block_size outputs, inputs], and with the inputs' rows outside
        self.gate_rows = torch.cat([tensors["ra"], tensors["ri"]], dim=1).contiguous()
        self.gate_cols = self.gate_rows.transpose(1, 2).contiguous()
        self.gate_bias = torch.stack([tensors["ra_bias"].reshape(-1), tensors["ri_bias"].reshape(-1)]).to(f32).contiguous()
        # log a = rate * r: a constant of the weights, once, in float32
        self.rate = (-GATE_POWER * torch.nn.functional.softplus(tensors["lam"].to(f32))).contiguous()
        self.w_o = tensors["o"]

    def first_product(self):
        return self.w_packed.shape[0], self.w_packed.shape[1], False

    def forward(self, x: torch.Tensor, ctx, call: int, fold=None) -> torch.Tensor:
        spec, rt, ops, ws = self.spec, self.rt, self.rt.ops, self.rt.workspace
        n, W, B = x.shape[0], spec.width, spec.blocks
        packed = ws.get("unit.packed", (n, self.packed_width), rt.dtype)
        ops.gemm(x, self.w_packed, packed, self.b_packed)
        gated = ws.get("unit.gated", (n, W), rt.dtype)
        y = ws.get("mixer.out", (n, spec.hidden_size), rt.dtype)
        conv_state = ctx.state(call, "conv") if spec.conv_taps > 1 else None
        plan = ctx.attention_plan
        single = plan is not None and plan.decode_only
        if single and ops.unit_step(packed, self.y_offset, B, self.conv_t, self.conv_bias, conv_state, self.gate_rows, self.gate_cols,
                                    self.gate_bias, self.rate, ctx.state(call), ctx.token_seq, ctx.state_slots, gated):
            return ops.gemm(gated, self.w_o, y, defer_sum=True, fold=fold) or y
        u = ws.get("unit.u", (n, W), rt.dtype)
        ops.short_conv(packed, W, self.conv_t, self.conv_bias, conv_state, ctx.token_seq, ctx.cu_seqlens, ctx.state_slots, ctx.n_seqs, u)
        z = ws.get("unit.z", (n, B, 2 * spec.block_size), torch.float32)
        ops.head_linear(u.view(n, B, spec.block_size), self.gate_cols, z, ctx.token_seq, w_rows=self.gate_rows)
        chunks = plan.units(ops.unit_chunk_tokens()) if plan is not None else n
        sums = ws.get("unit.chunks", (chunks, 2, W), torch.float32)
        ops.unit_scan(z, u, packed, self.y_offset, B, self.gate_bias, self.rate, ctx.state(call), ctx.token_seq, ctx.cu_seqlens,
                      ctx.state_slots, ctx.n_seqs, chunks, sums, gated)
        return ops.gemm(gated, self.w_o, y, defer_sum=True, fold=fold) or y
