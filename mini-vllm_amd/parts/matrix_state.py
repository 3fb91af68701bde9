"""Recurrent mixers whose state is one decayed matrix per head, written with scalar gates.

Per token and head, with query q and key k (``key_dim`` each), value v (``value_dim``) and two
scalars a (how much of the old state stays) and b (how strongly the token is written):

    S <- a S;   u = b (v - [delta] S^T k);   S <- S + k u^T;   o = S^T q

so the read-out sees the token's own write.

* ``gated_delta`` (the gated delta rule): [delta] is on. q and k come from ``num_kv_heads`` groups
  (head h reads group h // (num_heads / num_kv_heads)); q, k and v pass a short causal convolution
  over time per channel (``conv_taps`` taps, the last one the current token's, zeros before the
  start) and SiLU; q and k are then made unit vectors, x / sqrt(sum(x^2) + unit_eps), q also times
  key_dim^-1/2. b = sigmoid(W_b h) and a = exp(-exp(A_log) * softplus(W_a h + dt_bias)) per head.
  o is divided by its root mean square per head, multiplied by a weight of ``value_dim`` numbers
  that the heads share and by silu(W_g h).
* ``mlstm`` (the matrix memory of the xLSTM): [delta] is off. q = W_q h * key_dim^-1/2. With the log
  input gate i = cap tanh((W_i h + b_i) / cap), the log forget gate
  f = logsigmoid(cap tanh((W_f h + b_f) / cap)) and a running maximum m (0 at the start),
  m' = max(f + m, i), the scalars are a = exp(f + m - m'), b = exp(i - m'). A normaliser n (the same
  recurrence on k alone) is kept as one more column of S, fed with the value 1, and
  o <- o / (max(|n . q|, exp(-m')) + denom_eps). o is then divided by its root mean square per head,
  multiplied by a weight over all heads' channels and by sigmoid(W_g h).

* ``channel_delta`` (the gated delta rule with a decay per key channel): as ``gated_delta``, but a is a vector over
  the key channels, S <- diag(a) S, a = exp(-exp(A_log) * softplus(W_a2 (W_a1 h) + dt_bias)) per head and channel
  (A_log per head), and o, after its norm, is multiplied by sigmoid(W_g2 (W_g1 h)).
* ``constant_decay`` (lightning attention): [delta] is off, a is a constant per head and b = 1; q, k and v are SiLU of
  their projections. All heads' o together are divided by their root mean square, multiplied by a weight over all
  channels and by sigmoid(W_g h).

* ``gated_linear`` (gated linear attention): [delta] is off, b = 1, a is a vector over the key channels, S <- diag(a) S with
  a = sigmoid(z)^(1 / tau), z = W_a2 (W_a1 h) + bias per head and channel; q = W_q h * key_dim^-1/2, k and v are plain
  projections. o is divided by its root mean square per head, multiplied by a weight of ``value_dim`` numbers that the
  heads share and by silu(W_g h); ``out_scale`` is a constant on the result.

All keep S as float32 [heads, columns, key_dim] per request (a head's matrix column by column),
zero at a request's start; the convolution's last ``conv_taps - 1`` inputs (activation type) and the
running maximum (float32 [heads]) are state too. Gates, unit vectors and the recurrence are float32
whatever the activation type. All projections of the mixer's input are one packed product.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, Optional, Tuple

import torch

from ..kernels.ops import RowSums
from .base import Mixer, PartSpec, Runtime, TensorDecl, register_mixer


def _pack(tensors: Dict[str, torch.Tensor], names, hidden: int, what: str):
    dtypes = {tensors[p].dtype for p in names}
    if len(dtypes) != 1:
        raise ValueError(f"{what}: the projections are stored in different dtypes {dtypes}; cannot pack them")
    blocks = [tensors[p] for p in names]
    rows = sum(b.shape[0] for b in blocks)
    pad = (-rows) % 8             # rows of the packed product keep a pitch of a multiple of 8 elements
    if pad:
        blocks.append(torch.zeros((pad, hidden), dtype=blocks[0].dtype, device=blocks[0].device))
    return torch.cat(blocks, dim=0).contiguous()


@dataclass(frozen=True)
class GatedDeltaSpec(PartSpec):
    kind = "gated_delta"
    hidden_size: int = 0
    num_heads: int = 0
    num_kv_heads: int = 0
    key_dim: int = 0
    value_dim: int = 0
    conv_taps: int = 1                  # 1: no convolution (a single tap still scales each channel)
    unit_eps: float = 1e-6              # inside the root of a query's or key's length
    out_norm_eps: float = 1e-6          # of the per-head RMS of the output

    @property
    def conv_channels(self) -> int:
        return 2 * self.num_kv_heads * self.key_dim + self.num_heads * self.value_dim


@register_mixer(GatedDeltaSpec.kind)
class GatedDelta(Mixer):
    spec_class = GatedDeltaSpec
    PACKED = ("q", "k", "v", "g", "b", "a")

    @classmethod
    def tensors(cls, spec: GatedDeltaSpec) -> Dict[str, TensorDecl]:
        hid, qk, vd = spec.hidden_size, spec.num_kv_heads * spec.key_dim, spec.num_heads * spec.value_dim
        t = {"q": TensorDecl((qk, hid)), "k": TensorDecl((qk, hid)), "v": TensorDecl((vd, hid)), "g": TensorDecl((vd, hid)),
             "b": TensorDecl((spec.num_heads, hid)), "a": TensorDecl((spec.num_heads, hid)),
             "q_conv": TensorDecl((qk, spec.conv_taps)), "k_conv": TensorDecl((qk, spec.conv_taps)),
             "v_conv": TensorDecl((vd, spec.conv_taps)),
             "A_log": TensorDecl((spec.num_heads,), init="zeros_normal"),
             "dt_bias": TensorDecl((spec.num_heads,), init="zeros_normal"),
             "norm": TensorDecl((spec.value_dim,), init="ones_normal"),
             "o": TensorDecl((hid, vd))}
        return t

    @classmethod
    def state_shapes(cls, spec: GatedDeltaSpec):
        shapes = {"state": ((spec.num_heads, spec.value_dim, spec.key_dim), torch.float32)}
        if spec.conv_taps > 1:
            shapes["conv"] = ((spec.conv_taps - 1, spec.conv_channels), None)      # the activation type
        return shapes

    def __init__(self, spec: GatedDeltaSpec, tensors: Dict[str, torch.Tensor], rt: Runtime, position: Optional[object] = None):
        if min(spec.num_heads, spec.num_kv_heads, spec.key_dim, spec.value_dim, spec.conv_taps) < 1 \
                or spec.num_heads % spec.num_kv_heads:
            raise ValueError(f"gated delta rule: bad sizes {spec}")
        self.spec, self.rt = spec, rt
        self.w_packed = _pack(tensors, self.PACKED, spec.hidden_size, "gated delta rule")
        self.width = self.w_packed.shape[0]
        self.gate_offset = spec.conv_channels
        self.conv_w = torch.cat([tensors["q_conv"], tensors["k_conv"], tensors["v_conv"]], dim=0).contiguous()
        self.a_log = tensors["A_log"].to(self.conv_w.dtype).contiguous()
        self.dt_bias = tensors["dt_bias"].to(self.conv_w.dtype).contiguous()
        self.norm, self.w_o = tensors["norm"].to(self.conv_w.dtype).contiguous(), tensors["o"]

    def forward(self, x: torch.Tensor, ctx, call: int) -> torch.Tensor:
        spec, rt, ops, ws = self.spec, self.rt, self.rt.ops, self.rt.workspace
        n, H, G, dk, dv = x.shape[0], spec.num_heads, spec.num_kv_heads, spec.key_dim, spec.value_dim
        packed = ws.get("mstate.packed", (n, self.width), rt.dtype)
        ops.gemm(x, self.w_packed, packed)
        gated = ws.get("mstate.gated", (n, H * dv), rt.dtype)
        y = ws.get("mixer.out", (n, spec.hidden_size), rt.dtype)
        plan = ctx.attention_plan
        # every request brings one token: everything between the two products as one kernel
        if plan is not None and plan.decode_only and ops.state_step(
                True, packed, H, G, dk, dv, self.norm, spec.out_norm_eps, ctx.state(call), ctx.token_seq, ctx.cu_seqlens,
                ctx.state_slots, ctx.n_seqs, gated, taps=spec.conv_taps, conv_w=self.conv_w, a_log=self.a_log,
                dt_bias=self.dt_bias, conv_state=ctx.state(call, "conv") if spec.conv_taps > 1 else None,
                unit_eps=spec.unit_eps):
            return ops.gemm(gated, self.w_o, y, defer_sum=True) or y
        qk = ws.get("mstate.qk", (n, G, 2, dk), torch.float32)
        vals = ws.get("mstate.vals", (n, H, dv), torch.float32)
        gates = ws.get("mstate.gates", (n, H, 4), torch.float32)
        ops.gated_delta_prepare(packed, H, G, dk, dv, spec.conv_taps, self.conv_w, self.a_log, self.dt_bias,
                                ctx.state(call, "conv") if spec.conv_taps > 1 else None, spec.unit_eps, ctx.token_seq,
                                ctx.cu_seqlens, ctx.state_slots, ctx.n_seqs, qk, vals, gates)
        raw = ws.get("mstate.raw", (n, H, dv), torch.float32)
        ops.state_scan(qk, vals, gates, ctx.state(call), ctx.cu_seqlens, ctx.state_slots, ctx.n_seqs, H, G, dk, dv, True, raw)
        ops.state_finish(raw, gates, packed, self.gate_offset, self.norm, H, dv, spec.out_norm_eps, ctx.token_seq, gated,
                         shared_weight=True, silu_gate=True)
        return ops.gemm(gated, self.w_o, y, defer_sum=True) or y


@dataclass(frozen=True)
class MLSTMSpec(PartSpec):
    kind = "mlstm"
    hidden_size: int = 0
    num_heads: int = 0
    key_dim: int = 0
    value_dim: int = 0
    gate_cap: float = 15.0              # both gates' pre-activations are squashed into (-cap, cap)
    denom_eps: float = 1e-6             # added to the denominator
    out_norm_eps: float = 1e-6          # of the per-head RMS of the output


@register_mixer(MLSTMSpec.kind)
class MLSTM(Mixer):
    spec_class = MLSTMSpec
    PACKED = ("q", "k", "v", "g", "i", "f")

    @classmethod
    def tensors(cls, spec: MLSTMSpec) -> Dict[str, TensorDecl]:
        hid, qk, vd = spec.hidden_size, spec.num_heads * spec.key_dim, spec.num_heads * spec.value_dim
        return {"q": TensorDecl((qk, hid)), "k": TensorDecl((qk, hid)), "v": TensorDecl((vd, hid)), "g": TensorDecl((vd, hid)),
                "i": TensorDecl((spec.num_heads, hid)), "f": TensorDecl((spec.num_heads, hid)),
                "i_bias": TensorDecl((spec.num_heads,), init="zeros_normal"),
                "f_bias": TensorDecl((spec.num_heads,), init="zeros_normal"),
                "norm": TensorDecl((vd,), init="ones_normal"), "o": TensorDecl((hid, vd))}

    @classmethod
    def state_shapes(cls, spec: MLSTMSpec):
        # the matrix with the normaliser as its last column; the running maximum
        return {"state": ((spec.num_heads, spec.value_dim + 1, spec.key_dim), torch.float32),
                "max": ((spec.num_heads,), torch.float32)}

    def __init__(self, spec: MLSTMSpec, tensors: Dict[str, torch.Tensor], rt: Runtime, position: Optional[object] = None):
        if min(spec.num_heads, spec.key_dim, spec.value_dim) < 1 or not spec.gate_cap > 0:
            raise ValueError(f"mlstm: bad sizes {spec}")
        self.spec, self.rt = spec, rt
        self.w_packed = _pack(tensors, self.PACKED, spec.hidden_size, "mlstm")
        self.width = self.w_packed.shape[0]
        self.gate_offset = spec.num_heads * (2 * spec.key_dim + spec.value_dim)
        self.i_bias = tensors["i_bias"].contiguous()
        self.f_bias = tensors["f_bias"].to(self.i_bias.dtype).contiguous()
        self.norm, self.w_o = tensors["norm"].to(self.i_bias.dtype).contiguous(), tensors["o"]

    def forward(self, x: torch.Tensor, ctx, call: int) -> torch.Tensor:
        spec, rt, ops, ws = self.spec, self.rt, self.rt.ops, self.rt.workspace
        n, H, dk, dv = x.shape[0], spec.num_heads, spec.key_dim, spec.value_dim
        packed = ws.get("mstate.packed", (n, self.width), rt.dtype)
        ops.gemm(x, self.w_packed, packed)
        gated = ws.get("mstate.gated", (n, H * dv), rt.dtype)
        y = ws.get("mixer.out", (n, spec.hidden_size), rt.dtype)
        plan = ctx.attention_plan
        if plan is not None and plan.decode_only and ops.state_step(
                False, packed, H, H, dk, dv, self.norm, spec.out_norm_eps, ctx.state(call), ctx.token_seq, ctx.cu_seqlens,
                ctx.state_slots, ctx.n_seqs, gated, i_bias=self.i_bias, f_bias=self.f_bias, cap=spec.gate_cap,
                max_state=ctx.state(call, "max"), denom_eps=spec.denom_eps):
            return ops.gemm(gated, self.w_o, y, defer_sum=True) or y
        qk = ws.get("mstate.qk", (n, H, 2, dk), torch.float32)
        vals = ws.get("mstate.vals", (n, H, dv + 1), torch.float32)
        gates = ws.get("mstate.gates", (n, H, 4), torch.float32)
        ops.mlstm_prepare(packed, H, dk, dv, self.i_bias, self.f_bias, spec.gate_cap, ctx.state(call, "max"), ctx.token_seq,
                          ctx.cu_seqlens, ctx.state_slots, ctx.n_seqs, qk, vals, gates)
        raw = ws.get("mstate.raw", (n, H, dv + 1), torch.float32)
        ops.state_scan(qk, vals, gates, ctx.state(call), ctx.cu_seqlens, ctx.state_slots, ctx.n_seqs, H, H, dk, dv + 1, False, raw)
        ops.state_finish(raw, gates, packed, self.gate_offset, self.norm, H, dv, spec.out_norm_eps, ctx.token_seq, gated,
                         shared_weight=False, silu_gate=False, normaliser=True, denom_eps=spec.denom_eps)
        return ops.gemm(gated, self.w_o, y, defer_sum=True) or y


@dataclass(frozen=True)
class ChannelDeltaSpec(PartSpec):
    kind = "channel_delta"
    hidden_size: int = 0
    num_heads: int = 0
    num_kv_heads: int = 0
    key_dim: int = 0
    value_dim: int = 0
    conv_taps: int = 1                  # 1: no convolution (a single tap still scales each channel)
    decay_rank: int = 0                 # rows of W_a1
    gate_rank: int = 0                  # rows of W_g1
    unit_eps: float = 1e-6              # inside the root of a query's or key's length
    out_norm_eps: float = 1e-6          # of the per-head RMS of the output

    @property
    def conv_channels(self) -> int:
        return 2 * self.num_kv_heads * self.key_dim + self.num_heads * self.value_dim


@register_mixer(ChannelDeltaSpec.kind)
class ChannelDelta(Mixer):
    """Packed rows: [q | k | v | b, padded to a multiple of 8 | W_a1 h | W_g1 h, padded to a multiple of 32]. In steps with
    prompt portions the two second matrices are one product against the low-rank columns (block-diagonal, in float32
    rows [decays | gates]); in steps of single tokens the step's kernel makes them itself."""
    spec_class = ChannelDeltaSpec
    accepts_pending_norm = True         # the input is used by one packed product only
    accepts_fold = True                 # the output comes from one product

    @classmethod
    def tensors(cls, spec: ChannelDeltaSpec) -> Dict[str, TensorDecl]:
        hid, H = spec.hidden_size, spec.num_heads
        qk, dk, vd = spec.num_kv_heads * spec.key_dim, H * spec.key_dim, H * spec.value_dim
        return {"q": TensorDecl((qk, hid)), "k": TensorDecl((qk, hid)), "v": TensorDecl((vd, hid)), "b": TensorDecl((H, hid)),
                "q_conv": TensorDecl((qk, spec.conv_taps)), "k_conv": TensorDecl((qk, spec.conv_taps)),
                "v_conv": TensorDecl((vd, spec.conv_taps)),
                "A_log": TensorDecl((H,), init="zeros_normal"), "dt_bias": TensorDecl((dk,), init="zeros_normal"),
                "a1": TensorDecl((spec.decay_rank, hid)), "a2": TensorDecl((dk, spec.decay_rank)),
                "g1": TensorDecl((spec.gate_rank, hid)), "g2": TensorDecl((vd, spec.gate_rank)),
                "norm": TensorDecl((spec.value_dim,), init="ones_normal"), "o": TensorDecl((hid, vd))}

    @classmethod
    def state_shapes(cls, spec: ChannelDeltaSpec):
        shapes = {"state": ((spec.num_heads, spec.value_dim, spec.key_dim), torch.float32)}
        if spec.conv_taps > 1:
            shapes["conv"] = ((spec.conv_taps - 1, spec.conv_channels), None)      # the activation type
        return shapes

    def __init__(self, spec: ChannelDeltaSpec, tensors: Dict[str, torch.Tensor], rt: Runtime, position: Optional[object] = None):
        if min(spec.num_heads, spec.num_kv_heads, spec.key_dim, spec.value_dim, spec.conv_taps, spec.decay_rank, spec.gate_rank) < 1 \
                or spec.num_heads % spec.num_kv_heads:
            raise ValueError(f"channel-wise delta rule: bad sizes {spec}")
        self.spec, self.rt = spec, rt
        hid, H, dk, dv = spec.hidden_size, spec.num_heads, spec.key_dim, spec.value_dim
        ra, rg = spec.decay_rank, spec.gate_rank
        front = _pack(tensors, ("q", "k", "v", "b"), hid, "channel-wise delta rule")
        low = torch.cat([tensors["a1"], tensors["g1"]], dim=0)
        pad = (-low.shape[0]) % 32
        if pad:
            low = torch.cat([low, torch.zeros((pad, hid), dtype=low.dtype, device=low.device)], dim=0)
        self.b_offset, self.low_offset, self.low_width = spec.conv_channels, front.shape[0], low.shape[0]
        self.w_packed = torch.cat([front, low], dim=0).contiguous()
        self.width = self.w_packed.shape[0]
        second = torch.zeros((H * (dk + dv), self.low_width), dtype=low.dtype, device=low.device)
        second[:H * dk, :ra] = tensors["a2"]
        second[H * dk:, ra:ra + rg] = tensors["g2"]
        self.w_second = second.contiguous()
        self.conv_w = torch.cat([tensors["q_conv"], tensors["k_conv"], tensors["v_conv"]], dim=0).contiguous()
        dt = self.conv_w.dtype
        self.a_log, self.dt_bias = tensors["A_log"].to(dt).contiguous(), tensors["dt_bias"].to(dt).contiguous()
        self.a2t, self.g2t = tensors["a2"].to(dt).t().contiguous(), tensors["g2"].to(dt).t().contiguous()
        self.norm, self.w_o = tensors["norm"].to(dt).contiguous(), tensors["o"]

    def first_product(self):
        return self.w_packed.shape[0], self.w_packed.shape[1], False

    def forward(self, x: torch.Tensor, ctx, call: int, fold=None) -> torch.Tensor:
        spec, rt, ops, ws = self.spec, self.rt, self.rt.ops, self.rt.workspace
        n, H, G, dk, dv = x.shape[0], spec.num_heads, spec.num_kv_heads, spec.key_dim, spec.value_dim
        packed = ws.get("mstate.packed", (n, self.width), rt.dtype)
        ops.gemm(x, self.w_packed, packed)
        gated = ws.get("mstate.gated", (n, H * dv), rt.dtype)
        y = ws.get("mixer.out", (n, spec.hidden_size), rt.dtype)
        conv_state = ctx.state(call, "conv") if spec.conv_taps > 1 else None
        plan = ctx.attention_plan
        if plan is not None and plan.decode_only and ops.channel_step(
                packed, H, G, dk, dv, spec.conv_taps, self.b_offset, self.low_offset, self.conv_w, self.a_log, self.dt_bias, self.a2t,
                self.g2t, self.norm, conv_state, ctx.state(call), spec.unit_eps, spec.out_norm_eps, ctx.token_seq, ctx.cu_seqlens,
                ctx.state_slots, ctx.n_seqs, gated):
            return ops.gemm(gated, self.w_o, y, defer_sum=True, fold=fold) or y
        z = ws.get("mstate.z", (n, H * (dk + dv)), torch.float32)
        ops.gemm(packed[:, self.low_offset:self.low_offset + self.low_width], self.w_second, z)
        qk = ws.get("mstate.qk", (n, G, 2, dk), torch.float32)
        vals = ws.get("mstate.vals", (n, H, dv), torch.float32)
        beta = ws.get("mstate.beta", (n, H), torch.float32)
        ops.channel_prepare(packed, H, G, dk, dv, spec.conv_taps, self.b_offset, self.conv_w, self.a_log, self.dt_bias, conv_state,
                            spec.unit_eps, ctx.token_seq, ctx.cu_seqlens, ctx.state_slots, ctx.n_seqs, qk, vals, beta, z)
        raw = ws.get("mstate.raw", (n, H, dv), torch.float32)
        ops.channel_scan(qk, vals, beta, z, ctx.state(call), ctx.cu_seqlens, ctx.state_slots, ctx.n_seqs, H, G, dk, dv, raw)
        ops.state_finish(raw, None, z, H * dk, self.norm, H, dv, spec.out_norm_eps, ctx.token_seq, gated, shared_weight=True,
                         silu_gate=False)
        return ops.gemm(gated, self.w_o, y, defer_sum=True, fold=fold) or y


@dataclass(frozen=True)
class ConstantDecaySpec(PartSpec):
    kind = "constant_decay"
    hidden_size: int = 0
    num_heads: int = 0
    key_dim: int = 0
    value_dim: int = 0
    decay: Tuple[float, ...] = ()       # one per head
    out_norm_eps: float = 1e-6          # of the RMS over all heads' outputs

    @property
    def inner(self) -> int:
        return self.num_heads * self.value_dim


@register_mixer(ConstantDecaySpec.kind)
class ConstantDecay(Mixer):
    spec_class = ConstantDecaySpec
    PACKED = ("q", "k", "v", "g")

    @classmethod
    def tensors(cls, spec: ConstantDecaySpec) -> Dict[str, TensorDecl]:
        hid, qk, vd = spec.hidden_size, spec.num_heads * spec.key_dim, spec.inner
        return {"q": TensorDecl((qk, hid)), "k": TensorDecl((qk, hid)), "v": TensorDecl((vd, hid)), "g": TensorDecl((vd, hid)),
                "norm": TensorDecl((vd,), init="ones_normal"), "o": TensorDecl((hid, vd))}

    @classmethod
    def state_shapes(cls, spec: ConstantDecaySpec):
        return {"state": ((spec.num_heads, spec.value_dim, spec.key_dim), torch.float32)}

    def __init__(self, spec: ConstantDecaySpec, tensors: Dict[str, torch.Tensor], rt: Runtime, position: Optional[object] = None):
        if min(spec.num_heads, spec.key_dim, spec.value_dim) < 1 or len(spec.decay) != spec.num_heads:
            raise ValueError(f"constant decay: bad sizes, or not one decay for each head: {spec}")
        self.spec, self.rt = spec, rt
        self.w_packed = _pack(tensors, self.PACKED, spec.hidden_size, "constant decay")
        self.width = self.w_packed.shape[0]
        self.decay = torch.tensor(spec.decay, dtype=torch.float32, device=rt.device)
        # prompts go chunk by chunk through matrix products where the decays' powers are powers of two's logarithm
        self.chunked = all(0.0 < d <= 1.0 for d in spec.decay)
        self.norm, self.w_o = tensors["norm"].contiguous(), tensors["o"]

    def recur(self, packed: torch.Tensor, base: int, ctx, call: int, beside: Optional[dict] = None):
        """From rows that hold this mixer's projections from column ``base`` on: (the rows that go into the output
        projection, a ``RowSums`` when they are still to be divided by their root mean square, whether ``beside`` ran).
        ``beside``: a query/key norm and cache write on the same rows, to run in the same launch where there is one."""
        spec, rt, ops, ws = self.spec, self.rt, self.rt.ops, self.rt.workspace
        n, H, dk, dv = packed.shape[0], spec.num_heads, spec.key_dim, spec.value_dim
        gated = ws.get("mstate.gated", (n, H * dv), rt.dtype)
        plan = ctx.attention_plan
        if plan is not None and plan.decode_only:
            sums = ws.get("mstate.sums", (n, H), torch.float32)
            if ops.constant_step(packed, base, H, dk, dv, self.decay, self.norm, ctx.state(call), ctx.token_seq, ctx.state_slots, gated,
                                 sums, beside=beside):
                return gated, RowSums(sums, H * dv, spec.out_norm_eps), beside is not None
        raw = ws.get("mstate.raw", (n, H, dv), torch.float32)
        if self.chunked and plan is not None:
            chunks = plan.units(ops.constant_chunk_tokens())
            sums = ws.get("mstate.chunks", (chunks, H, dv, dk), torch.float32)
            ops.constant_chunks(packed, base, H, dk, dv, self.decay, ctx.state(call), ctx.token_seq, ctx.cu_seqlens, ctx.state_slots,
                                ctx.n_seqs, chunks, sums, raw)
        else:
            qk = ws.get("mstate.qk", (n, H, 2, dk), torch.float32)
            vals = ws.get("mstate.vals", (n, H, dv), torch.float32)
            gates = ws.get("mstate.gates", (n, H, 4), torch.float32)
            ops.constant_prepare(packed, base, H, dk, dv, self.decay, ctx.token_seq, qk, vals, gates)
            ops.state_scan(qk, vals, gates, ctx.state(call), ctx.cu_seqlens, ctx.state_slots, ctx.n_seqs, H, H, dk, dv, False, raw)
        ops.row_gate_finish(raw, packed, base + H * (2 * dk + dv), self.norm, spec.out_norm_eps, ctx.token_seq, gated)
        return gated, None, False

    def forward(self, x: torch.Tensor, ctx, call: int) -> torch.Tensor:
        spec, rt, ops, ws = self.spec, self.rt, self.rt.ops, self.rt.workspace
        n = x.shape[0]
        packed = ws.get("mstate.packed", (n, self.width), rt.dtype)
        ops.gemm(x, self.w_packed, packed)
        gated, sums, _ = self.recur(packed, 0, ctx, call)
        if sums is not None:
            whole = ws.get("mstate.scaled", (n, spec.inner), rt.dtype)
            ops.scale_rows(gated, sums.sums, sums.sums.shape[1], sums.eps, whole)
            gated = whole
        y = ws.get("mixer.out", (n, spec.hidden_size), rt.dtype)
        return ops.gemm(gated, self.w_o, y, defer_sum=True) or y


@dataclass(frozen=True)
class GatedLinearSpec(PartSpec):
    kind = "gated_linear"
    hidden_size: int = 0
    num_heads: int = 0
    key_dim: int = 0
    value_dim: int = 0
    decay_rank: int = 0                 # rows of W_a1
    tau: float = 1.0                    # a channel's decay is sigmoid(z)^(1 / tau)
    out_norm_eps: float = 1e-6          # of the per-head RMS of the output
    out_scale: float = 1.0              # on the gated rows (it goes into the norm's weight)

    @property
    def inner(self) -> int:
        return self.num_heads * self.value_dim


@register_mixer(GatedLinearSpec.kind)
class GatedLinear(Mixer):
    """Packed rows: [q | k | v | g, padded to a multiple of 8 | W_a1 h, padded to a multiple of 32]. In steps with prompt
    portions W_a2 is one product with float32 rows; in steps of single tokens the step's kernel makes them itself."""
    spec_class = GatedLinearSpec
    accepts_pending_norm = True         # the input is used by one packed product only
    accepts_fold = True                 # the output comes from one product
    PACKED = ("q", "k", "v", "g")

    @classmethod
    def tensors(cls, spec: GatedLinearSpec) -> Dict[str, TensorDecl]:
        hid, qk, vd = spec.hidden_size, spec.num_heads * spec.key_dim, spec.inner
        return {"q": TensorDecl((qk, hid)), "k": TensorDecl((qk, hid)), "v": TensorDecl((vd, hid)), "g": TensorDecl((vd, hid)),
                "a1": TensorDecl((spec.decay_rank, hid)), "a2": TensorDecl((qk, spec.decay_rank)),
                "a2_bias": TensorDecl((qk,), init="zeros_normal"), "norm": TensorDecl((spec.value_dim,), init="ones_normal"),
                "o": TensorDecl((hid, vd))}

    @classmethod
    def state_shapes(cls, spec: GatedLinearSpec):
        return {"state": ((spec.num_heads, spec.value_dim, spec.key_dim), torch.float32)}

    def __init__(self, spec: GatedLinearSpec, tensors: Dict[str, torch.Tensor], rt: Runtime, position: Optional[object] = None):
        if min(spec.num_heads, spec.key_dim, spec.value_dim, spec.decay_rank) < 1 or not spec.tau > 0:
            raise ValueError(f"gated linear attention: bad sizes {spec}")
        self.spec, self.rt = spec, rt
        hid, qk = spec.hidden_size, spec.num_heads * spec.key_dim
        front = _pack(tensors, self.PACKED, hid, "gated linear attention")
        pad = (-spec.decay_rank) % 32
        low, a2 = tensors["a1"], tensors["a2"]
        self.a2t = a2.t().contiguous()
        if pad:
            low = torch.cat([low, torch.zeros((pad, hid), dtype=low.dtype, device=low.device)], dim=0)
            a2 = torch.cat([a2, torch.zeros((qk, pad), dtype=a2.dtype, device=a2.device)], dim=1)
        self.low_offset, self.low_width = front.shape[0], low.shape[0]
        self.w_packed = torch.cat([front, low], dim=0).contiguous()
        self.width = self.w_packed.shape[0]
        self.w_second = a2.contiguous()
        self.a2_bias = tensors["a2_bias"].to(torch.float32).contiguous()
        # float32: the constant on the output costs no rounding of its own
        self.norm = (tensors["norm"].to(torch.float32) * spec.out_scale).contiguous()
        self.w_o = tensors["o"]

    def first_product(self):
        return self.w_packed.shape[0], self.w_packed.shape[1], False

    def recur(self, packed: torch.Tensor, base: int, ctx, call: int, out: torch.Tensor, beside: Optional[dict] = None) -> bool:
        """From rows that hold this mixer's projections from column ``base`` on: the gated rows that go into the output
        projection, in ``out`` [n, heads * value_dim]. ``beside``: a convolution and cache write of a softmax mixer on the same
        rows (``Attention.conv_store_args``), to run in the same launch where there is one; returns whether it ran."""
        spec, rt, ops, ws = self.spec, self.rt, self.rt.ops, self.rt.workspace
        n, H, dk, dv = packed.shape[0], spec.num_heads, spec.key_dim, spec.value_dim
        plan = ctx.attention_plan
        if plan is not None and plan.decode_only:
            ran = ops.gated_linear_step(packed, base, base + self.low_offset, H, dk, dv, self.a2t, self.a2_bias, spec.tau, self.norm,
                                        spec.out_norm_eps, ctx.state(call), ctx.token_seq, ctx.state_slots, out, beside=beside)
            if ran:
                return ran == 2
        z = ws.get("mstate.z", (n, H * dk), torch.float32)
        low = base + self.low_offset
        ops.gemm(packed[:, low:low + self.low_width], self.w_second, z)
        raw = ws.get("mstate.raw", (n, H, dv), torch.float32)
        chunks = plan.units(ops.gated_linear_chunk_tokens()) if plan is not None else n
        sums = ws.get("mstate.chunks", (chunks, H, dv, dk), torch.float32)
        decays = ws.get("mstate.decays", (chunks, H, dk), torch.float32)
        ops.gated_linear_chunks(packed, base, H, dk, dv, z, self.a2_bias, spec.tau, ctx.state(call), ctx.token_seq, ctx.cu_seqlens,
                                ctx.state_slots, ctx.n_seqs, chunks, sums, decays, raw)
        ops.state_finish(raw, None, packed, base + H * (2 * dk + dv), self.norm, H, dv, spec.out_norm_eps, ctx.token_seq, out,
                         shared_weight=True, silu_gate=True)
        return False

    def forward(self, x: torch.Tensor, ctx, call: int, fold=None) -> torch.Tensor:
        spec, rt, ops, ws = self.spec, self.rt, self.rt.ops, self.rt.workspace
        n = x.shape[0]
        packed = ws.get("mstate.packed", (n, self.width), rt.dtype)
        ops.gemm(x, self.w_packed, packed)
        gated = ws.get("mstate.gated", (n, spec.inner), rt.dtype)
        self.recur(packed, 0, ctx, call, gated)
        y = ws.get("mixer.out", (n, spec.hidden_size), rt.dtype)
        return ops.gemm(gated, self.w_o, y, defer_sum=True, fold=fold) or y
