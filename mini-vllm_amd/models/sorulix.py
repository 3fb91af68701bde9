"""Sorulix as a plan of parts.

Every layer is a pre-norm block whose norms have weights stored around zero. The mixer is two mixers side by side
(``parts/parallel.py``): softmax attention behind a norm over whole query and key rows, with a query temperature, capped
scores, a distance bias per head and a sink in the denominator (``parts/attention.py``), beside linear attention with a
constant decay per head (``parts/matrix_state.py``); or the gated delta rule with a decay per head and key channel
(``parts/matrix_state.py``). The feed-forward is the clamped gated pair with biases (``parts/mlp.py``); a layer may have
none. A run of layers may be run several times in a row with the same weights: each time is a call of its own, with a
cache and state of its own, entered through ``parts/entry.py``. The embedding's table is the output head.

Tensor names on disk: ``embed``, ``loop.step``, ``final.norm``; per layer i ``l<i>.norm1``, ``.norm2``,
``l<i>.mix.left.{q,k,v,q.norm,k.norm,o,out}`` and ``l<i>.mix.right.{q,k,v,g,norm,o,out}``, or
``l<i>.mix.{q,k,v,q.conv,k.conv,v.conv,b,A_log,dt_bias,a1,a2,g1,g2,norm,o}``, ``l<i>.mlp.{gate,up,down}`` and their ``.b``.
"""
from __future__ import annotations

from typing import FrozenSet

from ..config.model_config import SorulixConfig
from ..parts.attention import AttentionSpec
from ..parts.block import PreNormBlock, PreNormBlockSpec
from ..parts.entry import PassEntrySpec
from ..parts.matrix_state import ChannelDeltaSpec, ConstantDecaySpec
from ..parts.mlp import ClampedGLUSpec
from ..parts.norm import RMSNormSpec
from ..parts.parallel import ParallelMixerSpec
from ..parts.plan import Call, EmbeddingSpec, HeadSpec, LayerPlan, ModelPlan, TensorLocation
from .registry import Architecture, register_architecture

UNIT_EPS = 1e-6           # inside the root of a query's or key's length
GATE_SLOPE = 1.702        # the feed-forward's gate is g * sigmoid(GATE_SLOPE * g)


def _calls(config: SorulixConfig):
    n = len(config.layers)
    if config.loop is None:
        return [Call(layer=i) for i in range(n)]
    start, stop, times = config.loop
    calls = [Call(layer=i) for i in range(start)]
    for t in range(times):
        calls += [Call(layer=i, enters_pass=t if i == start else None) for i in range(start, stop)]
    return calls + [Call(layer=i) for i in range(stop, n)]


def sorulix_plan(config: SorulixConfig) -> ModelPlan:
    # (a size that neither config.json nor a loader has filled in is an error here)
    config = config.completed()
    hid, eps = config.hidden_size, config.norm_eps
    norm = RMSNormSpec(size=hid, eps=eps, unit_offset=True)
    layers = []
    for l in config.layers:
        if l.type == "parallel":
            a, b = l.left, l.right
            mixer = ParallelMixerSpec(
                hidden_size=hid, out_norm_eps=eps,
                left=AttentionSpec(hidden_size=hid, num_heads=a.heads, num_kv_heads=a.kv_heads, head_dim=a.dim, value_dim=a.vdim,
                                   scale=a.scale, qk_norm_eps=eps, row_norm=True, query_temperature=a.q_temp, softcap=a.softcap,
                                   distance_bias=True, sink=True),
                right=ConstantDecaySpec(hidden_size=hid, num_heads=b.heads, key_dim=b.dim, value_dim=b.vdim, decay=b.decay,
                                        out_norm_eps=eps))
        else:
            m = l.delta
            mixer = ChannelDeltaSpec(hidden_size=hid, num_heads=m.heads, num_kv_heads=m.kv_heads, key_dim=m.dim, value_dim=m.vdim,
                                     conv_taps=m.conv, decay_rank=m.decay_rank, gate_rank=m.gate_rank, unit_eps=UNIT_EPS,
                                     out_norm_eps=eps)
        ffn = None if l.ff is None else ClampedGLUSpec(hidden_size=hid, intermediate_size=l.ff, limit=l.limit, slope=GATE_SLOPE,
                                                       bias=True)
        slots = PreNormBlock.slots_for(ffn is not None)
        layers.append(LayerPlan(block=PreNormBlockSpec(), mixer=mixer, ffn=ffn, norms=tuple((s, norm) for s in slots)))
    plan = ModelPlan(hidden_size=hid, vocab_size=config.vocab_size, max_positions=config.max_position_embeddings,
                     embedding=EmbeddingSpec(vocab_size=config.vocab_size, hidden_size=hid, scale=1.0),
                     layers=tuple(layers), calls=tuple(_calls(config)), final_norm=norm,
                     head=HeadSpec(vocab_size=config.vocab_size, hidden_size=hid, tied=True),
                     entry=None if config.loop is None else PassEntrySpec(hidden_size=hid, times=config.loop[2]))
    plan.validate()
    return plan


_NORM_SLOTS = {"mixer": "norm1", "ffn": "norm2"}
_DELTA_NAMES = {"q_conv": "q.conv", "k_conv": "k.conv", "v_conv": "v.conv"}
_LEFT_NAMES = {"q_norm": "q.norm", "k_norm": "k.norm"}
_FFN_NAMES = {"gate_bias": "gate.b", "up_bias": "up.b", "down_bias": "down.b"}


def sorulix_tensor_name(config: SorulixConfig, loc: TensorLocation) -> str:
    if loc.layer is None:
        names = {"embedding": "embed", "head": "embed", "final_norm": "final.norm", "entry": "loop.step"}
        return names[loc.role]
    prefix = f"l{loc.layer}."
    if loc.role == "mixer":
        if config.layers[loc.layer].type == "channel_delta":
            return prefix + "mix." + _DELTA_NAMES.get(loc.name, loc.name)
        if loc.name in ("left_out", "right_out"):
            return prefix + "mix." + loc.name.replace("_", ".")
        side, name = loc.name.split(".", 1)
        return f"{prefix}mix.{side}.{_LEFT_NAMES.get(name, name)}"
    if loc.role == "ffn":
        return prefix + "mlp." + _FFN_NAMES.get(loc.name, loc.name)
    if loc.role.startswith("norm."):
        return prefix + _NORM_SLOTS[loc.role[len("norm."):]]
    raise KeyError(loc)


def sorulix_ignorable(config: SorulixConfig) -> FrozenSet[str]:
    # a layer without a feed-forward may still store the norm in front of it, a model without a loop its step vectors
    names = {f"l{i}.norm2" for i, l in enumerate(config.layers) if l.ff is None}
    return frozenset(names | (set() if config.loop is not None else {"loop.step"}))


def sorulix_complete(config: SorulixConfig, source) -> SorulixConfig:
    """The configuration with what only the stored tensors state: the ranks are the rows of ``a1`` and ``g1``; the other
    sizes may be left out of config.json too."""
    names = set(source.names())
    return config.completed(lambda name: tuple(source.shape(name)) if name in names else None)


SORULIX = register_architecture(Architecture(
    name=SorulixConfig.architecture,
    config_class=SorulixConfig,
    plan=sorulix_plan,
    tensor_name=sorulix_tensor_name,
    ignorable=sorulix_ignorable,
    complete=sorulix_complete,
))
