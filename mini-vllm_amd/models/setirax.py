"""Setirax as a plan of parts.

Every layer is a post-norm block: its sublayers read the residual itself and only their outputs are normed. The mixer is the
sum of two mixers side by side (``parts/parallel.py``: softmax attention over a window on convolved, rotated, unit-normed
queries and keys with capped scores, beside gated linear attention with a decay per key channel), the real-gated linear
recurrent unit (``parts/recurrent_unit.py``), or attention over a latent without positions, with a window and a sink
(``parts/latent_attention.py``). The feed-forward is two projections with squared ReLU and biases (``parts/mlp.py``); a layer
may have none. A layer with ``weights_of`` runs another layer's parts again, as a call with a cache and state of its own. The
embedding's table is the output head; its logits are capped.

Tensor names on disk: ``embed``, ``final.norm``; per layer i with tensors of its own ``l<i>.norm1``, ``.norm2``,
``l<i>.mix.left.{q,k,v,q.conv,k.conv,v.conv,o}`` and ``l<i>.mix.right.{q,k,v,g,o,norm,a1,a2,a2.b}``, or
``l<i>.mix.{x,x.b,y,y.b,conv,conv.b,ra,ra.b,ri,ri.b,lam,o}``, or ``l<i>.mix.{q,dkv,dkv.norm,uk,uv,sink,o}``; and
``l<i>.mlp.{up,up.b,down,down.b}``.
"""
from __future__ import annotations

from typing import Dict, FrozenSet, List

from ..config.model_config import SetiraxConfig, SetiraxLayer
from ..parts.attention import AttentionSpec
from ..parts.block import PostNormBlock, PostNormBlockSpec
from ..parts.io import CappedHeadSpec
from ..parts.latent_attention import LatentAttentionSpec
from ..parts.matrix_state import GatedLinearSpec
from ..parts.mlp import SquaredReLUSpec
from ..parts.norm import RMSNormSpec
from ..parts.parallel import ParallelSumSpec
from ..parts.plan import Call, EmbeddingSpec, HeadSpec, LayerPlan, ModelPlan, TensorLocation
from ..parts.recurrent_unit import RecurrentUnitSpec
from ..parts.rope import RotarySpec
from .registry import Architecture, register_architecture


def _owners(config: SetiraxConfig) -> List[int]:
    """Config indices of the layers that own tensors, in the plan's order."""
    return [i for i, l in enumerate(config.layers) if l.weights_of is None]


def _left_of(window):
    """The configuration counts the query's own position into the window, the parts count the positions left of it."""
    return None if window is None else window - 1


def _mixer(l: SetiraxLayer, hid: int, eps: float):
    if l.type == "rglru":
        return RecurrentUnitSpec(hidden_size=hid, width=l.unit.width, blocks=l.unit.blocks, conv_taps=l.unit.conv)
    if l.type == "latent_attention":
        c = l.latent
        return LatentAttentionSpec(hidden_size=hid, num_heads=c.heads, plain_dim=c.dim, rot_dim=0, value_dim=c.vdim, q_rank=0,
                                   kv_rank=c.kv_rank, scale=c.scale, norm_eps=eps, window=_left_of(c.window), sink=True)
    a, b = l.left, l.right
    rope = RotarySpec(rotary_dim=a.rot_dims, theta=a.rot_base, by_wavelength=a.rot_scaling) if a.rot_dims else None
    return ParallelSumSpec(
        hidden_size=hid,
        left=AttentionSpec(hidden_size=hid, num_heads=a.heads, num_kv_heads=a.kv_heads, head_dim=a.dim, value_dim=a.vdim, scale=a.scale,
                           qk_norm_eps=eps, window=_left_of(a.window), position=rope, unit_norm_after_rotation=True, softcap=a.softcap,
                           conv_taps=a.conv, out_scale=l.left_scale),
        right=GatedLinearSpec(hidden_size=hid, num_heads=b.heads, key_dim=b.dim, value_dim=b.vdim, decay_rank=b.rank, tau=b.tau,
                              out_norm_eps=eps, out_scale=l.right_scale))


def setirax_plan(config: SetiraxConfig) -> ModelPlan:
    # (a size that neither config.json nor a loader has filled in is an error here)
    config = config.completed()
    hid, eps = config.hidden_size, config.norm_eps
    norm = RMSNormSpec(size=hid, eps=eps)
    index_of: Dict[int, int] = {i: k for k, i in enumerate(_owners(config))}
    layers, calls = [], []
    for i, l in enumerate(config.layers):
        calls.append(Call(layer=index_of[config.owner_of(i)]))
        if l.weights_of is not None:
            continue
        ffn = None if l.ff is None else SquaredReLUSpec(hidden_size=hid, intermediate_size=l.ff)
        slots = PostNormBlock.slots_for(ffn is not None)
        layers.append(LayerPlan(block=PostNormBlockSpec(), mixer=_mixer(l, hid, eps), ffn=ffn, norms=tuple((s, norm) for s in slots)))
    head = (HeadSpec(vocab_size=config.vocab_size, hidden_size=hid, tied=True) if config.logit_softcap is None
            else CappedHeadSpec(vocab_size=config.vocab_size, hidden_size=hid, cap=config.logit_softcap))
    plan = ModelPlan(hidden_size=hid, vocab_size=config.vocab_size, max_positions=config.max_position_embeddings,
                     embedding=EmbeddingSpec(vocab_size=config.vocab_size, hidden_size=hid, scale=1.0),
                     layers=tuple(layers), calls=tuple(calls), final_norm=norm, head=head)
    plan.validate()
    return plan


_SIDE_NAMES = {"q_conv": "q.conv", "k_conv": "k.conv", "v_conv": "v.conv", "a2_bias": "a2.b"}
_UNIT_NAMES = {"x_bias": "x.b", "y_bias": "y.b", "conv_bias": "conv.b", "ra_bias": "ra.b", "ri_bias": "ri.b"}
_LATENT_NAMES = {"dkv_norm": "dkv.norm"}
_FFN_NAMES = {"up_bias": "up.b", "down_bias": "down.b"}


def setirax_tensor_name(config: SetiraxConfig, loc: TensorLocation) -> str:
    if loc.layer is None:
        return {"embedding": "embed", "head": "embed", "final_norm": "final.norm"}[loc.role]
    owner = _owners(config)[loc.layer]
    prefix = f"l{owner}."
    if loc.role == "mixer":
        kind = config.layers[owner].type
        if kind == "parallel":
            side, name = loc.name.split(".", 1)
            return f"{prefix}mix.{side}.{_SIDE_NAMES.get(name, name)}"
        names = _UNIT_NAMES if kind == "rglru" else _LATENT_NAMES
        return prefix + "mix." + names.get(loc.name, loc.name)
    if loc.role == "ffn":
        return prefix + "mlp." + _FFN_NAMES.get(loc.name, loc.name)
    if loc.role.startswith("norm."):
        return prefix + loc.role[len("norm."):]
    raise KeyError(loc)


def setirax_ignorable(config: SetiraxConfig) -> FrozenSet[str]:
    # a layer without a feed-forward may still store the norm behind it
    return frozenset(f"l{i}.norm2" for i, l in enumerate(config.layers) if l.ff is None)


def setirax_complete(config: SetiraxConfig, source) -> SetiraxConfig:
    """The configuration with what only the stored tensors state: the decay's rank is the rows of ``a1``; the other sizes may
    be left out of config.json too."""
    names = set(source.names())
    return config.completed(lambda name: tuple(source.shape(name)) if name in names else None)


SETIRAX = register_architecture(Architecture(
    name=SetiraxConfig.architecture,
    config_class=SetiraxConfig,
    plan=setirax_plan,
    tensor_name=setirax_tensor_name,
    ignorable=setirax_ignorable,
    complete=setirax_complete,
))
