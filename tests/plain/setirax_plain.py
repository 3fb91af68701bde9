"""A plain, slow Setirax forward pass: whole sequences, no cache, one function per mechanism.

It imports nothing from the engine and runs on the CPU in the dtype of its inputs (tests use
float64). ``weights`` maps the names on disk (``l0.mix.left.q.conv``, ``l1.mlp.up.b`` ...) to tensors;
``cfg`` is the raw dictionary of ``config.json``.

Notation: n tokens of one sequence at positions first..first+n-1; matrices are stored [out, in] and
applied as ``x @ W.T``. Every mixer also takes and returns its state (recurrent states, kept inputs of
the convolutions, and for the softmax mixers all keys so far), so that a sequence can be fed in pieces.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional, Tuple

import torch

GATE_POWER = 8.0         # the gated unit's decay is exp(-GATE_POWER r softplus(lam))

Tensors = Dict[str, torch.Tensor]


def keep(t: torch.Tensor) -> torch.Tensor:
    return t


def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def rms_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    return unit_rms(x, eps) * weight


def capped(x: torch.Tensor, cap: Optional[float]) -> torch.Tensor:
    return x if cap is None else cap * torch.tanh(x / cap)


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def short_conv(x: torch.Tensor, taps: torch.Tensor, before: Optional[torch.Tensor] = None) -> Tuple[torch.Tensor, torch.Tensor]:
    """Causal convolution along time, channel by channel: x [n, c], taps [c, T], the last column the current token's;
    ``before`` [T-1, c] the inputs in front of x. Returns (y [n, c], the last T-1 inputs)."""
    n, c = x.shape
    T = taps.shape[1]
    ext = torch.cat([torch.zeros(T - 1, c, dtype=x.dtype) if before is None else before, x], dim=0)
    y = torch.zeros_like(x)
    for j in range(T):
        y = y + ext[j:j + n] * taps[:, j]
    return y, ext[n:]


# ---------------------------------------------------------------------------------------
# rotation
# ---------------------------------------------------------------------------------------
def frequencies(dims: int, base: float, scaling: Optional[dict]) -> torch.Tensor:
    """Radians a position for each pair. With ``scaling``: pairs whose wavelength is short against ``original`` keep their
    frequency, long ones are slowed by ``factor``, and those between are blended linearly in original / wavelength."""
    out = []
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if scaling:
            turns = scaling["original"] * f / (2.0 * math.pi)            # original / wavelength
            if turns < scaling["low"]:
                f = f / scaling["factor"]
            elif turns <= scaling["high"]:
                s = (turns - scaling["low"]) / (scaling["high"] - scaling["low"])
                f = (1.0 - s) * f / scaling["factor"] + s * f
        out.append(f)
    return torch.tensor(out, dtype=torch.float64)


def rotate(x: torch.Tensor, first: int, rot: dict) -> torch.Tensor:
    """x [n, heads, d] at positions first, first + 1, ...: channel i < dims / 2 pairs with i + dims / 2."""
    dims = rot["dims"]
    f = frequencies(dims, rot["base"], rot.get("scaling"))
    a = torch.arange(first, first + x.shape[0], dtype=torch.float64)[:, None] * f
    c, s = torch.cos(a).to(x.dtype)[:, None], torch.sin(a).to(x.dtype)[:, None]
    u, v = x[..., :dims // 2], x[..., dims // 2:dims]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., dims:]], dim=-1)


# ---------------------------------------------------------------------------------------
# softmax over a window
# ---------------------------------------------------------------------------------------
def windowed(scores: torch.Tensor, first: int, size: Optional[int]) -> torch.Tensor:
    """scores [n, m] of queries at positions first .. against keys 0 .. m-1; -inf where query i does not see key j, that
    is unless 0 <= i - j < size."""
    i = torch.arange(first, first + scores.shape[0])[:, None]
    j = torch.arange(scores.shape[1])[None, :]
    seen = j <= i
    if size is not None:
        seen = seen & (i - j < size)
    return torch.where(seen, scores, torch.full_like(scores, -math.inf))


def sink_softmax(scores: torch.Tensor, sink: Optional[torch.Tensor]) -> torch.Tensor:
    """exp(s_j) / (exp(sink) + sum_j exp(s_j)) along the last axis; without a sink an ordinary softmax."""
    top = scores.max(-1, keepdim=True).values
    if sink is not None:
        top = torch.maximum(top, sink)
    e = torch.exp(scores - top)
    den = e.sum(-1, keepdim=True)
    return e / (den if sink is None else den + torch.exp(sink - top))


def window_size(m: dict) -> Optional[int]:
    return m["mask"]["size"] if m.get("mask") else None


def left_mixer(h: torch.Tensor, w: Tensors, p: str, m: dict, eps: float, state: Optional[dict] = None, rnd=keep):
    """Attention on convolved projections, rotated, then divided by their root mean square per head."""
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    n = h.shape[0]
    first = 0 if state is None else state["k"].shape[0]
    new, proj = {}, {}
    for name in ("q", "k", "v"):
        proj[name], new["conv." + name] = short_conv(rnd(h @ w[p + name].T), w[p + name + ".conv"],
                                                     None if state is None else state["conv." + name])
    q, k = proj["q"].view(n, H, d), proj["k"].view(n, G, d)
    if m.get("rot"):
        q, k = rotate(q, first, m["rot"]), rotate(k, first, m["rot"])
    q, k, v = rnd(unit_rms(q, eps)), rnd(unit_rms(k, eps)), rnd(proj["v"]).view(n, G, dv)
    if state is not None:
        k, v = torch.cat([state["k"], k]), torch.cat([state["v"], v])
    new["k"], new["v"] = k, v
    out = torch.empty(n, H, dv, dtype=h.dtype)
    for head in range(H):
        g = head // (H // G)
        s = windowed(capped((q[:, head] @ k[:, g].T) * m["scale"], m.get("softcap")), first, window_size(m))
        out[:, head] = sink_softmax(s, None) @ v[:, g]
    return rnd(rnd(out.reshape(n, H * dv)) @ w[p + "o"].T), new


def latent_mixer(h: torch.Tensor, w: Tensors, p: str, m: dict, eps: float, state: Optional[dict] = None, rnd=keep):
    """Attention whose keys and values are linear maps of a normed latent; only the latent is kept."""
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    n = h.shape[0]
    first = 0 if state is None else state["c"].shape[0]
    q = rnd(h @ w[p + "q"].T).view(n, H, d)
    c = rnd(rms_norm(rnd(h @ w[p + "dkv"].T), w[p + "dkv.norm"], eps))
    if state is not None:
        c = torch.cat([state["c"], c])
    k, v = (c @ w[p + "uk"].T).view(-1, H, d), (c @ w[p + "uv"].T).view(-1, H, dv)
    out = torch.empty(n, H, dv, dtype=h.dtype)
    for head in range(H):
        s = windowed((q[:, head] @ k[:, head].T) * m["scale"], first, window_size(m))
        out[:, head] = sink_softmax(s, w[p + "sink"][head]) @ v[:, head]
    return rnd(rnd(out.reshape(n, H * dv)) @ w[p + "o"].T), {"c": c}


# ---------------------------------------------------------------------------------------
# gated linear attention: a matrix state with a decay per key channel
# ---------------------------------------------------------------------------------------
def gated_linear_scan(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, alpha: torch.Tensor, state: Optional[torch.Tensor] = None
                      ) -> Tuple[torch.Tensor, torch.Tensor]:
    """One head. q, k, alpha [n, dk]; v [n, dv]; S [dk, dv] <- diag(alpha) S + k v^T;  o = S^T q."""
    S = torch.zeros(k.shape[1], v.shape[1], dtype=k.dtype) if state is None else state.clone()
    out = torch.empty_like(v)
    for t in range(k.shape[0]):
        S = alpha[t][:, None] * S + k[t][:, None] * v[t][None, :]
        out[t] = q[t] @ S
    return out, S


def channel_decay(h: torch.Tensor, w: Tensors, p: str, tau: float, rnd=keep) -> torch.Tensor:
    """sigmoid(z)^(1 / tau) with z = W_a2 (W_a1 h) + bias."""
    z = rnd(h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "a2.b"]
    return torch.exp(torch.nn.functional.logsigmoid(z) / tau)


def right_mixer(h: torch.Tensor, w: Tensors, p: str, m: dict, eps: float, state: Optional[dict] = None, rnd=keep):
    H, d, dv, n = m["heads"], m["dim"], m["vdim"], h.shape[0]
    q = rnd(h @ w[p + "q"].T).view(n, H, d) * d ** -0.5
    k, v = rnd(h @ w[p + "k"].T).view(n, H, d), rnd(h @ w[p + "v"].T).view(n, H, dv)
    alpha = channel_decay(h, w, p, m["tau"], rnd).view(n, H, d)
    out = torch.empty(n, H, dv, dtype=h.dtype)
    states = []
    for head in range(H):
        out[:, head], S = gated_linear_scan(q[:, head], k[:, head], v[:, head], alpha[:, head], None if state is None else state["S"][head])
        states.append(S)
    g = rnd(h @ w[p + "g"].T)
    y = rms_norm(out, w[p + "norm"], eps).reshape(n, H * dv) * (g * torch.sigmoid(g))
    return rnd(rnd(y) @ w[p + "o"].T), {"S": torch.stack(states)}


def parallel_mixer(h, w, p, m, eps, state=None, rnd=keep):
    state = state or {}
    left, new_left = left_mixer(h, w, p + "left.", m["left"], eps, state.get("left"), rnd)
    right, new_right = right_mixer(h, w, p + "right.", m["right"], eps, state.get("right"), rnd)
    return m["left_scale"] * left + m["right_scale"] * right, {"left": new_left, "right": new_right}


# ---------------------------------------------------------------------------------------
# the real-gated linear recurrent unit
# ---------------------------------------------------------------------------------------
def block_diagonal(u: torch.Tensor, matrices: torch.Tensor, bias: torch.Tensor) -> torch.Tensor:
    """u [n, W] in B equal parts, part b times matrices[b] [out, in], plus bias[b]."""
    B, size = bias.shape
    parts = [u[:, b * size:(b + 1) * size] @ matrices[b].T + bias[b] for b in range(B)]
    return torch.cat(parts, dim=1)


def linear_recurrence(a: torch.Tensor, x: torch.Tensor, state: Optional[torch.Tensor] = None) -> Tuple[torch.Tensor, torch.Tensor]:
    """Channel by channel: S_t = a_t S_{t-1} + x_t. a, x [n, W]; state [W]. Returns (all S_t, the last)."""
    S = torch.zeros(a.shape[1], dtype=a.dtype) if state is None else state
    out = torch.empty_like(x)
    for t in range(a.shape[0]):
        S = a[t] * S + x[t]
        out[t] = S
    return out, S


def rglru_mixer(h: torch.Tensor, w: Tensors, p: str, m: dict, eps: float, state: Optional[dict] = None, rnd=keep):
    state = state or {}
    y = gelu_tanh(rnd(h @ w[p + "y"].T + w[p + "y.b"]))
    conv, before = short_conv(rnd(h @ w[p + "x"].T + w[p + "x.b"]), w[p + "conv"], state.get("conv"))
    u = rnd(conv + w[p + "conv.b"])
    r = torch.sigmoid(block_diagonal(u, w[p + "ra"], w[p + "ra.b"]))
    i = torch.sigmoid(block_diagonal(u, w[p + "ri"], w[p + "ri.b"]))
    log_a = -GATE_POWER * r * torch.nn.functional.softplus(w[p + "lam"])
    S, last = linear_recurrence(torch.exp(log_a), torch.sqrt(-torch.expm1(2.0 * log_a)) * i * u, state.get("S"))
    return rnd(rnd(S * y) @ w[p + "o"].T), {"conv": before, "S": last}


MIXERS = {"parallel": parallel_mixer, "rglru": rglru_mixer, "latent_attention": latent_mixer}


# ---------------------------------------------------------------------------------------
# feed-forward, order of layers, output
# ---------------------------------------------------------------------------------------
def feed_forward(h: torch.Tensor, w: Tensors, p: str, rnd=keep) -> torch.Tensor:
    z = rnd(h @ w[p + "up"].T + w[p + "up.b"])
    return rnd(rnd(torch.relu(z) ** 2) @ w[p + "down"].T + w[p + "down.b"])


def weights_layer(cfg: dict, i: int) -> int:
    """The layer whose tensors layer i uses."""
    while cfg["layers"][i].get("weights_of") is not None:
        i = cfg["layers"][i]["weights_of"]
    return i


def forward(cfg: dict, w: Tensors, tokens: List[int], state: Optional[list] = None, rnd=keep, keep_layers: bool = False):
    """(logits [n, vocab], states of the layers[, residual after every layer]). ``rnd`` rounds what an engine with 16-bit
    activations would store; the residual sum is never rounded."""
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.tensor(tokens, dtype=torch.long)].clone()
    new, kept = [], []
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{weights_layer(cfg, i)}."
        y, s = MIXERS[layer["type"]](rnd(x), w, p + "mix.", layer["mixer"], eps, None if state is None else state[i], rnd)
        new.append(s)
        x = x + rms_norm(y, w[p + "norm1"], eps)
        if layer.get("mlp") is not None:
            x = x + rms_norm(feed_forward(rnd(x), w, p + "mlp.", rnd), w[p + "norm2"], eps)
        kept.append(x)
    logits = capped(rnd(rms_norm(x, w["final.norm"], eps)) @ w["embed"].T, cfg.get("logit_softcap"))
    return (logits, new, kept) if keep_layers else (logits, new)


def round_to_bfloat16(t: torch.Tensor) -> torch.Tensor:
    return t.to(torch.bfloat16).to(t.dtype)
