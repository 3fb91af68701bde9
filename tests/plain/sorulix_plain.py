"""A plain, slow Sorulix forward pass: whole sequences, no cache, one function per mechanism.

It imports nothing from the engine and runs on the CPU in the dtype of its inputs (tests use
float64). ``weights`` maps the names on disk (``l0.mix.left.q``, ``l1.mlp.gate.b`` ...) to tensors;
``cfg`` is the raw dictionary of ``config.json``.

Notation: n tokens of one sequence at positions 0..n-1; matrices are stored [out, in] and applied
as ``x @ W.T``. Every recurrent function also takes and returns its state, so that a sequence can be
fed in pieces; the softmax mixer takes the keys and values in front of the piece.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional, Tuple

import torch

UNIT_EPS = 1e-6          # inside the root of a query's or key's length
GATE_SLOPE = 1.702       # of the feed-forward's gate

Tensors = Dict[str, torch.Tensor]


def rms_norm(x: torch.Tensor, weight: torch.Tensor, eps: float, around_zero: bool = False) -> torch.Tensor:
    y = x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)
    return y * (1.0 + weight) if around_zero else y * weight


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


# ---------------------------------------------------------------------------------------
# softmax attention: whole-row norm, query temperature, soft cap, distance bias, sink
# ---------------------------------------------------------------------------------------
def query_temperature(position: int, coef: float, every: int) -> float:
    return 1.0 + coef * math.log((position + 1) // every + 1.0)


def distance_slope(head: int, heads: int) -> float:
    return 2.0 ** (-8.0 * (head + 1) / heads)


def capped(score: torch.Tensor, cap: Optional[float]) -> torch.Tensor:
    return score if cap is None else cap * torch.tanh(score / cap)


def sink_softmax(scores: torch.Tensor) -> torch.Tensor:
    """exp(s_j) / (1 + sum_j exp(s_j)) along the last axis: a softmax with one more score, 0, that has no value."""
    top = torch.clamp(scores.max(-1, keepdim=True).values, min=0.0)
    e = torch.exp(scores - top)
    return e / (torch.exp(-top) + e.sum(-1, keepdim=True))


def attention_scores(q: torch.Tensor, k: torch.Tensor, first: int, head: int, heads: int, m: dict) -> torch.Tensor:
    """q [n, d] at positions first .. first + n - 1 against k [first + n, d] from position 0 on; -inf where the key lies behind."""
    i = torch.arange(first, first + q.shape[0])[:, None]
    j = torch.arange(k.shape[0])[None, :]
    s = capped((q @ k.T) * m["scale"], m.get("softcap"))
    s = s - distance_slope(head, heads) * (i - j).to(q.dtype)
    return torch.where(j <= i, s, torch.full_like(s, -math.inf))


def left_mixer(h: torch.Tensor, w: Tensors, p: str, m: dict, eps: float, state: Optional[dict] = None, rnd=None
               ) -> Tuple[torch.Tensor, dict]:
    rnd = rnd or (lambda t: t)
    H, G, d, dv = m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m["vdim"]
    n = h.shape[0]
    first = 0 if state is None else state["k"].shape[0]
    q = rms_norm(rnd(h @ w[p + "q"].T), w[p + "q.norm"], eps)
    k = rms_norm(rnd(h @ w[p + "k"].T), w[p + "k.norm"], eps)
    v = rnd(h @ w[p + "v"].T)
    temp = m.get("q_temp")
    if temp is not None:
        q = q * torch.tensor([query_temperature(first + t, temp["coef"], temp["every"]) for t in range(n)], dtype=q.dtype)[:, None]
    q, k = rnd(q).view(n, H, d), rnd(k).view(n, G, d)
    v = v.view(n, G, dv)
    if state is not None:
        k, v = torch.cat([state["k"], k]), torch.cat([state["v"], v])
    out = torch.empty(n, H, dv, dtype=h.dtype)
    for head in range(H):
        g = head // (H // G)
        out[:, head] = sink_softmax(attention_scores(q[:, head], k[:, g], first, head, H, m)) @ v[:, g]
    return rnd(rnd(out.reshape(n, H * dv)) @ w[p + "o"].T), {"k": k, "v": v}


# ---------------------------------------------------------------------------------------
# lightning attention: a matrix state with one constant decay per head
# ---------------------------------------------------------------------------------------
def constant_decay_scan(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, decay: float, state: Optional[torch.Tensor] = None
                        ) -> Tuple[torch.Tensor, torch.Tensor]:
    """One head. S <- decay S + k v^T;  o = S^T q."""
    S = torch.zeros(k.shape[1], v.shape[1], dtype=k.dtype) if state is None else state.clone()
    out = torch.empty_like(v)
    for t in range(k.shape[0]):
        S = decay * S + k[t][:, None] * v[t][None, :]
        out[t] = q[t] @ S
    return out, S


def right_mixer(h: torch.Tensor, w: Tensors, p: str, m: dict, eps: float, state: Optional[dict] = None, rnd=None
                ) -> Tuple[torch.Tensor, dict]:
    rnd = rnd or (lambda t: t)
    H, d, dv, n = m["heads"], m["dim"], m["vdim"], h.shape[0]
    q, k = (silu(rnd(h @ w[p + x].T)).view(n, H, d) for x in ("q", "k"))
    v = silu(rnd(h @ w[p + "v"].T)).view(n, H, dv)
    out = torch.empty(n, H, dv, dtype=h.dtype)
    states = []
    for head in range(H):
        out[:, head], S = constant_decay_scan(q[:, head], k[:, head], v[:, head], m["decay"][head],
                                              None if state is None else state["S"][head])
        states.append(S)
    y = rms_norm(out.reshape(n, H * dv), w[p + "norm"], eps) * torch.sigmoid(rnd(h @ w[p + "g"].T))
    return rnd(rnd(y) @ w[p + "o"].T), {"S": torch.stack(states)}


def parallel_mixer(h, w, p, m, eps, state=None, rnd=None):
    """Half the sum of the two mixers' outputs, each RMS-normed over the model's width first."""
    state = state or {}
    left, new_left = left_mixer(h, w, p + "left.", m["left"], eps, state.get("left"), rnd)
    right, new_right = right_mixer(h, w, p + "right.", m["right"], eps, state.get("right"), rnd)
    y = 0.5 * (rms_norm(left, w[p + "left.out"], eps) + rms_norm(right, w[p + "right.out"], eps))
    return y, {"left": new_left, "right": new_right}


# ---------------------------------------------------------------------------------------
# gated delta rule with a decay per head and key channel
# ---------------------------------------------------------------------------------------
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


def unit(x: torch.Tensor) -> torch.Tensor:
    return x / torch.sqrt(x.pow(2).sum(-1, keepdim=True) + UNIT_EPS)


def channel_delta_scan(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, g: torch.Tensor, beta: torch.Tensor,
                       state: Optional[torch.Tensor] = None) -> Tuple[torch.Tensor, torch.Tensor]:
    """One head. q, k, g [n, dk]; v [n, dv]; beta [n]; state [dk, dv].
    S <- diag(g) S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q."""
    S = torch.zeros(k.shape[1], v.shape[1], dtype=k.dtype) if state is None else state.clone()
    out = torch.empty_like(v)
    for t in range(k.shape[0]):
        S = g[t][:, None] * S
        u = beta[t] * (v[t] - k[t] @ S)
        S = S + k[t][:, None] * u[None, :]
        out[t] = q[t] @ S
    return out, S


def channel_decay(h: torch.Tensor, w: Tensors, p: str, heads: int, dim: int, rnd=None) -> torch.Tensor:
    rnd = rnd or (lambda t: t)
    z = rnd(h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "dt_bias"]
    return torch.exp(-torch.exp(w[p + "A_log"])[:, None] * torch.nn.functional.softplus(z).view(-1, heads, dim))


def channel_delta_mixer(h: torch.Tensor, w: Tensors, p: str, m: dict, eps: float, state: Optional[dict] = None, rnd=None
                        ) -> Tuple[torch.Tensor, dict]:
    rnd = rnd or (lambda t: t)
    H, G, d, dv, n = m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m["vdim"], h.shape[0]
    state = state or {}
    new, proj = {}, {}
    for name in ("q", "k", "v"):
        y, new["conv." + name] = short_conv(rnd(h @ w[p + name].T), w[p + name + ".conv"], state.get("conv." + name))
        proj[name] = silu(y)
    q = unit(proj["q"].view(n, G, d)) * d ** -0.5
    k = unit(proj["k"].view(n, G, d))
    v = proj["v"].view(n, H, dv)
    beta = torch.sigmoid(rnd(h @ w[p + "b"].T))
    decay = channel_decay(h, w, p, H, d, rnd)
    gate = torch.sigmoid(rnd(rnd(h @ w[p + "g1"].T) @ w[p + "g2"].T)).view(n, H, dv)
    out = torch.empty(n, H, dv, dtype=h.dtype)
    states = []
    for head in range(H):
        g = head // (H // G)
        out[:, head], S = channel_delta_scan(q[:, g], k[:, g], v[:, head], decay[:, head], beta[:, head],
                                             None if "S" not in state else state["S"][head])
        states.append(S)
    new["S"] = torch.stack(states)
    y = rnd((rms_norm(out, w[p + "norm"], eps) * gate).reshape(n, H * dv))
    return rnd(y @ w[p + "o"].T), new


MIXERS = {"parallel": parallel_mixer, "channel_delta": channel_delta_mixer}


# ---------------------------------------------------------------------------------------
# feed-forward, order of layers, output
# ---------------------------------------------------------------------------------------
def clamped_feed_forward(h: torch.Tensor, w: Tensors, p: str, limit: float, rnd=None) -> torch.Tensor:
    rnd = rnd or (lambda t: t)
    g = torch.clamp(rnd(h @ w[p + "gate"].T + w[p + "gate.b"]), max=limit)
    u = torch.clamp(rnd(h @ w[p + "up"].T + w[p + "up.b"]), -limit, limit)
    y = rnd(g * torch.sigmoid(GATE_SLOPE * g) * (u + 1.0))
    return rnd(y @ w[p + "down"].T + w[p + "down.b"])


def layer_runs(cfg: dict) -> List[Tuple[int, Optional[int]]]:
    """(layer, number of the pass when it is the first layer of one) in the order in which layers run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    runs = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        runs += [(i, t if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
    return runs + [(i, None) for i in range(loop["stop"], n)]


def forward(cfg: dict, w: Tensors, tokens: List[int], state: Optional[list] = None, rnd=None, keep_layers: bool = False):
    """(logits [n, vocab], states of the layer runs[, residual after every layer run]). ``rnd`` rounds what an engine
    with 16-bit activations would store; the residual sum is never rounded."""
    r = rnd or (lambda t: t)
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.tensor(tokens, dtype=torch.long)].clone()
    at_start = x.clone()
    runs = layer_runs(cfg)
    new, kept = [], []
    for index, (i, passes) in enumerate(runs):
        layer, p = cfg["layers"][i], f"l{i}."
        if passes is not None:
            if passes > 0:
                x = x + at_start
            x = x + w["loop.step"][passes]
        h = r(rms_norm(x, w[p + "norm1"], eps, around_zero=True))
        y, s = MIXERS[layer["type"]](h, w, p + "mix.", layer["mixer"], eps, None if state is None else state[index], rnd)
        new.append(s)
        x = x + y
        if layer.get("mlp") is not None:
            h = r(rms_norm(x, w[p + "norm2"], eps, around_zero=True))
            x = x + clamped_feed_forward(h, w, p + "mlp.", layer["mlp"]["limit"], rnd)
        kept.append(x)
    logits = r(rms_norm(x, w["final.norm"], eps, around_zero=True)) @ w["embed"].T
    return (logits, new, kept) if keep_layers else (logits, new)


def round_to_bfloat16(t: torch.Tensor) -> torch.Tensor:
    return t.to(torch.bfloat16).to(t.dtype)
