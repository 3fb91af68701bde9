"""Shared by the Sorulix tests: small configurations that differ in every size and option, random weights by on-disk
name (made here, not by the engine), and the plain model's logits."""
from __future__ import annotations

from typing import Dict, List

import numpy as np
import torch

from plain import sorulix_plain as plain


def dense(ff, limit):
    return {"kind": "dense", "ff": ff, "limit": limit}


def parallel(left, right, mlp):
    heads, kv_heads, dim, vdim, scale, softcap, temp = left
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if softcap is not None:
        m["softcap"] = softcap
    if temp is not None:
        m["q_temp"] = {"coef": temp[0], "every": temp[1]}
    decay, rdim, rvdim = right
    return {"type": "parallel", "mlp": mlp, "mixer": {"left": m, "right": {"heads": len(decay), "dim": rdim, "vdim": rvdim, "decay": list(decay)}}}


def delta(heads, kv_heads, dim, vdim, conv, mlp, ranks=(8, 8)):
    """``ranks`` are for the weights alone: config.json does not state them."""
    return {"type": "channel_delta", "mlp": mlp, "ranks": ranks,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


# A: both mixers, grouped heads on both, values of another size than keys, a run of two layers run three times, a layer
# without feed-forward inside it
SOR_A = {"architecture": "Sorulix", "vocab": 200, "width": 64, "norm": {"eps": 1e-5}, "loop": {"start": 1, "stop": 3, "times": 3},
         "layers": [delta(4, 2, 16, 24, 3, dense(96, 1.5), (12, 20)),
                    parallel((4, 2, 16, 24, 0.3, 9.0, (0.25, 8)), ([0.7, 0.97, 0.999], 12, 20), None),
                    delta(2, 2, 24, 8, 2, dense(72, 0.8), (5, 9)),
                    parallel((6, 3, 8, 8, 0.5, 15.0, (0.1, 20)), ([0.5, 0.9], 16, 8), dense(40, 3.0))]}
# B: nothing is a multiple of eight, one tap, no cap and no temperature on one side, no loop
SOR_B = {"architecture": "Sorulix", "vocab": 77, "width": 50, "norm": {"eps": 3e-6},
         "layers": [parallel((3, 1, 10, 6, 0.4, None, None), ([0.6, 0.93, 0.99, 0.2, 0.85], 6, 10), dense(30, 1.0)),
                    delta(3, 1, 10, 14, 1, dense(34, 0.5), (3, 7)),
                    parallel((5, 5, 6, 10, 0.3, 4.0, (0.5, 3)), ([0.98], 10, 18), None),
                    delta(6, 3, 6, 5, 5, None, (17, 2))]}
# C: head sizes that the MFMA attention kernels serve (64, 128), widths that the MFMA products serve, the whole model a loop
SOR_C = {"architecture": "Sorulix", "vocab": 512, "width": 192, "norm": {"eps": 1e-6}, "loop": {"start": 0, "stop": 3, "times": 2},
         "layers": [parallel((6, 2, 64, 64, 0.125, 24.0, (0.2, 96)), ([0.75, 0.95, 0.998], 64, 64), dense(256, 2.0)),
                    delta(4, 2, 64, 128, 4, dense(384, 1.2), (32, 48)),
                    parallel((2, 1, 128, 128, 0.09, 30.0, (0.15, 200)), ([0.9, 0.99], 32, 128), dense(320, 4.0))]}
# D: one head everywhere, the loop is the last layer, once
SOR_D = {"architecture": "Sorulix", "vocab": 90, "width": 32, "norm": {"eps": 1e-5}, "loop": {"start": 2, "stop": 3, "times": 1},
         "layers": [parallel((1, 1, 12, 12, 0.35, 6.0, (0.3, 1)), ([0.995], 8, 16), dense(48, 0.7)),
                    delta(1, 1, 20, 12, 6, None, (4, 4)),
                    parallel((1, 1, 12, 20, 0.3, 11.0, None), ([1.0], 12, 12), dense(24, 1.0))]}
# E: delta layers only (no cache group at all), a loop over one of them; F: parallel layers only, head size 64 with groups
# of sixteen query heads, a loop in the middle
SOR_E = {"architecture": "Sorulix", "vocab": 120, "width": 48, "norm": {"eps": 1e-6}, "loop": {"start": 0, "stop": 1, "times": 4},
         "layers": [delta(4, 4, 12, 12, 4, dense(64, 1.1), (6, 10)), delta(2, 1, 28, 20, 3, None, (16, 8))]}
SOR_F = {"architecture": "Sorulix", "vocab": 150, "width": 128, "norm": {"eps": 2e-5}, "loop": {"start": 1, "stop": 2, "times": 2},
         "layers": [parallel((16, 1, 64, 64, 0.11, 18.0, (0.4, 32)), ([0.8, 0.9, 0.99, 0.999], 16, 16), dense(96, 1.0)),
                    parallel((4, 4, 64, 64, 0.2, 12.0, (0.1, 50)), ([0.3, 0.96], 24, 40), dense(128, 2.5)),
                    parallel((2, 2, 64, 32, 0.15, None, (0.2, 10)), ([0.97], 64, 64), None)]}
SOR = {"A": SOR_A, "B": SOR_B, "C": SOR_C, "D": SOR_D, "E": SOR_E, "F": SOR_F}


def stored_config(cfg: Dict) -> Dict:
    """What goes into config.json: without the ranks, which only the stored tensors state."""
    return dict(cfg, layers=[{k: v for k, v in l.items() if k != "ranks"} for l in cfg["layers"]])


def tensor_shapes(cfg: Dict) -> Dict[str, tuple]:
    V, W = cfg["vocab"], cfg["width"]
    shapes = {"embed": (V, W), "final.norm": (W,)}
    if cfg.get("loop"):
        shapes["loop.step"] = (cfg["loop"]["times"], W)
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        x = p + "mix."
        shapes[p + "norm1"] = (W,)
        if layer["type"] == "parallel":
            a, b = m["left"], m["right"]
            H, G, d, dv = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            y = x + "left."
            shapes.update({y + "q": (H * d, W), y + "k": (G * d, W), y + "v": (G * dv, W), y + "q.norm": (H * d,), y + "k.norm": (G * d,),
                           y + "o": (W, H * dv), y + "out": (W,)})
            R, d, dv = b["heads"], b["dim"], b["vdim"]
            y = x + "right."
            shapes.update({y + "q": (R * d, W), y + "k": (R * d, W), y + "v": (R * dv, W), y + "g": (R * dv, W), y + "norm": (R * dv,),
                           y + "o": (W, R * dv), y + "out": (W,)})
        else:
            H, G, d, dv, (ra, rg) = m["heads"], m["kv_heads"], m["dim"], m["vdim"], layer["ranks"]
            for name, rows in (("q", G * d), ("k", G * d), ("v", H * dv)):
                shapes[x + name] = (rows, W)
                shapes[x + name + ".conv"] = (rows, m["conv"])
            shapes.update({x + "b": (H, W), x + "A_log": (H,), x + "dt_bias": (H * d,), x + "a1": (ra, W), x + "a2": (H * d, ra),
                           x + "g1": (rg, W), x + "g2": (H * dv, rg), x + "norm": (dv,), x + "o": (W, H * dv)})
        if layer.get("mlp") is not None:
            shapes[p + "norm2"] = (W,)
            ff, y = layer["mlp"]["ff"], p + "mlp."
            shapes.update({y + "gate": (ff, W), y + "gate.b": (ff,), y + "up": (ff, W), y + "up.b": (ff,), y + "down": (W, ff),
                           y + "down.b": (W,)})
    return shapes


def make_weights(cfg: Dict, seed: int, stored: torch.dtype = torch.bfloat16, key_gain: float = 1.0) -> Dict[str, torch.Tensor]:
    """Matrices N(0, 1/sqrt(columns)); plain norm weights 1 + N(0, 0.1), weights stored around zero N(0, 0.1); convolution
    taps N(0, 0.6); A_log, dt_bias and the feed-forward's biases N(0, 0.5), A_log lower (a long memory); step vectors
    N(0, 0.3). ``key_gain`` multiplies the query and key norms (steep softmax, so that a wrong key shows). Rounded to
    ``stored``."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        t = torch.randn(shape, generator=g)
        if name.endswith(".conv"):
            t = 0.6 * t
        elif name == "loop.step":
            t = 0.3 * t
        elif len(shape) == 2:
            t = t / shape[1] ** 0.5 * (1.0 if name != "embed" else shape[1] ** 0.5 * 0.5)
        elif name.endswith(".A_log"):
            t = 0.5 * t - 1.0
        elif name.endswith(".dt_bias") or name.endswith(".b"):
            t = 0.5 * t
        elif name.endswith(("norm1", "norm2", "final.norm")):
            t = 0.1 * t
        else:
            t = 1.0 + 0.1 * t
            if name.endswith(("q.norm", "k.norm")):
                t = t * key_gain
        out[name] = t.to(stored)
    return out


def as_f64(weights: Dict[str, torch.Tensor]) -> Dict[str, torch.Tensor]:
    return {k: v.to(torch.float64) for k, v in weights.items()}


def plain_logits(cfg: Dict, weights: Dict[str, torch.Tensor], tokens: List[int], rnd=None) -> np.ndarray:
    return plain.forward(cfg, as_f64(weights), tokens, rnd=rnd)[0].numpy()


def plain_logits_bf16(cfg: Dict, weights: Dict[str, torch.Tensor], tokens: List[int]) -> np.ndarray:
    return plain_logits(cfg, weights, tokens, rnd=plain.round_to_bfloat16)


def plain_logits_f32(cfg: Dict, weights: Dict[str, torch.Tensor], tokens: List[int]) -> np.ndarray:
    """The plain model evaluated in float32: how far 32-bit arithmetic alone moves the logits."""
    return plain.forward(cfg, {k: v.to(torch.float32) for k, v in weights.items()}, tokens)[0].numpy()


def random_tokens(cfg: Dict, n: int, seed: int) -> List[int]:
    return [int(t) for t in np.random.default_rng(seed).integers(0, cfg["vocab"], size=n)]


def random_config(rng: np.random.Generator, fast_sizes: bool) -> Dict:
    """A configuration drawn at random; ``fast_sizes``: head sizes and widths that the MFMA kernels serve."""
    pick = lambda values: values[int(rng.integers(len(values)))]
    width = pick([64, 128, 192, 320] if fast_sizes else [40, 56, 74, 100, 132])
    layers = []
    for _ in range(int(rng.integers(2, 5))):
        mlp = None if rng.random() < 0.2 else dense(pick([64, 128, 160] if fast_sizes else [30, 52, 75]), pick([0.6, 1.0, 3.0, 7.0]))
        if rng.random() < 0.55:
            G = pick([1, 2, 3])
            dim = pick([64, 128]) if fast_sizes else pick([8, 10, 16, 36])
            vdim = dim if fast_sizes and rng.random() < 0.8 else pick([8, 12, 20, 64])
            temp = None if rng.random() < 0.2 else (pick([0.1, 0.35]), pick([1, 5, 16, 64]))
            cap = None if rng.random() < 0.2 else pick([5.0, 20.0, 50.0])
            heads = int(rng.integers(1, 6))
            layers.append(parallel((G * pick([1, 2, 4]), G, dim, vdim, float(pick([0.5, 1.0, 2.0])) * dim ** -0.5, cap, temp),
                                   ([float(x) for x in rng.uniform(0.3, 1.0, size=heads)], pick([8, 16, 24, 32, 64, 70]), pick([8, 12, 32, 64, 100])), mlp))
        else:
            G = pick([1, 2, 3])
            layers.append(delta(G * pick([1, 1, 2]), G, pick([8, 16, 20, 32, 64, 128]), pick([8, 12, 32, 64, 72]), pick([1, 2, 3, 4, 6]), mlp,
                                (int(rng.integers(1, 40)), int(rng.integers(1, 40)))))
    cfg = {"architecture": "Sorulix", "vocab": pick([97, 300, 512]), "width": width, "norm": {"eps": pick([1e-6, 1e-5])}, "layers": layers}
    if rng.random() < 0.7:
        start = int(rng.integers(0, len(layers)))
        cfg["loop"] = {"start": start, "stop": int(rng.integers(start + 1, len(layers) + 1)), "times": int(rng.integers(1, 4))}
    return cfg
