"""Shared by the Setirax tests: small configurations that differ in every size and option, random weights by on-disk
name (made here, not by the engine), and the plain model's logits."""
from __future__ import annotations

import copy
from typing import Dict, List

import numpy as np
import torch

from plain import setirax_plain as plain


def dense(ff):
    return {"kind": "dense", "ff": ff}


def parallel(left, right, mlp, scales=(0.8, 0.5), **extra):
    """left: (heads, kv_heads, dim, vdim, scale, softcap, window, taps, (rotated dims, base, scaling) or None);
    right: (heads, dim, vdim, tau, rank), the rank for the weights alone: config.json does not state it."""
    heads, kv_heads, dim, vdim, scale, softcap, window, taps, rot = left
    a = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "conv": taps}
    if softcap is not None:
        a["softcap"] = softcap
    if window is not None:
        a["mask"] = {"size": window}
    if rot is not None:
        a["rot"] = {"dims": rot[0], "base": rot[1]}
        if rot[2] is not None:
            a["rot"]["scaling"] = dict(zip(("factor", "low", "high", "original"), rot[2]))
    heads, dim, vdim, tau, rank = right
    m = {"left": a, "right": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}, "left_scale": scales[0], "right_scale": scales[1]}
    return {"type": "parallel", "mixer": m, "mlp": mlp, "rank": rank, **extra}


def unit(width, blocks, conv, mlp, **extra):
    return {"type": "rglru", "mixer": {"width": width, "blocks": blocks, "conv": conv}, "mlp": mlp, **extra}


def latent(heads, dim, vdim, kv_rank, scale, window, mlp, **extra):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale}
    if window is not None:
        m["mask"] = {"size": window}
    return {"type": "latent_attention", "mixer": m, "mlp": mlp, **extra}


def model(vocab, width, eps, cap, layers):
    return {"architecture": "Setirax", "vocab": vocab, "width": width, "norm": {"eps": eps}, "logit_softcap": cap, "layers": layers}


# A: every mixer, grouped heads, values of another size than keys, a window of its own for each softmax mixer, part of a head
# rotated, two layers with another layer's tensors
_A1 = parallel((4, 2, 16, 24, 0.4, 9.0, 11, 3, (8, 700.0, (4.0, 1.0, 3.0, 40.0))), (3, 12, 20, 8.0, 6), dense(96))
_A2 = unit(48, 3, 4, None)
SET_A = model(200, 64, 1e-5, 12.0, [
    latent(3, 12, 20, 24, 0.4, 14, dense(72)), _A1, _A2, dict(copy.deepcopy(_A1), weights_of=1), dict(copy.deepcopy(_A2), weights_of=2),
    parallel((2, 1, 24, 8, 0.3, None, None, 2, None), (2, 20, 8, 3.0, 5), None, (1.0, -0.7))])
# B: nothing is a multiple of eight, one tap, a window of one, no cap on the logits, the unit with a feed-forward
SET_B = model(77, 50, 3e-6, None, [
    unit(33, 3, 1, dense(30)),
    parallel((3, 1, 10, 6, 0.5, 4.0, 5, 1, (6, 50.0, None)), (5, 6, 10, 16.0, 3), dense(34), (0.3, 1.1)),
    latent(5, 6, 10, 13, 0.5, 1, None),
    parallel((6, 3, 6, 11, 0.6, 7.0, 9, 6, (2, 90.0, (2.0, 0.5, 2.5, 12.0))), (1, 9, 5, 1.0, 17), None, (1.2, 0.6)),
    unit(45, 5, 6, None)])
# C: sizes that the MFMA kernels serve (heads of 64 and 128, latents of 64 and 128)
SET_C = model(512, 128, 1e-6, 24.0, [
    parallel((6, 2, 64, 64, 0.2, 20.0, 37, 4, (64, 5000.0, (8.0, 1.0, 4.0, 128.0))), (3, 64, 64, 16.0, 32), dense(256), (0.7, 0.8)),
    latent(4, 32, 64, 64, 0.25, 50, dense(384)),
    unit(192, 2, 4, dense(320)),
    latent(20, 64, 32, 128, 0.15, 33, None),
    parallel((2, 1, 128, 128, 0.12, 40.0, 70, 3, (32, 20000.0, None)), (2, 32, 128, 4.0, 48), dense(192), (0.9, 0.4))])
# D: one of everything; a window of two
SET_D = model(90, 32, 1e-5, 6.0, [
    parallel((1, 1, 12, 12, 0.5, 6.0, 2, 5, (12, 30.0, (3.0, 1.0, 1.5, 20.0))), (1, 8, 16, 2.0, 1), dense(48), (1.0, 1.0)),
    unit(20, 1, 2, None),
    latent(1, 12, 20, 8, 0.5, 2, dense(24))])
# E: units alone (no cache at all), one of them run three times; F: latents alone, with and without a window
SET_E = model(120, 48, 1e-6, 10.0, [unit(64, 4, 4, dense(64)), unit(64, 4, 4, dense(64), weights_of=0), unit(40, 2, 3, None),
                                    unit(64, 4, 4, dense(64), weights_of=1)])
SET_F = model(150, 80, 2e-5, 18.0, [latent(4, 24, 16, 32, 0.35, 25, dense(96)), latent(2, 16, 40, 40, 0.4, None, dense(64)),
                                    latent(4, 24, 16, 32, 0.35, 25, dense(96), weights_of=0)])
# G: parallel layers alone, sixteen query heads on one key/value head, decays that hold on for long
SET_G = model(160, 96, 5e-6, 15.0, [
    parallel((16, 1, 64, 64, 0.2, 15.0, 29, 4, (16, 100.0, (5.0, 1.0, 2.0, 60.0))), (4, 16, 16, 30.0, 16), dense(128)),
    parallel((4, 4, 64, 32, 0.25, 12.0, 46, 4, (64, 800.0, None)), (2, 70, 40, 5.0, 9), None, (0.4, 0.9))])
SET = {"A": SET_A, "B": SET_B, "C": SET_C, "D": SET_D, "E": SET_E, "F": SET_F, "G": SET_G}


def stored_config(cfg: Dict) -> Dict:
    """What goes into config.json: without the ranks, which only the stored tensors state."""
    return dict(cfg, layers=[{k: v for k, v in l.items() if k != "rank"} for l in cfg["layers"]])


def sharpened(cfg: Dict, gain: float) -> Dict:
    """The same model with steeper softmax scores, so that a wrong key shows."""
    cfg = copy.deepcopy(cfg)
    for layer in cfg["layers"]:
        m = layer["mixer"].get("left", layer["mixer"])
        if "scale" in m:
            m["scale"] *= gain
    return cfg


def tensor_shapes(cfg: Dict) -> Dict[str, tuple]:
    V, W = cfg["vocab"], cfg["width"]
    shapes = {"embed": (V, W), "final.norm": (W,)}
    for i, layer in enumerate(cfg["layers"]):
        if layer.get("weights_of") is not None:
            continue
        p, m = f"l{i}.", layer["mixer"]
        x = p + "mix."
        shapes[p + "norm1"] = (W,)
        if layer["type"] == "parallel":
            a, b, y = m["left"], m["right"], x + "left."
            H, G, d, dv = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            for name, rows in (("q", H * d), ("k", G * d), ("v", G * dv)):
                shapes[y + name] = (rows, W)
                shapes[y + name + ".conv"] = (rows, a["conv"])
            shapes[y + "o"] = (W, H * dv)
            R, d, dv, rank, y = b["heads"], b["dim"], b["vdim"], layer["rank"], x + "right."
            shapes.update({y + "q": (R * d, W), y + "k": (R * d, W), y + "v": (R * dv, W), y + "g": (R * dv, W), y + "o": (W, R * dv),
                           y + "norm": (dv,), y + "a1": (rank, W), y + "a2": (R * d, rank), y + "a2.b": (R * d,)})
        elif layer["type"] == "rglru":
            N, B, T = m["width"], m["blocks"], m["conv"]
            P = N // B
            shapes.update({x + "y": (N, W), x + "y.b": (N,), x + "x": (N, W), x + "x.b": (N,), x + "conv": (N, T), x + "conv.b": (N,),
                           x + "ra": (B, P, P), x + "ra.b": (B, P), x + "ri": (B, P, P), x + "ri.b": (B, P), x + "lam": (N,), x + "o": (W, N)})
        else:
            H, d, dv, R = m["heads"], m["dim"], m["vdim"], m["kv_rank"]
            shapes.update({x + "q": (H * d, W), x + "dkv": (R, W), x + "dkv.norm": (R,), x + "uk": (H * d, R), x + "uv": (H * dv, R),
                           x + "sink": (H,), x + "o": (W, H * dv)})
        if layer.get("mlp") is not None:
            ff, y = layer["mlp"]["ff"], p + "mlp."
            shapes[p + "norm2"] = (W,)
            shapes.update({y + "up": (ff, W), y + "up.b": (ff,), y + "down": (W, ff), y + "down.b": (W,)})
    return shapes


def make_weights(cfg: Dict, seed: int, stored: torch.dtype = torch.bfloat16) -> Dict[str, torch.Tensor]:
    """Matrices N(0, 1/sqrt(columns)); norm weights 1 + N(0, 0.1); taps N(0, 0.6); biases N(0, 0.5), the decays' higher (a long
    memory); ``lam`` low (the unit's decays near one for some channels, short for others); sinks N(1, 0.7). Rounded to
    ``stored``."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        t = torch.randn(shape, generator=g)
        if name.endswith(".conv"):
            t = 0.6 * t
        elif name == "embed":
            t = 0.5 * t
        elif len(shape) == 3:
            t = 1.5 * t / shape[2] ** 0.5
        elif name.endswith((".a2.b",)):
            t = t + 1.0
        elif name.endswith(".b"):
            t = 0.5 * t
        elif name.endswith(".lam"):
            t = 1.5 * t - 3.0
        elif name.endswith(".sink"):
            t = 0.7 * t + 1.0
        elif len(shape) == 2:
            t = t / shape[1] ** 0.5
        else:
            t = 1.0 + 0.1 * t
        out[name] = t.to(stored)
    return out


def as_f64(weights: Dict[str, torch.Tensor]) -> Dict[str, torch.Tensor]:
    return {k: v.to(torch.float64) for k, v in weights.items()}


def plain_logits(cfg: Dict, weights: Dict[str, torch.Tensor], tokens: List[int], rnd=plain.keep) -> np.ndarray:
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
    width = pick([64, 128, 224, 320] if fast_sizes else [40, 56, 74, 100, 132])
    layers: List[Dict] = []
    for i in range(int(rng.integers(2, 5))):
        mlp = None if rng.random() < 0.25 else dense(pick([64, 128, 160] if fast_sizes else [30, 52, 75]))
        kind = rng.random()
        if layers and kind < 0.2:
            j = int(rng.integers(len(layers)))
            layers.append(dict(copy.deepcopy(layers[j]), weights_of=j))
        elif kind < 0.5:
            G, dim = pick([1, 2, 3]), pick([64, 128]) if fast_sizes else pick([8, 10, 16, 36])
            vdim = dim if fast_sizes and rng.random() < 0.8 else pick([8, 12, 20, 64])
            scaling = None if rng.random() < 0.3 else (pick([2.0, 8.0]), 1.0, pick([2.0, 4.0]), pick([16.0, 64.0, 300.0]))
            rot = None if rng.random() < 0.15 else (pick([dim, dim // 2 // 2 * 2]), pick([50.0, 10000.0]), scaling)
            layers.append(parallel(
                (G * pick([1, 2, 4]), G, dim, vdim, float(pick([1.0, 2.0])) * dim ** -0.5, None if rng.random() < 0.2 else pick([5.0, 20.0, 50.0]),
                 None if rng.random() < 0.15 else pick([2, 7, 16, 33, 48]), pick([1, 2, 3, 4, 6]), rot),
                (pick([1, 2, 3, 5]), pick([8, 16, 24, 64, 70]), pick([8, 12, 32, 64, 100]), pick([1.0, 6.0, 16.0]), int(rng.integers(1, 40))),
                mlp, (float(rng.uniform(0.3, 1.2)), float(rng.uniform(0.3, 1.2)))))
        elif kind < 0.75:
            blocks = pick([1, 2, 3, 4])
            layers.append(unit(blocks * pick([16, 32, 64] if fast_sizes else [5, 12, 18]), blocks, pick([1, 2, 3, 4, 6]), mlp))
        else:
            layers.append(latent(pick([1, 3, 4, 18]), pick([8, 32, 64] if fast_sizes else [6, 10, 20]), pick([16, 64] if fast_sizes else [7, 12]),
                                 pick([32, 64, 96, 128] if fast_sizes else [11, 24, 40]), pick([0.2, 0.4]),
                                 None if rng.random() < 0.15 else pick([1, 5, 17, 40]), mlp))
    return model(pick([97, 300, 512]), width, pick([1e-6, 1e-5]), pick([None, 8.0, 30.0]), layers)
