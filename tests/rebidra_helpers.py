"""Configurations and weights of the tests' own for the Rebidra decoder.

Weights are drawn at magnitudes that keep every mechanism alive (biases and sinks of the scores' size, convolutions whose taps
all weigh, gates around a half, a loop whose passes change the stream, norms away from one) and are bfloat16-exact, so that a
32-bit run, a bfloat16 run and the plain implementation read the same numbers.
"""
from __future__ import annotations

import json
import os
from typing import Dict, List

import numpy as np
import torch


# --- layers -----------------------------------------------------------------------------------------------------------
def windowed(heads, kv_heads, dim, size, conv=3, rot_dims=None, base=10000.0, scaling=None, scale=None):
    """Mixer ``attention``; ``scaling``: (factor, original, fast, slow); ``size`` 0: no mask."""
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "conv": conv,
         "scale": float(scale if scale is not None else dim ** -0.5)}
    if size:
        m["mask"] = {"size": size}
    dims = dim if rot_dims is None else rot_dims
    if dims:
        m["rot"] = {"dims": dims, "base": float(base)}
        if scaling:
            m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return {"type": "attention", "mixer": m}


def moe(ff, experts, top, shared=None):
    mlp = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared:
        mlp["shared"] = {"ff": shared}
    return mlp


def config(vocab, width, layers, mlps, loop=None, side=8, eps=1e-5, embedding_scale=1.5, logit_scale=0.7):
    """``loop``: (start, stop, times) or None; ``side`` 0: no side table."""
    assert len(layers) == len(mlps)
    out = {"architecture": "Rebidra", "embedding": {"scale": embedding_scale}, "norm": {"eps": eps}, "logit_scale": logit_scale,
           "vocab": vocab, "width": width, "layers": [dict(layer, mlp=mlp) for layer, mlp in zip(layers, mlps)]}
    if loop:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    if side:
        out["token_side"] = {"dim": side}
    return out


def single(layer, mlp=None, vocab=97, width=64, side=0, **kw):
    return config(vocab, width, [layer], [mlp], side=side, **kw)


YARN = (8.0, 64, 8.0, 1.0)

# Two models that have every mechanism; the second at other sizes: three passes through a loop that ends with the last layer,
# windows of other sizes in other layers (groups of their own in the cache), one key head, as many key heads as heads, one tap
# and six, part of a head rotated and none, more experts chosen than not, no shared expert, no feed-forward, widths that are
# no multiples of 8.
R1 = config(83, 48, [
    windowed(4, 2, 16, 11, conv=3, base=500.0, scaling=YARN),
    windowed(4, 2, 16, 11, conv=3, base=500.0, scaling=YARN),
    windowed(6, 3, 8, 19, conv=4, rot_dims=4, base=77.0),
    windowed(4, 4, 16, 11, conv=2, base=500.0, scaling=YARN),
], [moe(24, 5, 2, 40), moe(24, 5, 2, 40), moe(32, 8, 3, 16), moe(24, 3, 1, 24)], loop=(1, 3, 2), side=8)

R2 = config(61, 50, [
    windowed(3, 1, 10, 7, conv=6, rot_dims=6, base=100.0, scale=0.4),
    windowed(5, 5, 24, 16, conv=1, rot_dims=0),
    windowed(2, 1, 20, 7, conv=2, base=1000.0, scaling=(2.0, 40, 4.0, 0.5)),
], [None, moe(20, 4, 3), moe(12, 1, 1, 30)], loop=(1, 3, 3), side=5, eps=1e-6, embedding_scale=0.75, logit_scale=1.0)


def random_config(seed: int) -> dict:
    """A configuration drawn at random: one to five layers, any range of them in a loop of one to three passes or none; head
    counts, widths, windows, taps, rotations, experts, side tables and constants from lists that hold ones, equal values, odd
    values and values beyond a page or a tile."""
    rng = np.random.default_rng(seed)
    pick = lambda xs: xs[int(rng.integers(0, len(xs)))]
    layers, mlps = [], []
    count = int(rng.integers(1, 6))
    for _ in range(count):
        kv, dim = pick([1, 2, 3]), pick([4, 8, 10, 16, 24, 32, 48, 64, 80])
        rot = pick([0, 2, dim // 2 // 2 * 2, dim // 2 * 2])
        scaling = pick([None, (float(pick([2.0, 8.0])), pick([16, 64, 1024]), float(pick([4.0, 32.0])), 1.0)])
        layers.append(windowed(kv * pick([1, 2, 3, 4]), kv, dim, pick([1, 2, 3, 7, 16, 17, 31, 64, 65, 100, 500]),
                               conv=pick([1, 2, 3, 4, 5, 7]), rot_dims=rot, base=float(pick([50.0, 1e4, 1e6])), scaling=scaling))
        experts = pick([1, 2, 3, 5, 8, 17])
        mlps.append(pick([None, moe(pick([8, 16, 24, 33, 72]), experts, int(rng.integers(1, experts + 1)), pick([None, 8, 24, 40, 65]))]))
    loop = None
    if pick([True, True, False]):
        start = int(rng.integers(0, count))
        loop = (start, int(rng.integers(start + 1, count + 1)), pick([1, 2, 3]))
    return config(pick([31, 61, 97, 128]), pick([24, 40, 56, 64, 72, 96, 50]), layers, mlps, loop=loop, side=pick([0, 1, 4, 8, 24]),
                  eps=float(pick([1e-6, 1e-5, 1e-3])), embedding_scale=float(pick([0.5, 1.0, 3.0])),
                  logit_scale=float(pick([0.25, 1.0, 2.0])))


# --- weights -----------------------------------------------------------------------------------------------------------
def _bf16(a) -> torch.Tensor:
    return torch.from_numpy(np.asarray(a, dtype=np.float32)).to(torch.bfloat16)


def make_weights(cfg: dict, seed: int, sharp: float = 1.0) -> Dict[str, torch.Tensor]:
    """``sharp`` scales the weights of the query norms: above 1 attention weights are peaked."""
    rng = np.random.default_rng(seed)
    W = cfg["width"]
    side = int((cfg.get("token_side") or {}).get("dim") or 0)
    out: Dict[str, torch.Tensor] = {}

    def mat(rows, cols, gain=1.0):
        return _bf16(rng.standard_normal((rows, cols)) * gain / np.sqrt(cols))

    def gain(width, factor=1.0):
        return _bf16(factor * (1.0 + 0.2 * rng.standard_normal(width)))

    out["embed"] = _bf16(rng.standard_normal((cfg["vocab"], W)))
    if cfg.get("loop"):
        out["loop.in"] = mat(W, 2 * W, 1.2)
    if side:
        out["side.embed"] = _bf16(rng.standard_normal((cfg["vocab"], side * len(cfg["layers"]))))
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}.mix."
        H, G, d = m["heads"], m["kv_heads"], m["dim"]
        out[f"l{i}.norm1"] = gain(W)
        for name, rows in (("q", H * d), ("k", G * d)):
            out[p + name], out[p + name + ".b"] = mat(rows, W), _bf16(0.5 * rng.standard_normal(rows))
            out[p + name + ".conv"] = _bf16(rng.standard_normal((rows, m["conv"])) / np.sqrt(m["conv"]))
            out[p + name + ".norm"] = gain(d, 1.5 * sharp if name == "q" else 1.0)
        out[p + "sink"] = _bf16(rng.standard_normal(H))
        out[p + "g"], out[p + "o"] = mat(H, W, 1.5), mat(W, H * d, 1.5)
        mlp = layer.get("mlp")
        if mlp is not None:
            q = f"l{i}.mlp."
            out[f"l{i}.norm2"] = gain(W)
            E, ff = mlp["router"]["experts"], mlp["expert"]["ff"]
            out[q + "router"], out[q + "router.b"] = mat(E, W, 2.0), _bf16(0.5 * rng.standard_normal(E))
            for e in range(E):
                out[f"{q}e{e}.up"], out[f"{q}e{e}.down"] = mat(ff, W), mat(W, ff)
            if mlp.get("shared"):
                out[q + "shared.up"], out[q + "shared.down"] = mat(mlp["shared"]["ff"], W), mat(W, mlp["shared"]["ff"])
                out[q + "shared.sg"] = mat(1, W, 1.5)
        if side:
            s = f"l{i}.side."
            out[s + "gate"], out[s + "proj"], out[s + "norm"] = mat(side, W, 1.5), mat(W, side), gain(W, 0.5)
    out["final.norm"] = gain(W)
    out["head"] = mat(cfg["vocab"], W)
    return out


def make_folder(path, cfg: dict, seed: int, dtype=torch.float32, sharp: float = 1.0, edit=None) -> str:
    """Write ``config.json`` and ``model.safetensors``; ``edit(tensors)`` may change the weights before."""
    from vipera_rs_amd.weights import write_safetensors

    path = str(path)
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as handle:
        json.dump(cfg, handle)
    tensors = make_weights(cfg, seed, sharp)
    if edit is not None:
        edit(tensors)
    write_safetensors(os.path.join(path, "model.safetensors"), [(name, t.to(dtype)) for name, t in tensors.items()])
    return path


def load_folder(folder):
    """(configuration dict, tensors as float64 numpy arrays) of a model folder, for the plain implementation."""
    from safetensors.torch import load_file

    with open(os.path.join(folder, "config.json")) as handle:
        cfg = json.load(handle)
    w = {name: t.to(torch.float64).numpy() for name, t in load_file(os.path.join(folder, "model.safetensors")).items()}
    return cfg, w


def tokens_of(vocab: int, count: int, seed: int) -> List[int]:
    return [int(t) for t in np.random.default_rng(seed).integers(0, vocab, count)]
