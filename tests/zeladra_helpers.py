"""Configurations and weights of the tests' own for the Zeladra decoder.

Weights are drawn at magnitudes that keep every mechanism alive (decays spread below one, step sizes of either side of
one, gates around a half, streams that differ and mix, norms with biases) and are bfloat16-exact, so that a 32-bit run, a
bfloat16 run and the plain implementation read the same numbers.
"""
from __future__ import annotations

import json
import os
from typing import Dict, List

import numpy as np
import torch


# --- layers -----------------------------------------------------------------------------------------------------------
def latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, base=10000.0, scaling=None, kv_from=None, scale=None):
    """Mixer ``latent_attention``; ``scaling``: (factor, original, fast, slow)."""
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
         "scale": float(scale if scale is not None else (dim + rot_dim) ** -0.5), "rot": {"dims": rot_dim, "base": float(base)}}
    if scaling:
        m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m}


def mamba2(heads, vdim, state, groups=1, norm_groups=1, conv=4):
    return {"type": "mamba2", "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups,
                                        "norm_groups": norm_groups, "conv": conv}}


def windowed(heads, kv_heads, dim, vdim, size, keep_first=0, rot_dims=None, base=10000.0, scale=None):
    """Mixer ``attention``: a sliding window that keeps the first positions."""
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": size, "keep_first": keep_first},
         "scale": float(scale if scale is not None else dim ** -0.5)}
    dims = dim if rot_dims is None else rot_dims
    if dims:
        m["rot"] = {"dims": dims, "base": float(base)}
    return {"type": "attention", "mixer": m}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def config(vocab, width, layers, mlps, streams=2, eps=1e-5, embedding_scale=1.5):
    assert len(layers) == len(mlps)
    return {"architecture": "Zeladra", "embedding": {"scale": embedding_scale}, "norm": {"eps": eps}, "streams": streams,
            "vocab": vocab, "width": width, "layers": [dict(layer, mlp=mlp) for layer, mlp in zip(layers, mlps)]}


def single(layer, mlp=None, vocab=97, width=64, **kw):
    return config(vocab, width, [layer], [mlp], **kw)


YARN = (8.0, 64, 8.0, 1.0)

# Two models that have every kind of layer; the second at other sizes: three streams, widths that are no multiples of 16,
# one head, groups of their own for B and C, another order (two latent layers on one cache with a recurrence between
# them, a window without kept positions), no feed-forward in other places.
Z1 = config(83, 48, [
    mamba2(4, 12, 20, groups=2, norm_groups=2, conv=4),
    latent(4, 16, 8, 16, 24, 24, base=500.0, scaling=YARN),
    windowed(4, 2, 16, 16, 11, keep_first=3, rot_dims=8),
    latent(2, 8, 8, 24, 16, 24, base=500.0, scaling=YARN, kv_from=1),
], [None, dense(40), dense(56), dense(24)], streams=2)

Z2 = config(61, 40, [
    latent(3, 10, 6, 14, 20, 18, base=100.0, scale=0.4),
    windowed(3, 1, 8, 24, 7, keep_first=0, rot_dims=4, base=50.0, scale=0.6),
    mamba2(6, 10, 7, groups=3, norm_groups=4, conv=2),
    latent(1, 24, 6, 8, 12, 18, base=100.0, kv_from=0),
    mamba2(2, 24, 33, groups=1, norm_groups=1, conv=5),
    latent(5, 8, 4, 8, 16, 28, base=1000.0, scaling=(2.0, 40, 4.0, 0.5)),
], [dense(40), None, dense(24), None, dense(32), dense(72)], streams=3, eps=1e-6, embedding_scale=0.75)


def random_config(seed: int) -> dict:
    """A configuration drawn at random: one to six layers of any kind in any order, head counts, widths, windows, ranks,
    states, groups, taps, rotations, streams and constants from lists that hold ones, equal values, odd values and values
    beyond a page, a tile or a chunk of the recurrence."""
    rng = np.random.default_rng(seed)
    pick = lambda xs: xs[int(rng.integers(0, len(xs)))]
    layers, mlps, owners = [], [], []
    for index in range(int(rng.integers(1, 7))):
        kind = pick(["latent", "latent", "space", "space", "window"])
        if kind == "latent":
            source = pick(owners) if owners and pick([True, False]) else None
            dim, vdim, heads = pick([4, 8, 10, 16, 32, 64]), pick([4, 8, 12, 16, 40, 64]), pick([1, 2, 3, 4, 8])
            if source is None:
                rot = pick([2, 4, 8, 16, 32])
                scaling = pick([None, (float(pick([2.0, 8.0])), pick([16, 64, 1024]), float(pick([4.0, 32.0])), 1.0)])
                layers.append(latent(heads, dim, rot, vdim, pick([8, 20, 64]), pick([8, 16, 22, 40, 96]),
                                     base=float(pick([50.0, 1e4, 1e6])), scaling=scaling))
                owners.append(index)
            else:
                m = layers[source]["mixer"]
                layer = latent(heads, dim, m["rot_dim"], vdim, pick([8, 20, 64]), m["kv_rank"], kv_from=source)
                layer["mixer"]["rot"] = json.loads(json.dumps(m["rot"]))
                layers.append(layer)
        elif kind == "space":
            groups = pick([1, 2, 3])
            heads, vdim = groups * pick([1, 2, 4]), pick([4, 8, 12, 16, 20, 40, 64])
            parts = pick([p for p in (1, 2, groups, heads) if heads * vdim % p == 0])
            layers.append(mamba2(heads, vdim, pick([1, 4, 6, 16, 20, 40, 64, 100, 128]), groups, parts, pick([1, 2, 3, 4, 6])))
        else:
            kv = pick([1, 2, 3])
            dim = pick([4, 8, 10, 16, 24, 32, 64])
            layers.append(windowed(kv * pick([1, 2, 4]), kv, dim, pick([dim, 4, 8, 12, 16, 40, 64]),
                                   pick([1, 2, 3, 7, 16, 17, 31, 64, 65, 100, 500]), pick([0, 1, 4, 9, 70]),
                                   rot_dims=pick([0, 2, dim // 2 // 2 * 2, dim // 2 * 2]), base=float(pick([50.0, 1e4, 1e6]))))
        mlps.append(pick([None, dense(pick([16, 24, 40, 64, 100]))]))
    return config(pick([31, 61, 97, 128]), pick([24, 40, 56, 64, 72, 96, 50]), layers, mlps, streams=pick([1, 2, 3, 4, 5]),
                  eps=float(pick([1e-6, 1e-5, 1e-3])), embedding_scale=float(pick([0.5, 1.0, 3.0])))


# --- weights -----------------------------------------------------------------------------------------------------------
def _bf16(a) -> torch.Tensor:
    return torch.from_numpy(np.asarray(a, dtype=np.float32)).to(torch.bfloat16)


def make_weights(cfg: dict, seed: int, sharp: float = 1.0) -> Dict[str, torch.Tensor]:
    """``sharp`` scales the projections that queries come from: above 1 attention weights are peaked."""
    rng = np.random.default_rng(seed)
    W, S = cfg["width"], cfg["streams"]
    out: Dict[str, torch.Tensor] = {}

    def mat(rows, cols, gain=1.0):
        return _bf16(rng.standard_normal((rows, cols)) * gain / np.sqrt(cols))

    def norm(name, width=W, bias=True):
        out[name] = _bf16(1.0 + 0.1 * rng.standard_normal(width))
        if bias:
            out[name + ".b"] = _bf16(0.2 * rng.standard_normal(width))

    def connection(name):
        out[name + ".in"] = _bf16((1.0 + 0.3 * rng.standard_normal(S)) / S)
        out[name + ".out"] = _bf16(0.4 + 0.15 * rng.standard_normal(S))
        out[name + ".mix"] = _bf16(0.8 * np.eye(S) + 0.3 / S * rng.standard_normal((S, S)))

    out["embed"] = _bf16(rng.standard_normal((cfg["vocab"], W)))
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}.mix."
        norm(f"l{i}.norm1")
        connection(f"l{i}.hc1")
        if layer["type"] == "latent_attention":
            H, d, r, dv, qr, kr = (m[k] for k in ("heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank"))
            out[p + "dq"] = mat(qr, W)
            norm(p + "dq.norm", qr, bias=False)
            out[p + "uq"] = mat(H * (d + r), qr, sharp)
            if m.get("kv_from") is None:
                out[p + "dkv"] = mat(kr + r, W)
                norm(p + "dkv.norm", kr, bias=False)
            out[p + "uk"], out[p + "uv"] = mat(H * d, kr), mat(H * dv, kr, 1.5)
            out[p + "g"], out[p + "o"] = mat(H, W, 1.5), mat(W, H * dv, 1.5)
        elif layer["type"] == "mamba2":
            H, P, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
            inner, channels = H * P, H * P + 2 * G * N
            out[p + "in"] = mat(inner + channels + H, W)
            out[p + "conv"] = _bf16(rng.standard_normal((channels, m["conv"])) / np.sqrt(m["conv"]))
            out[p + "conv.b"] = _bf16(0.3 * rng.standard_normal(channels))
            out[p + "dt_bias"] = _bf16(rng.uniform(-4.0, 0.0, H))
            out[p + "A_log"] = _bf16(rng.uniform(-1.5, 1.5, H))
            out[p + "D"] = _bf16(rng.standard_normal(H))
            norm(p + "norm", inner, bias=False)
            out[p + "o"] = mat(W, inner)
        else:
            H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            out[p + "q"], out[p + "k"], out[p + "v"] = mat(H * d, W, sharp), mat(G * d, W), mat(G * dv, W, 1.5)
            out[p + "o"] = mat(W, H * dv)
        if layer.get("mlp") is not None:
            norm(f"l{i}.norm2")
            connection(f"l{i}.hc2")
            ff = layer["mlp"]["ff"]
            q = f"l{i}.mlp."
            out[q + "gate"], out[q + "up"], out[q + "down"] = mat(ff, W, 1.5), mat(ff, W, 1.5), mat(W, ff)
    norm("final.norm")
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
