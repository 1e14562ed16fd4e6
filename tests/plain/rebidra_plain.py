"""A plain, slow implementation of the Rebidra decoder in float64 numpy: one function per mechanism, whole sequences
only (no cache, no state passing, no batching).  It shares no code with the engine; the tests hold the engine's
kernels, cache, state slots and scheduler to it.

Notation: ``x`` [T, width] is a sublayer's input, ``w`` the dict of a folder's tensors as float64 arrays, ``pre`` a
tensor-name prefix such as ``l3.mix.``, ``m`` the layer's ``mixer`` object from the configuration, ``eps`` the model's
``norm.eps``.
"""
import math

import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def over_rms(x, eps):
    """x divided by its root mean square over the last axis, eps inside the root."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def layer_norm(x, weight, eps):
    """Mean taken off, divided by the standard deviation (eps inside the root), times the weight; no bias."""
    d = x - np.mean(x, axis=-1, keepdims=True)
    return d / np.sqrt(np.mean(d * d, axis=-1, keepdims=True) + eps) * weight


def causal_conv(u, taps):
    """u [T, channels], taps [channels, n]: y_t = sum_b taps[:, n - 1 - b] u_{t - b}, nothing before the first row."""
    T, n = u.shape[0], taps.shape[1]
    y = np.zeros_like(u)
    for back in range(min(n, T)):
        y[back:] += taps[:, n - 1 - back] * u[:T - back]
    return y


def frequencies(rot):
    """One frequency per rotated pair: base^(-2i/dims); with ``rot.scaling`` the slow ones are divided by ``factor``
    and those in between blended by a ramp over the pair's index (YaRN)."""
    dims, base = int(rot["dims"]), float(rot["base"])
    scaling = rot.get("scaling")
    out = []
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if scaling:
            factor, original = float(scaling["factor"]), float(scaling["original"])
            # the pair index at which a wave makes so many turns within ``original`` positions
            at = [dims * math.log(original / (2.0 * math.pi * float(scaling[k]))) / (2.0 * math.log(base)) for k in ("fast", "slow")]
            low, high = max(math.floor(at[0]), 0), min(math.ceil(at[1]), dims - 1)
            share = min(max((i - low) / max(high - low, 0.001), 0.0), 1.0)
            f = f / factor * share + f * (1.0 - share)
        out.append(f)
    return np.array(out)


def amplitude(rot):
    """What sines and cosines are multiplied by."""
    scaling = (rot or {}).get("scaling")
    return 1.0 + 0.1 * math.log(float(scaling["factor"])) if scaling else 1.0


def rotate(x, positions, rot):
    """x [T, heads, dim]: numbers i and i + dims/2 of a head's first ``dims`` are a pair and turn by position * f_i."""
    dims = int((rot or {}).get("dims") or 0)
    if not dims:
        return x
    half = dims // 2
    turn = np.asarray(positions, dtype=np.float64)[:, None, None] * frequencies(rot)
    c, s = amplitude(rot) * np.cos(turn), amplitude(rot) * np.sin(turn)
    first, second = x[..., :half], x[..., half:dims]
    return np.concatenate([first * c - second * s, second * c + first * s, x[..., dims:]], axis=-1)


def visible(size, T):
    """[T, T] booleans: position i sees j if 0 <= i - j < size; size 0: every earlier one and itself."""
    back = np.arange(T)[:, None] - np.arange(T)[None, :]
    return (back >= 0) & ((back < size) if size else True)


def sink_attention(q, k, v, scale, mask, sink):
    """q [T, H, d], k [T, G, d], v [T, G, dv] -> [T, H, dv]; the softmax's denominator of head h also holds exp(sink[h])."""
    T, H, _ = q.shape
    group = H // k.shape[1]
    out = np.zeros((T, H, v.shape[2]))
    for h in range(H):
        s = np.where(mask, scale * (q[:, h] @ k[:, h // group].T), -np.inf)
        top = np.maximum(s.max(axis=1), sink[h])
        e = np.exp(s - top[:, None])
        out[:, h] = (e @ v[:, h // group]) / (e.sum(axis=1) + np.exp(sink[h] - top))[:, None]
    return out


def attention(x, w, pre, m, eps):
    """Mixer ``attention``: convolved queries and keys, values that are the convolved keys themselves."""
    T = x.shape[0]
    H, G, d = int(m["heads"]), int(m["kv_heads"]), int(m["dim"])
    q = causal_conv(x @ w[pre + "q"].T + w[pre + "q.b"], w[pre + "q.conv"]).reshape(T, H, d)
    k = causal_conv(x @ w[pre + "k"].T + w[pre + "k.b"], w[pre + "k.conv"]).reshape(T, G, d)
    v = k
    pos = np.arange(T)
    q = rotate(over_rms(q, eps) * w[pre + "q.norm"], pos, m.get("rot"))
    k = rotate(over_rms(k, eps) * w[pre + "k.norm"], pos, m.get("rot"))
    seen = visible(int((m.get("mask") or {}).get("size") or 0), T)
    o = sink_attention(q, k, v, float(m["scale"]), seen, w[pre + "sink"])
    o = o * sigmoid(x @ w[pre + "g"].T)[:, :, None]
    return o.reshape(T, H * d) @ w[pre + "o"].T


def relu2_mlp(x, w, pre):
    return np.maximum(x @ w[pre + "up"].T, 0.0) ** 2 @ w[pre + "down"].T


def choose(z, top):
    """z [T, experts] -> (ids [T, top], weights [T, top]): the largest logits and the softmax over those alone."""
    ids = np.argsort(-z, axis=1, kind="stable")[:, :top]
    e = np.take_along_axis(z, ids, axis=1)
    e = np.exp(e - e.max(axis=1, keepdims=True))
    return ids, e / e.sum(axis=1, keepdims=True)


def mixture(x, w, pre, mlp):
    """Feed-forward ``moe``: the chosen experts' weighted sum, and the shared expert times its gate."""
    ids, weights = choose(x @ w[pre + "router"].T + w[pre + "router.b"], int(mlp["router"]["top"]))
    y = np.zeros_like(x)
    for t in range(x.shape[0]):
        for e, share in zip(ids[t], weights[t]):
            y[t] += share * relu2_mlp(x[t], w, f"{pre}e{e}.")
    if mlp.get("shared"):
        y += sigmoid(x @ w[pre + "shared.sg"].T) * relu2_mlp(x, w, pre + "shared.")
    return y


def token_side(x, rows, w, pre, eps):
    """What a layer adds from its own columns ``rows`` [T, dim] of the per-token table."""
    y = (gelu_tanh(x @ w[pre + "gate"].T) * rows) @ w[pre + "proj"].T
    return over_rms(y, eps) * w[pre + "norm"]


def run_order(cfg):
    """(layer, whether a pass of the loop starts with it), in the order in which layers run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    start, stop = int(loop["start"]), int(loop["stop"])
    body = [(i, i == start) for i in range(start, stop)] * int(loop["times"])
    return [(i, False) for i in range(start)] + body + [(i, False) for i in range(stop, n)]


def forward(cfg, w, tokens, residuals=None):
    """Logits [T, vocab]; ``residuals`` (a list) receives the residual stream after every run of a layer."""
    eps, tokens = float(cfg["norm"]["eps"]), np.asarray(tokens)
    x = start = w["embed"][tokens] * float((cfg.get("embedding") or {}).get("scale", 1.0))
    side = int((cfg.get("token_side") or {}).get("dim") or 0)
    for i, enters in run_order(cfg):
        layer, pre = cfg["layers"][i], f"l{i}."
        if enters:
            x = np.concatenate([x, start], axis=1) @ w["loop.in"].T
        x = x + attention(layer_norm(x, w[pre + "norm1"], eps), w, pre + "mix.", layer["mixer"], eps)
        if layer.get("mlp") is not None:
            x = x + mixture(layer_norm(x, w[pre + "norm2"], eps), w, pre + "mlp.", layer["mlp"])
        if side:
            x = x + token_side(x, w["side.embed"][tokens, i * side:(i + 1) * side], w, pre + "side.", eps)
        if residuals is not None:
            residuals.append(x)
    return layer_norm(x, w["final.norm"], eps) @ w["head"].T * float(cfg.get("logit_scale", 1.0))


def greedy_generate(cfg, w, prompt, new_tokens):
    tokens = list(prompt)
    for _ in range(new_tokens):
        tokens.append(int(np.argmax(forward(cfg, w, tokens)[-1])))
    return tokens[len(prompt):]
