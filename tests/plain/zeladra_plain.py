"""A plain, slow implementation of the Zeladra decoder in float64 numpy: one function per mechanism, whole sequences
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


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.maximum(z, 0.0) + np.log1p(np.exp(-np.abs(z)))


def over_rms(x, eps):
    """x divided by its root mean square over the last axis, eps inside the root."""
    return x / np.sqrt(np.mean(np.square(x), axis=-1, keepdims=True) + eps)


def layer_norm(x, weight, bias, eps):
    """Mean taken off, divided by the standard deviation (eps inside the root), weight, bias."""
    d = x - x.mean(axis=-1, keepdims=True)
    return d / np.sqrt(np.mean(d * d, axis=-1, keepdims=True) + eps) * weight + bias


def frequencies(rot):
    """One frequency per rotated pair: base^(-2i/dims); with ``rot.scaling`` the slow ones are divided by ``factor``
    and those in between blended by a ramp over the pair's index (YaRN)."""
    dims, base = int(rot["dims"]), float(rot["base"])
    f = base ** (-2.0 * np.arange(dims // 2) / dims)
    s = rot.get("scaling")
    if not s:
        return f
    factor, original = float(s["factor"]), float(s["original"])

    def index_of(turns):          # the (fractional) pair index whose wave makes ``turns`` turns in ``original`` positions
        return dims * math.log(original / (turns * 2.0 * math.pi)) / (2.0 * math.log(base))

    low = max(math.floor(index_of(float(s["fast"]))), 0)
    high = min(math.ceil(index_of(float(s["slow"]))), dims - 1)
    out = np.empty_like(f)
    for i in range(dims // 2):
        ramp = min(max((i - low) / max(high - low, 0.001), 0.0), 1.0)
        out[i] = f[i] / factor * ramp + f[i] * (1.0 - ramp)
    return out


def amplitude(rot):
    """What sines and cosines are multiplied by."""
    s = (rot or {}).get("scaling")
    return 0.1 * math.log(float(s["factor"])) + 1.0 if s else 1.0


def rotate(x, positions, rot):
    """x [T, heads, dim]: pairs (2i, 2i + 1) of the first ``dims`` numbers of a head turn by position * f_i."""
    dims = int((rot or {}).get("dims") or 0)
    if not dims:
        return x
    angle = np.asarray(positions, dtype=np.float64)[:, None] * frequencies(rot)[None, :]
    a = amplitude(rot)
    c, s = a * np.cos(angle)[:, None, :], a * np.sin(angle)[:, None, :]
    out = x.copy()
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2] = u * c - v * s
    out[..., 1:dims:2] = v * c + u * s
    return out


def visible(size, keep_first, T):
    """[T, T] booleans: which earlier positions j a position i sees; size 0: all of them."""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    causal = j <= i
    return causal if not size else causal & ((i - j < size) | (j < keep_first))


def softmax_attention(q, k, v, scale, mask):
    """q [T, H, d], k [T, G, d], v [T, G, dv] -> [T, H, dv]."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = np.zeros((T, H, v.shape[2]))
    for h in range(H):
        g = h // (H // G)
        s = np.where(mask, (q[:, h] @ k[:, g].T) * scale, -np.inf)
        e = np.exp(s - s.max(axis=1, keepdims=True))
        out[:, h] = (e / e.sum(axis=1, keepdims=True)) @ v[:, g]
    return out


def windowed_attention(x, w, pre, m, eps):
    """Mixer ``attention``."""
    T = x.shape[0]
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    pos = np.arange(T)
    q = rotate((x @ w[pre + "q"].T).reshape(T, H, d), pos, m.get("rot"))
    k = rotate((x @ w[pre + "k"].T).reshape(T, G, d), pos, m.get("rot"))
    v = (x @ w[pre + "v"].T).reshape(T, G, dv)
    mask = m.get("mask") or {}
    seen = visible(int(mask.get("size") or 0), int(mask.get("keep_first") or 0), T)
    o = softmax_attention(q, k, v, float(m["scale"]), seen)
    return o.reshape(T, H * dv) @ w[pre + "o"].T


def latent_rows(x, w, pre, m, eps):
    """What a latent layer keeps per position: (the normed latent [T, rank], the rotated key part [T, rot_dim])."""
    T = x.shape[0]
    rank = int(m["kv_rank"])
    down = x @ w[pre + "dkv"].T
    latent = over_rms(down[:, :rank], eps) * w[pre + "dkv.norm"]
    key_part = rotate(down[:, None, rank:], np.arange(T), m.get("rot"))[:, 0]
    return latent, key_part


def latent_attention(x, w, pre, m, eps, rows):
    """Mixer ``latent_attention`` over ``rows`` (this layer's own or another's, see ``latent_rows``)."""
    T = x.shape[0]
    H, d, r, dv = int(m["heads"]), int(m["dim"]), int(m["rot_dim"]), int(m["vdim"])
    latent, key_part = rows
    q = (over_rms(x @ w[pre + "dq"].T, eps) * w[pre + "dq.norm"]) @ w[pre + "uq"].T
    q = q.reshape(T, H, d + r)
    q = np.concatenate([q[..., :d], rotate(q[..., d:], np.arange(T), m.get("rot"))], axis=-1)
    k = np.concatenate([(latent @ w[pre + "uk"].T).reshape(T, H, d), np.repeat(key_part[:, None], H, axis=1)], axis=-1)
    v = (latent @ w[pre + "uv"].T).reshape(T, H, dv)
    o = softmax_attention(q, k, v, float(m["scale"]), visible(0, 0, T))
    o = o * sigmoid(x @ w[pre + "g"].T)[:, :, None]
    return o.reshape(T, H * dv) @ w[pre + "o"].T


def causal_conv(x, conv, bias):
    """Per channel over time, zeros before the start; the last column of ``conv`` [channels, taps] is the current token's."""
    T, taps = x.shape[0], conv.shape[1]
    out = np.repeat(bias[None, :], T, axis=0)
    for t in range(T):
        for j in range(taps):
            back = taps - 1 - j
            if t - back >= 0:
                out[t] += conv[:, j] * x[t - back]
    return out


def state_space(xs, B, C, dt, a_log, skip):
    """The recurrence alone.  xs [T, H, P], B and C [T, G, N], dt [T, H] (behind its softplus); per head
    S <- exp(-exp(a_log) dt) S + dt B xs^T,  y = S^T C + skip xs."""
    T, H, P = xs.shape
    G, N = B.shape[1:]
    y = np.zeros_like(xs)
    for h in range(H):
        g = h // (H // G)
        S = np.zeros((N, P))
        for t in range(T):
            S = math.exp(-math.exp(a_log[h]) * dt[t, h]) * S + dt[t, h] * np.outer(B[t, g], xs[t, h])
            y[t, h] = S.T @ C[t, g] + skip[h] * xs[t, h]
    return y


def gated_group_norm(y, z, weight, groups, eps):
    """y * silu(z), then each of ``groups`` equal parts of a row over its own root mean square, then the weight."""
    T, width = y.shape
    y = y * silu(z)
    return over_rms(y.reshape(T, groups, width // groups), eps).reshape(T, width) * weight


def mamba2(x, w, pre, m, eps):
    """Mixer ``mamba2``."""
    T = x.shape[0]
    H, P, N, G = int(m["heads"]), int(m["vdim"]), int(m["state"]), int(m["groups"])
    inner = H * P
    proj = x @ w[pre + "in"].T
    z, xbc, dt = proj[:, :inner], proj[:, inner:2 * inner + 2 * G * N], proj[:, 2 * inner + 2 * G * N:]
    xbc = silu(causal_conv(xbc, w[pre + "conv"], w[pre + "conv.b"]))
    xs = xbc[:, :inner].reshape(T, H, P)
    B = xbc[:, inner:inner + G * N].reshape(T, G, N)
    C = xbc[:, inner + G * N:].reshape(T, G, N)
    y = state_space(xs, B, C, softplus(dt + w[pre + "dt_bias"]), w[pre + "A_log"], w[pre + "D"])
    y = gated_group_norm(y.reshape(T, inner), z, w[pre + "norm"], int(m["norm_groups"]), eps)
    return y @ w[pre + "o"].T


def feed_forward(x, w, pre):
    return (silu(x @ w[pre + "gate"].T) * (x @ w[pre + "up"].T)) @ w[pre + "down"].T


def hyper_connection(streams, w, pre, sublayer):
    """streams [s, T, width]: the sublayer reads a weighted sum of them; all of them are mixed anew and each takes its
    share of the sublayer's output."""
    read, mix, write = w[pre + "in"], w[pre + "mix"], w[pre + "out"]
    y = sublayer(np.einsum("s,stw->tw", read, streams))
    return np.einsum("st,skw->tkw", mix, streams) + write[:, None, None] * y[None]


def forward(cfg, w, tokens, residuals=None):
    """Logits [T, vocab]; ``residuals`` (a list) receives the sum of the streams after every layer."""
    eps = float(cfg["norm"]["eps"])
    x = w["embed"][np.asarray(tokens)] * float(cfg["embedding"]["scale"])
    streams = np.repeat(x[None], int(cfg["streams"]), axis=0)
    kept = {}
    for i, layer in enumerate(cfg["layers"]):
        m, base = layer["mixer"], f"l{i}."
        pre = base + "mix."

        def mixer(u):
            h = layer_norm(u, w[base + "norm1"], w[base + "norm1.b"], eps)
            if layer["type"] == "mamba2":
                return mamba2(h, w, pre, m, eps)
            if layer["type"] == "attention":
                return windowed_attention(h, w, pre, m, eps)
            source = m.get("kv_from")
            if source is None:
                kept[i] = latent_rows(h, w, pre, m, eps)
            return latent_attention(h, w, pre, m, eps, kept[i if source is None else int(source)])

        streams = hyper_connection(streams, w, base + "hc1.", mixer)
        if layer.get("mlp") is not None:
            streams = hyper_connection(streams, w, base + "hc2.", lambda u: feed_forward(
                layer_norm(u, w[base + "norm2"], w[base + "norm2.b"], eps), w, base + "mlp."))
        if residuals is not None:
            residuals.append(streams.sum(axis=0))
    h = layer_norm(streams.sum(axis=0), w["final.norm"], w["final.norm.b"], eps)
    return h @ w["head"].T


def greedy_generate(cfg, w, prompt, new_tokens):
    tokens = list(prompt)
    for _ in range(new_tokens):
        tokens.append(int(np.argmax(forward(cfg, w, tokens)[-1])))
    return tokens[len(prompt):]
