"""Zeladra on the GPU against the plain implementation (``plain/zeladra_plain.py``): kernels and mechanisms alone, then
whole models through the step function (whole prompts, single tokens, portions down to two tokens, mixed batches, slots
and pages that are used again, far keys, slow states, the edges of windows, kept first positions, pages and chunks of the
recurrence), and greedy generation through the engine.

The plain implementation runs whole sequences in float64; every check feeds the engine's logits at all positions of a
request, however they were cut into steps, against its logits of the whole sequence.
"""
import copy
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import zeladra_helpers as Z
from helpers import assert_tokens_follow_plain, rel_err
from plain import zeladra_plain as P

pytestmark = pytest.mark.gpu

TOL = {"float32": 5e-5, "bfloat16": 0.1}     # of a position's largest logit
SHARP_TOL = {"float32": 1e-4, "bfloat16": 8e-2}    # peaked attention weights amplify the rounding of queries and keys


def open_runner(folder, dtype, pages=64, page=8, slots=4):
    from vipera_rs_amd.engine.runner import ModelRunner

    return ModelRunner.from_folder(folder, dtype=dtype, block_size=page, num_blocks=pages, num_slots=slots)


def replay(runner, requests, plan, keep=()):
    """Run ``plan`` (steps of (request, tokens) pairs) and return every request's logits at all its positions.
    A request gives back its pages and slot when its last token has run, unless it is in ``keep``."""
    from vipera_rs_amd.engine.batch import StepEntry

    at = {r: 0 for r in requests}
    rows = {r: [] for r in requests}
    for step in plan:
        entries = []
        for r, size in step:
            runner.cache.reserve(r, at[r], at[r] + size)
            entries.append(StepEntry(r, at[r], requests[r][at[r]:at[r] + size], list(range(size))))
        logits = runner.step(entries).float().cpu().numpy()
        row = 0
        for r, size in step:
            rows[r].append(logits[row:row + size])
            row += size
            at[r] += size
            runner.cache.advance(r, at[r])
            if at[r] == len(requests[r]) and r not in keep:
                runner.cache.release(r)
    return {r: np.concatenate(v) for r, v in rows.items() if v}


def check(got, want, tol, label=""):
    """Position by position, so that one wrong token cannot hide among many right ones.  In 32-bit every position must
    hold.  In bfloat16 a narrow recurrence amplifies the rounding of single tokens (products of three convolved factors
    behind a norm of a dozen numbers): there one position in twenty may be over, and none by more than three times, which
    a fault of a page, a slot, a state or a mask still exceeds."""
    strict = tol < 1e-3
    over, total = [], 0
    for r in got:
        assert want[r].shape == got[r].shape
        for t in range(got[r].shape[0]):
            err = rel_err(got[r][t], want[r][t])
            total += 1
            assert err < (tol if strict else 3 * tol), \
                f"{label}: request {r}, position {t} of {got[r].shape[0]}: relative error {err:.3g}"
            if err >= tol:
                over.append((r, t, round(err, 3)))
    assert len(over) <= total // 20, f"{label}: {len(over)} of {total} positions are over {tol}: {over[:8]}"


def portions(total, sizes):
    out, k = [], 0
    while total:
        size = min(sizes[k % len(sizes)], total)
        out.append(size)
        total -= size
        k += 1
    return out


def dev(a, dtype=torch.float32):
    return torch.from_numpy(np.ascontiguousarray(a)).to(dtype).cuda()


# --- kernels alone ------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("streams, width", [(1, 64), (2, 48), (3, 50), (4, 1028), (4, 2500), (5, 72), (8, 33), (2, 5000), (3, 2049)])
def test_streams_joined_read_and_normed(streams, width, dtype):
    """Every register layout of the kernel (vector and scalar columns, a fixed and any number of streams): the output
    joins, the streams are written in place, weighed and normed; a first reading of equal streams; chosen rows."""
    from vipera_rs_amd.ops import kernels

    rng = np.random.default_rng(streams * 1000 + width)
    tokens, eps = 5, 1e-3
    x, y = rng.standard_normal((tokens, streams, width)), rng.standard_normal((tokens, width))
    mix, share, read = rng.standard_normal((streams, streams)), rng.standard_normal(streams), rng.standard_normal(streams)
    weight, bias = 1 + 0.2 * rng.standard_normal(width), 0.3 * rng.standard_normal(width)
    tol = 1e-5 if dtype == torch.float32 else 1e-2
    new = np.einsum("st,ksw->ktw", mix, x) + share[None, :, None] * y[:, None]
    u = np.einsum("s,ksw->kw", read, new)
    norms = {"none": u, "rms": P.over_rms(u, eps) * weight, "layer": P.layer_norm(u, weight, bias, eps)}
    for norm, want in norms.items():
        held, out = dev(x), torch.empty((tokens, width), dtype=dtype, device="cuda")
        kernels.streams_step(held, streams, dev(y), dev(mix), dev(share), held, dev(read), out, norm,
                             dev(weight) if norm != "none" else None, dev(bias) if norm == "layer" else None, eps)
        assert rel_err(held.cpu().numpy(), new) < 1e-6 and rel_err(out.float().cpu().numpy(), want) < tol, norm
    # all streams still one row: the first reading, and the first joining into a buffer of its own
    row = rng.standard_normal((tokens, width))
    out = torch.empty((tokens, width), dtype=dtype, device="cuda")
    kernels.streams_step(dev(row), streams, None, None, None, None, dev(read), out, "layer", dev(weight), dev(bias), eps)
    assert rel_err(out.float().cpu().numpy(), P.layer_norm(read.sum() * row, weight, bias, eps)) < tol
    held = torch.full((tokens, streams, width), float("nan"), device="cuda")
    kernels.streams_step(dev(row), streams, dev(y), dev(mix), dev(share), held, None, None)
    first = mix.sum(axis=0)[None, :, None] * row[:, None] + share[None, :, None] * y[:, None]
    assert rel_err(held.cpu().numpy(), first) < 1e-6
    # some rows of the plain sum, the last output still to join; the streams stay as they are
    rows = torch.tensor([4, 0, 2], dtype=torch.int32, device="cuda")
    held, out = dev(x), torch.empty((3, width), dtype=dtype, device="cuda")
    kernels.streams_step(held, streams, dev(y), dev(mix), dev(share), None, None, out, "layer", dev(weight), dev(bias), eps, rows)
    want = P.layer_norm(new.sum(axis=1), weight, bias, eps)[[4, 0, 2]]
    assert rel_err(out.float().cpu().numpy(), want) < tol and np.array_equal(held.cpu().numpy(), np.float32(x))


def test_a_layer_norm_of_a_large_mean_keeps_its_digits():
    from vipera_rs_amd.ops import kernels

    x = np.float32(1000.0 + np.random.default_rng(1).standard_normal((3, 320)))
    out = torch.empty((3, 320), device="cuda")
    kernels.streams_step(dev(x), 1, None, None, None, None, None, out, "layer", None, None, 1e-5)
    assert rel_err(out.cpu().numpy(), P.layer_norm(np.float64(x), 1.0, 0.0, 1e-5)) < 2e-4


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_streams_and_layer_norms_beside_other_norms(dtype):
    """The streams with a norm that their kernel applies itself (layer, RMS) and one that it does not know (Dynamic Tanh),
    and a layer norm behind a sublayer, as another design may put them together."""
    from vipera_rs_amd.config.base import PartSpec
    from vipera_rs_amd.parts import part_class
    from vipera_rs_amd.parts.streams import ResidualStreams
    from vipera_rs_amd.runtime import Runtime

    rng, runtime = np.random.default_rng(6), Runtime("cuda:0", dtype)
    tokens, width, eps, tol = 5, 24, 1e-5, 1e-5 if dtype == "float32" else 1e-2
    weight, bias, alpha = 1 + 0.2 * rng.standard_normal(width), 0.3 * rng.standard_normal(width), 0.7
    row, y1, y2 = (rng.standard_normal((tokens, width)) for _ in range(3))
    mix, share, read = rng.standard_normal((3, 3)), rng.standard_normal(3), rng.standard_normal(3)
    two = np.repeat(row[None], 3, axis=0)
    for y in (y1, y2):
        two = np.einsum("st,skw->tkw", mix, two) + share[:, None, None] * y
    u = np.einsum("s,skw->kw", read, two)
    kinds = {"layernorm": lambda x: P.layer_norm(x, weight, bias, eps), "rmsnorm": lambda x: P.over_rms(x, eps) * weight,
             "dyt": lambda x: np.tanh(alpha * x) * weight + bias}
    for kind, apply in kinds.items():
        norm = part_class("norm", kind)(PartSpec(kind, {"width": width, "eps": eps, "name": "n", "tensor": "n"}), "", runtime)
        norm.load({"n": dev(weight), "n.b": dev(bias), "n.alpha": dev(np.array(alpha))})
        x = ResidualStreams(dev(row), 3)
        x.leave(dev(y1), dev(mix), dev(share))
        x.leave(dev(y2), dev(mix), dev(share))           # nobody has read in between: the first joins now
        rows = torch.tensor([3, 1], dtype=torch.int32, device="cuda")
        assert rel_err(x.read_rows(norm, rows, runtime).float().cpu().numpy(), apply(two.sum(axis=0))[[3, 1]]) < tol, kind
        assert rel_err(x.read(dev(read), norm, runtime).float().cpu().numpy(), apply(u)) < tol, kind
        assert rel_err(x.total().cpu().numpy(), two.sum(axis=0)) < 1e-6 and x.pending is None
        if kind == "layernorm":
            stream = dev(row)
            out = norm.add_into(dev(y1), stream, follow=norm)
            assert rel_err(stream.cpu().numpy(), row + apply(y1)) < tol
            assert rel_err(out.float().cpu().numpy(), apply(row + apply(y1))) < 2 * tol
            assert rel_err(norm.add_into(dev(y2), stream, as_input=True).float().cpu().numpy(), row + apply(y1) + apply(y2)) < 2 * tol


SPACES = [(1, 1, 4, 1), (4, 2, 12, 20), (6, 3, 10, 7), (2, 1, 64, 128), (8, 2, 40, 64), (3, 1, 16, 33), (2, 2, 24, 200), (4, 1, 20, 256)]


@pytest.mark.parametrize("heads, groups, vdim, states", SPACES)
def test_the_state_space_recurrence_token_by_token_and_in_chunks(heads, groups, vdim, states):
    """Entries of unequal lengths in one launch, some going on from a state, in both forms: portions that end on, before
    and behind a chunk's edge; the two forms leave the same state."""
    from vipera_rs_amd.ops import kernels

    rng = np.random.default_rng(heads * 100 + states)
    counts, firsts = [1, 63, 64, 65, 2, 130, 7], [0, 0, 9, 0, 5, 64, 0]
    T, E = sum(counts), len(counts)
    inner, gn = heads * vdim, groups * states
    buffer = rng.standard_normal((T, inner + 2 * gn))
    dt_raw = rng.standard_normal((T, heads + 3)) * 2.0
    dt_bias, a_log, skip = rng.uniform(-2, 0.5, heads), rng.uniform(-3, 1, heads), rng.standard_normal(heads)
    floats = heads * kernels.state_space_head_floats(vdim, states)
    padded = kernels.state_space_head_floats(1, states)
    before = rng.standard_normal((E + 1, heads, vdim, padded))
    starts = np.concatenate([[0], np.cumsum(counts)])
    slots = rng.permutation(E)
    y_want, s_want = np.zeros((T, inner)), {}
    for e in range(E):
        S = np.zeros((heads, states, vdim)) if firsts[e] == 0 else before[slots[e], :, :, :states].transpose(0, 2, 1).copy()
        for t in range(starts[e], starts[e + 1]):
            for h in range(heads):
                g = h // (heads // groups)
                x = buffer[t, h * vdim:(h + 1) * vdim]
                B = buffer[t, inner + g * states:inner + (g + 1) * states]
                C = buffer[t, inner + gn + g * states:inner + gn + (g + 1) * states]
                d = P.softplus(dt_raw[t, h] + dt_bias[h])
                S[h] = np.exp(-np.exp(a_log[h]) * d) * S[h] + d * np.outer(B, x)
                y_want[t, h * vdim:(h + 1) * vdim] = S[h].T @ C + skip[h] * x
        s_want[e] = S.transpose(0, 2, 1)
    buf, dts = dev(buffer), dev(dt_raw)
    i32 = lambda a: dev(np.asarray(a), torch.int32)
    for step_tokens in (0, 6, 64, 10 ** 6):
        rows = before.copy()
        rows[..., states:] = np.nan                                   # what lies in the padding reaches nothing
        for e in range(E):
            if firsts[e] == 0:
                rows[slots[e]] = np.nan
        state = dev(rows.reshape(E + 1, floats))
        out = torch.full((T, inner), float("nan"), device="cuda")
        kernels.state_space(buf[:, :inner], buf[:, inner:inner + gn], buf[:, inner + gn:], dts[:, :heads], dev(dt_bias), dev(a_log),
                            dev(skip), state, i32(starts), i32(firsts), i32(slots), heads, groups, vdim, states, out, E,
                            min(counts), max(counts), step_tokens)
        got = out.cpu().numpy()
        left = state.cpu().numpy().reshape(E + 1, heads, vdim, padded)
        for e in range(E):
            assert rel_err(got[starts[e]:starts[e + 1]], y_want[starts[e]:starts[e + 1]]) < 2e-5, (step_tokens, counts[e])
            assert rel_err(left[slots[e], ..., :states], s_want[e]) < 2e-5, (step_tokens, counts[e])
        assert np.array_equal(left[E, ..., :states], np.float32(before[E, ..., :states]))          # nobody's row


def test_step_sizes_of_hundreds_cost_no_digits():
    """Sums of the decays' exponents in the thousands within a chunk: a difference of two of them near zero still counts."""
    from vipera_rs_amd.ops import kernels

    rng = np.random.default_rng(5)
    T, N = 64, 16
    buffer = rng.standard_normal((T, 16 + 2 * N))
    dt = rng.uniform(50.0, 90.0, (T, 1))
    dt[1::2] = 1e-3                                    # every second token keeps what the one before left
    raw = np.log(np.expm1(np.minimum(dt, 30.0))) + np.maximum(dt - 30.0, 0.0)
    raw32 = np.float64(np.float32(raw))
    want = P.state_space(buffer[:, None, :16], buffer[:, None, 16:16 + N], buffer[:, None, 16 + N:], P.softplus(raw32),
                         np.array([0.5]), np.array([0.3]))[:, 0]
    buf, out = dev(buffer), torch.empty((T, 16), device="cuda")
    i32 = lambda a: dev(np.asarray(a), torch.int32)
    kernels.state_space(buf[:, :16], buf[:, 16:16 + N], buf[:, 16 + N:], dev(raw), dev([0.0]), dev([0.5]), dev([0.3]),
                        torch.zeros((2, 16 * N), device="cuda"), i32([0, T]), i32([0]), i32([0]), 1, 1, 16, N, out, 1, T, T)
    for t in range(T):
        assert rel_err(out[t].cpu().numpy(), want[t]) < 2e-5, t


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width, parts", [(48, 2), (40, 4), (96, 1), (2048, 8), (5000, 1), (4100, 1), (1024, 4), (36, 12)])
def test_gated_norm_in_parts(width, parts, dtype):
    from vipera_rs_amd.ops import kernels

    rng = np.random.default_rng(width)
    y, z, weight = rng.standard_normal((6, width)), rng.standard_normal((6, width + 7)), 1 + 0.2 * rng.standard_normal(width)
    out = torch.empty((6, width), dtype=dtype, device="cuda")
    kernels.gated_part_norm(dev(y), dev(z)[:, 3:3 + width], dev(weight), 1e-5, parts, out)
    want = P.gated_group_norm(y, z[:, 3:3 + width], weight, parts, 1e-5)
    assert rel_err(out.float().cpu().numpy(), want) < (1e-5 if dtype == torch.float32 else 1e-2)


@pytest.mark.parametrize("channels, taps", [(20, 4), (24, 1), (300, 2), (515, 3), (64, 6), (1028, 4)])
def test_the_convolution_over_portions_and_single_tokens(channels, taps):
    """Entries of every length around the number of taps and around the tokens a workgroup takes, with and without
    inputs of their own in the state; then a step of single tokens (a kernel of its own)."""
    from vipera_rs_amd.ops import kernels

    rng = np.random.default_rng(channels + taps)
    conv, bias = rng.standard_normal((channels, taps)), rng.standard_normal(channels)
    counts = [1, 2, taps, taps + 1, 15, 16, 17, 40]
    histories = [rng.standard_normal((n, channels)) for n in (0, 1, 0, 2, 5, 0, taps, 1)]
    E, offset = len(counts), 8
    i32 = lambda a: dev(np.asarray(a), torch.int32)
    slots = rng.permutation(E)
    state = torch.full((E + 1, offset + (taps - 1) * channels), float("nan"), device="cuda")
    for e, past in enumerate(histories):
        if len(past):
            kept = np.concatenate([np.zeros((taps - 1, channels)), past])[len(past):]
            state[slots[e], offset:] = dev(kept.reshape(-1))
    whole = [list(past) for past in histories]
    for sizes in (counts, [1] * E, [3] + [1] * (E - 1), [1] * E, [5, 70, 1, 130, 16, 33, 2, 64], [2] * E):
        T = sum(sizes)
        starts = np.concatenate([[0], np.cumsum(sizes)])
        x = rng.standard_normal((T, channels + 5))
        out = torch.empty((T, channels), device="cuda")
        run = torch.empty((T, channels), dtype=torch.bfloat16, device="cuda")
        kernels.causal_conv(dev(x)[:, 2:2 + channels], dev(conv), dev(bias), state, offset, i32(np.repeat(np.arange(E), sizes)),
                            i32(starts), i32([len(past) for past in whole]), i32(slots), out, run, E)
        for e in range(E):
            whole[e] += list(x[starts[e]:starts[e + 1], 2:2 + channels])
            want = P.silu(P.causal_conv(np.array(whole[e]), conv, bias))[-sizes[e]:]
            assert rel_err(out[starts[e]:starts[e + 1]].cpu().numpy(), want) < 1e-5, (sizes, e)
            assert rel_err(run[starts[e]:starts[e + 1]].float().cpu().numpy(), want) < 1e-2
    assert torch.isnan(state[E]).all()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_latents_normed_rotated_and_paged_in_one_launch(dtype):
    from vipera_rs_amd.ops import kernels

    rng = np.random.default_rng(7)
    tokens, rank, rot, q_rank, block = 11, 20, 12, 28, 4
    x = rng.standard_normal((tokens, rank + rot + q_rank + 3))
    weight, q_weight = 1 + 0.2 * rng.standard_normal(rank), 1 + 0.2 * rng.standard_normal(q_rank)
    freq = rng.uniform(0.01, 1.0, rot // 2)
    positions = np.arange(3, 3 + tokens)
    table = np.array([[5, 1, 7, 2]])
    k = torch.zeros((9, 1, block, rank + rot), dtype=dtype, device="cuda")
    v = torch.zeros((9, 1, rank + rot, block), dtype=dtype, device="cuda")
    c_q = torch.empty((tokens, q_rank), dtype=dtype, device="cuda")
    i32 = lambda a: dev(np.asarray(a), torch.int32)
    down = dev(x)
    args = (dev(weight), 1e-5, rank, rot, rot, i32(positions), dev(freq), i32(np.zeros(tokens)), i32(table), k, v, 1.3)
    kernels.latent_prepare(down[:, :rank + rot], *args, x_q=down[:, rank + rot:rank + rot + q_rank], q_weight=dev(q_weight), q_out=c_q)
    angle = positions[:, None] * freq[None, :]
    lo, hi = x[:, rank:rank + rot // 2], x[:, rank + rot // 2:rank + rot]
    turned = 1.3 * np.concatenate([lo * np.cos(angle) - hi * np.sin(angle), hi * np.cos(angle) + lo * np.sin(angle)], axis=1)
    rows = np.concatenate([P.over_rms(x[:, :rank], 1e-5) * weight, turned], axis=1)
    tol = 1e-5 if dtype == torch.float32 else 1e-2
    for t, p in enumerate(positions):
        page = table[0, p // block]
        assert rel_err(k[page, 0, p % block].float().cpu().numpy(), rows[t]) < tol
        assert torch.equal(k[page, 0, p % block], v[page, 0, :, p % block])
    q_want = P.over_rms(x[:, rank + rot:rank + rot + q_rank], 1e-5) * q_weight
    assert rel_err(c_q.float().cpu().numpy(), q_want) < tol
    # a layer that keeps no rows: only the queries' latent
    kept = k.clone()
    c_q.zero_()
    kernels.latent_prepare(None, None, *args[1:], x_q=down[:, rank + rot:rank + rot + q_rank], q_weight=dev(q_weight), q_out=c_q)
    assert rel_err(c_q.float().cpu().numpy(), q_want) < tol and torch.equal(k, kept)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("k, n", [(24, 16), (18, 10), (136, 130)])
def test_a_product_per_head_with_a_gate_per_head(dtype, k, n):
    from vipera_rs_amd.ops import kernels

    rng = np.random.default_rng(k)
    tokens, heads = 70, 3
    a, w = dev(rng.standard_normal((tokens, heads * (k + 8))), dtype), dev(rng.standard_normal((heads, n, k)), dtype)
    gate = rng.standard_normal((tokens, heads + 2))
    out = torch.empty((tokens, heads * n), dtype=dtype, device="cuda")
    kernels.head_linear(a, k + 8, k, w, out, n, gate=dev(gate)[:, 1:1 + heads])
    left = a.float().cpu().numpy().astype(np.float64).reshape(tokens, heads, k + 8)[..., :k]
    want = np.stack([left[:, h] @ w[h].float().cpu().numpy().astype(np.float64).T for h in range(heads)], axis=1)
    want = want * P.sigmoid(gate[:, 1:1 + heads])[:, :, None]
    assert rel_err(out.float().cpu().numpy(), want.reshape(tokens, heads * n)) < (1e-5 if dtype == torch.float32 else 1e-2)


def test_amplitudes_of_rotations():
    """The amplitude of sines and cosines in every kernel that rotates: the table of a step's angles, the queries' rotated
    part and the kernel that lays heads out."""
    from vipera_rs_amd.ops import kernels

    rng = np.random.default_rng(8)
    tokens, heads, dim, rot = 6, 2, 16, 8
    freq, positions = rng.uniform(0.01, 1.0, rot // 2), rng.integers(0, 3000, tokens)
    pos = dev(positions, torch.int32)
    angle = np.float64(np.float32(positions)[:, None] * np.float32(freq)[None, :])
    table = kernels.rope_angles(pos, dev(freq), tokens, 1.5).cpu().numpy()
    assert np.allclose(table, 1.5 * np.stack([np.sin(angle), np.cos(angle)], axis=-1), atol=1e-5)

    def turned(x):
        lo, hi = x[..., :rot // 2], x[..., rot // 2:rot]
        c, s = 1.5 * np.cos(angle)[:, None], 1.5 * np.sin(angle)[:, None]
        return np.concatenate([lo * c - hi * s, hi * c + lo * s, x[..., rot:]], axis=-1)
    x = rng.standard_normal((tokens, heads, dim))
    out = torch.empty((tokens, heads * dim), device="cuda")
    kernels.latent_q_rotate(dev(x.reshape(tokens, -1)), dim, 0, out, dim, 0, heads, dim, rot, pos, dev(freq), 1.5)
    assert rel_err(out.cpu().numpy().reshape(x.shape), turned(x)) < 1e-5
    qkv = torch.empty((tokens, 3 * dim), device="cuda")
    kernels.head_prepare(dev(x.reshape(tokens, -1).repeat(2, axis=1)[:, :3 * dim]), None, None, False, False, 0.0, pos, dev(freq),
                         rot, 1, 1, 1, dim, dim, dim, qkv, amplitude=1.5)
    want = x.reshape(tokens, -1).repeat(2, axis=1)[:, :3 * dim].reshape(tokens, 3, dim)
    want = np.concatenate([turned(want[:, :2]), want[:, 2:]], axis=1)
    assert rel_err(qkv.cpu().numpy().reshape(tokens, 3, dim), want) < 1e-5


# --- each mechanism alone, as a model of one layer -------------------------------------------------------------------
ONE_LAYER = {
    # the recurrence: shared and own B and C, parts of the norm, one tap and six, odd widths, several tiles and chunks
    "space": Z.single(Z.mamba2(4, 16, 16, groups=2, norm_groups=2)),
    "space_one_head_one_tap": Z.single(Z.mamba2(1, 8, 1, conv=1), width=40),
    "space_odd": Z.single(Z.mamba2(6, 10, 7, groups=3, norm_groups=4, conv=6), width=50),
    "space_groups_equal_heads": Z.single(Z.mamba2(3, 12, 36, groups=3, norm_groups=3, conv=2), width=48),
    "space_wide": Z.single(Z.mamba2(4, 72, 130, groups=1, norm_groups=1, conv=3), width=136),
    # latent attention: with and without the blend, widths that are no multiples of 8, one head, values wider than keys
    "latent": Z.single(Z.latent(4, 16, 8, 16, 24, 24, base=500.0, scaling=Z.YARN)),
    "latent_odd": Z.single(Z.latent(3, 10, 6, 14, 20, 19, base=77.0, scale=0.4), width=50),
    "latent_one_head_wide_values": Z.single(Z.latent(1, 8, 4, 40, 16, 28, scaling=(2.0, 16, 4.0, 4.0)), width=40),
    "latent_ranks_above_the_width": Z.single(Z.latent(2, 64, 32, 48, 96, 160, base=1e6, scaling=(32.0, 4096, 32.0, 1.0)), width=48),
    "latent_wide": Z.single(Z.latent(8, 72, 64, 24, 136, 192), width=136),
    # windows: full, partial and no rotation, kept positions, none, more kept than seen, values of other widths
    "window": Z.single(Z.windowed(4, 2, 16, 16, 7, keep_first=3, rot_dims=8, base=300.0)),
    "window_none_kept_narrow_values": Z.single(Z.windowed(3, 1, 24, 8, 12), width=48),
    "window_no_rotation_odd": Z.single(Z.windowed(2, 2, 10, 6, 5, keep_first=1, rot_dims=0, scale=0.4), width=50),
    "window_more_kept_than_seen": Z.single(Z.windowed(3, 1, 8, 40, 4, keep_first=11, rot_dims=2, scale=0.5), width=40),
    "window_wide": Z.single(Z.windowed(5, 5, 72, 136, 100, keep_first=70, rot_dims=32), width=136),
    # the feed-forward, and numbers of streams
    "dense": Z.single(Z.windowed(1, 1, 8, 8, 6), Z.dense(56), width=48, streams=1),
    "dense_odd_three_streams": Z.single(Z.windowed(1, 1, 8, 8, 6), Z.dense(30), width=50, streams=3),
    "dense_four_streams": Z.single(Z.mamba2(2, 8, 8), Z.dense(130), width=136, streams=4, eps=1e-2),
    "seven_streams": Z.single(Z.mamba2(2, 8, 8), Z.dense(24), width=40, streams=7),
}
LONG = {"space_wide", "latent_wide", "window_wide", "dense_four_streams"}    # a prompt of 330 tokens: several tiles


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(ONE_LAYER))
def test_a_mechanism_alone_whole_prompt_then_single_tokens(tmp_path, name, dtype):
    cfg = ONE_LAYER[name]
    folder = Z.make_folder(tmp_path / name, cfg, 11)
    plain_cfg, w = Z.load_folder(folder)
    first = 330 if name in LONG else 45
    requests = {0: Z.tokens_of(cfg["vocab"], first, 1), 1: Z.tokens_of(cfg["vocab"], 30, 2)}
    want = {r: P.forward(plain_cfg, w, t) for r, t in requests.items()}
    runner = open_runner(folder, dtype)
    plan = [[(0, first)], [(1, 19)]] + [[(1, 1)]] * 11
    check(replay(runner, requests, plan), want, TOL[dtype], name)
    assert runner.cache.check() == "" and runner.cache.live_requests() == 0


def test_pages_of_two_positions_take_the_general_kernel(tmp_path):
    folder = Z.make_folder(tmp_path / "z1", Z.Z1, 21)
    cfg, w = Z.load_folder(folder)
    tokens = Z.tokens_of(cfg["vocab"], 50, 3)
    runner = open_runner(folder, "float32", pages=64, page=2)
    for plan in ([[(0, 50)]], [[(0, 31)]] + [[(0, 1)]] * 19):
        check(replay(runner, {0: tokens}, plan), {0: P.forward(cfg, w, tokens)}, TOL["float32"], "pages of two")


def test_the_residual_after_every_layer(tmp_path):
    """32-bit, layer by layer: a fault shows in the layer that has it, not only in the logits."""
    for name, model in (("z1", Z.Z1), ("z2", Z.Z2)):
        folder = Z.make_folder(tmp_path / name, model, 21)
        plain_cfg, w = Z.load_folder(folder)
        tokens = Z.tokens_of(model["vocab"], 80, 5)
        residuals = []
        want = P.forward(plain_cfg, w, tokens, residuals)
        runner = open_runner(folder, "float32")
        seen = []
        for layer in runner.model.layers:
            def wrapped(x, *args, _forward=layer.forward, **kwargs):
                _forward(x, *args, **kwargs)
                seen.append(x.total())
            layer.forward = wrapped
        got = replay(runner, {0: tokens}, [[(0, 80)]])
        assert len(seen) == len(residuals) == len(model["layers"])
        for index, (mine, ref) in enumerate(zip(seen, residuals)):
            assert rel_err(mine.cpu().numpy(), ref) < 2e-5, f"{name}: after layer {index} ({model['layers'][index]['type']})"
        check(got, {0: want}, TOL["float32"], name)       # reading the sum on the way changed nothing


# --- whole models through the step function ------------------------------------------------------------------------
@pytest.fixture(scope="module")
def z1(tmp_path_factory):
    folder = Z.make_folder(tmp_path_factory.mktemp("z1"), Z.Z1, 31)
    return (folder,) + Z.load_folder(folder)


@pytest.fixture(scope="module")
def z2(tmp_path_factory):
    folder = Z.make_folder(tmp_path_factory.mktemp("z2"), Z.Z2, 32)
    return (folder,) + Z.load_folder(folder)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which", ["z1", "z2"])
def test_token_by_token_equals_the_whole_prompt(request, which, dtype):
    folder, cfg, w = request.getfixturevalue(which)
    tokens = Z.tokens_of(cfg["vocab"], 150, 7)
    want = {0: P.forward(cfg, w, tokens)}
    runner = open_runner(folder, dtype, page=4 if which == "z2" and dtype == "float32" else 8, pages=128)
    whole = replay(runner, {0: tokens}, [[(0, 150)]])
    check(whole, want, TOL[dtype], "whole")
    single = replay(runner, {0: tokens}, [[(0, 1)]] * 150)      # long decoding from the very first token
    check(single, want, TOL[dtype], "token by token")
    if dtype == "float32":   # the two ways differ by rounding only
        assert rel_err(single[0], whole[0].astype(np.float64)) < 2e-5


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("sizes", [[2], [3, 2, 17, 2, 5], [13, 1, 8], [16, 2], [64, 7], [6, 7], [65, 63, 66]])
@pytest.mark.parametrize("which", ["z1", "z2"])
def test_portions_of_a_prompt(request, which, sizes, dtype):
    """Portions cut inside pages (8), at their borders, inside windows (7 and 11), around a chunk of the recurrence (64)
    and around the length from which a portion runs in chunks."""
    folder, cfg, w = request.getfixturevalue(which)
    n = 200 if max(sizes) > 20 else 83
    tokens = Z.tokens_of(cfg["vocab"], n, 9)
    want = {0: P.forward(cfg, w, tokens)}
    runner = open_runner(folder, dtype)
    plan = [[(0, size)] for size in portions(n, sizes)]
    check(replay(runner, {0: tokens}, plan), want, TOL[dtype], f"portions {sizes}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which", ["z1", "z2"])
def test_a_mixed_batch_equals_each_request_alone(request, which, dtype):
    """Up to four live requests of unequal lengths: portions of some beside single tokens of others; requests end and
    later ones take their slots and pages; the pool holds less than all requests together; one request sits a step out."""
    folder, cfg, w = request.getfixturevalue(which)
    lengths = {0: 61, 1: 9, 2: 40, 3: 1, 4: 33, 5: 26, 6: 2}
    requests = {r: Z.tokens_of(cfg["vocab"], n, 40 + r) for r, n in lengths.items()}
    want = {r: P.forward(cfg, w, t) for r, t in requests.items()}
    plan = [[(0, 20), (1, 2), (2, 7)], [(0, 1), (1, 7), (2, 2), (3, 1)], [(0, 17), (2, 1), (4, 30)],
            [(0, 2), (2, 30), (4, 1), (5, 5)], [(0, 1), (4, 1), (5, 2), (6, 2)], [(0, 20), (4, 1), (5, 19)]]
    runner = open_runner(folder, dtype, pages=22, page=8, slots=4)    # 176 positions for 172 tokens in all
    got = replay(runner, requests, plan)
    assert {r: v.shape[0] for r, v in got.items()} == lengths
    check(got, want, TOL[dtype], "mixed")
    assert runner.cache.check() == "" and runner.cache.live_requests() == 0


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_slot_and_pages_that_are_used_again_start_clean(z1, dtype):
    """One slot and few pages: every request runs in the state row and the pages the one before it left full."""
    folder, cfg, w = z1
    runner = open_runner(folder, dtype, pages=9, page=8, slots=1)
    for r, (n, cut) in enumerate([(60, [60]), (41, [5, 2, 30, 1, 1, 1, 1]), (17, [1] * 17), (64, [33, 31]), (70, [2, 68])]):
        tokens = Z.tokens_of(cfg["vocab"], n, 70 + r)
        got = replay(runner, {r: tokens}, [[(r, size)] for size in cut])
        check(got, {r: P.forward(cfg, w, tokens)}, TOL[dtype], f"request {r} in the used slot")
        assert runner.cache.slot(r) == -1 and runner.cache.free_slots() == 1


def test_state_rows_and_pages_full_of_nan_do_not_reach_a_new_request(z2):
    """A slot's row and a pool's pages may hold anything when a request takes them."""
    folder, cfg, w = z2
    runner = open_runner(folder, "float32", slots=2)
    for state in runner.storage.state:
        if state is not None:
            state.fill_(float("nan"))
    for kv in runner.storage.kv:
        if kv is not None:
            kv.k.fill_(float("nan"))
            kv.v.fill_(float("nan"))
    tokens = Z.tokens_of(cfg["vocab"], 91, 4)
    want = {0: P.forward(cfg, w, tokens)}
    check(replay(runner, {0: tokens}, [[(0, 1)], [(0, 12)], [(0, 1)], [(0, 77)]]), want, TOL["float32"], "NaN rows")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", [seed for seed in range(1, 18) if seed != 13])    # 13 amplifies rounding a hundredfold
def test_configurations_drawn_at_random(tmp_path, seed, dtype):
    """Other sizes, head counts, layer orders, windows and constants than any other test's: whole prompts, a portion
    beside single tokens of two requests, and portions down to one token."""
    folder = Z.make_folder(tmp_path / "any", Z.random_config(seed), seed)
    cfg, w = Z.load_folder(folder)
    requests = {0: Z.tokens_of(cfg["vocab"], 90, seed), 1: Z.tokens_of(cfg["vocab"], 21, seed + 1)}
    want = {r: P.forward(cfg, w, t) for r, t in requests.items()}
    runner = open_runner(folder, dtype, pages=64, page=16 if seed % 2 else 8)
    for plan in ([[(0, 90)], [(1, 21)]], [[(0, 70), (1, 3)]] + [[(0, 1), (1, 1)]] * 18 + [[(0, 2)]],
                 [[(0, size)] for size in portions(90, [2, 7, 1, 19, 3])] + [[(1, 1)]] * 21):
        check(replay(runner, requests, plan), want, TOL[dtype], f"configuration {seed}")
    assert runner.cache.check() == "" and runner.cache.live_requests() == 0


# --- edges: windows, kept first positions, far keys, shared rows, slow states ----------------------------------------
def edge_plans(n):
    return ([[(0, n)]], [[(0, n - 25)]] + [[(0, 1)]] * 25, [[(0, size)] for size in portions(n, [2, 7, 1, 19, 3])],
            [[(0, 1)]] * n)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("size, keep", [(5, 3), (19, 6), (8, 8), (6, 0)])
def test_the_edges_of_a_window_and_of_the_kept_positions(tmp_path, size, keep, dtype):
    """Attention peaked enough that the one key just inside the window (or the last one kept) carries weight and the one just
    outside would: in prompts, token by token and in portions that end on, before and behind the edge."""
    cfg = Z.single(Z.windowed(2, 1, 16, 16, size, keep_first=keep, rot_dims=8, scale=0.5), vocab=61)
    folder = Z.make_folder(tmp_path / "edge", cfg, 8, sharp=1.0)
    cfg, w = Z.load_folder(folder)
    tokens = Z.tokens_of(61, 70, 18)
    want = P.forward(cfg, w, tokens)
    for key, off in (("keep_first", -1), ("keep_first", 1), ("size", -1), ("size", 1)):
        if keep + off < 0 and key == "keep_first":
            continue
        other = copy.deepcopy(cfg)       # the test has teeth: a mask one off moves the logits clearly
        other["layers"][0]["mixer"]["mask"][key] += off
        moved = P.forward(other, w, tokens)
        assert sum(rel_err(moved[t], want[t]) > 1e-2 for t in range(size + keep, 70)) > 15, (key, off)
    runner = open_runner(folder, dtype, pages=16, page=8)
    for plan in edge_plans(70):
        check(replay(runner, {0: tokens}, plan), {0: want}, SHARP_TOL[dtype], f"window of {size}, {keep} kept")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind", ["latent", "shared", "window"])
def test_a_far_key_among_hundreds(tmp_path, kind, dtype):
    """Peaked attention over 400 positions: a late query puts most of its weight on single keys hundreds of positions and
    many pages back (through the other layer's rows in ``shared``, whose own layer is silenced; among the kept first
    positions in ``window``); portions end on page borders, one before and one behind them."""
    mine = Z.latent(2, 16, 8, 24, 24, 32, base=1e4, scaling=(4.0, 100, 8.0, 1.0), scale=0.5)
    layers = {"latent": [mine], "shared": [mine, dict(Z.latent(2, 16, 8, 24, 24, 32, base=1e4, scaling=(4.0, 100, 8.0, 1.0),
                                                               scale=0.5, kv_from=0))],
              "window": [Z.windowed(2, 1, 16, 24, 150, keep_first=40, rot_dims=8, scale=0.5)]}[kind]
    cfg = Z.config(61, 64, layers, [None] * len(layers))
    folder = Z.make_folder(tmp_path / "far", cfg, 8, sharp=3.0,
                           edit=lambda t: t["l0.mix.o"].zero_() if kind == "shared" else None)
    cfg, w = Z.load_folder(folder)
    tokens = Z.tokens_of(61, 400, 17)
    want = P.forward(cfg, w, tokens)
    # the test has teeth: other tokens far back move the late positions' logits clearly
    first, last = (0, 40) if kind == "window" else (0, 100)
    cut = P.forward(cfg, w, tokens[:first] + Z.tokens_of(61, last - first, 99) + tokens[last:])
    assert sum(rel_err(cut[t], want[t]) > 1e-2 for t in range(300, 400)) > 30
    runner = open_runner(folder, dtype, pages=60, page=16)
    for plan in ([[(0, 400)]], [[(0, 340)]] + [[(0, 1)]] * 60, [[(0, n)] for n in portions(400, [127, 2, 64, 33])],
                 [[(0, 16)], [(0, 15)], [(0, 17)], [(0, 208)]] + [[(0, 1)]] * 12 + [[(0, 132)]]):
        check(replay(runner, {0: tokens}, plan), {0: want}, SHARP_TOL[dtype], f"far key, {kind}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_prompts_on_the_prompt_kernels_of_full_head_widths(tmp_path, dtype):
    """1,300 tokens through latent rows of 128 numbers, a window of heads of 64 and the recurrence at its full tiles."""
    scaling = (4.0, 512, 32.0, 1.0)
    cfg = Z.config(61, 64, [Z.latent(4, 32, 32, 32, 48, 96, base=1e4, scaling=scaling), Z.mamba2(2, 64, 64, conv=4),
                            Z.windowed(4, 2, 64, 64, 300, keep_first=70, rot_dims=32),
                            Z.latent(2, 16, 32, 64, 24, 96, base=1e4, scaling=scaling, kv_from=0)], [None] * 4, streams=4)
    folder = Z.make_folder(tmp_path / "long", cfg, 12)
    cfg, w = Z.load_folder(folder)
    tokens = Z.tokens_of(61, 1300, 23)
    want = P.forward(cfg, w, tokens)
    runner = open_runner(folder, dtype, pages=90, page=16)
    for plan in ([[(0, 1300)]], [[(0, 700)], [(0, 590)]] + [[(0, 1)]] * 10):
        check(replay(runner, {0: tokens}, plan), {0: want}, TOL[dtype], "long prompt")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_state_that_forgets_slowly_remembers_the_first_tokens(tmp_path, dtype):
    """Decays near one: after 300 tokens, in pieces, the first tokens still weigh in the output, which a state that is
    lost or cleared between steps would not show."""
    def slow(t):
        t["l0.mix.A_log"].fill_(-6.0)
        t["l0.mix.D"].zero_()
    cfg = Z.single(Z.mamba2(2, 16, 16), vocab=61, width=32)
    folder = Z.make_folder(tmp_path / "slow", cfg, 9, edit=slow)
    cfg, w = Z.load_folder(folder)
    tokens = Z.tokens_of(61, 300, 19)
    want = P.forward(cfg, w, tokens)
    other = P.forward(cfg, w, Z.tokens_of(61, 150, 20) + tokens[150:])
    assert rel_err(other[-20:], want[-20:]) > 0.05            # the first half matters to the end
    runner = open_runner(folder, dtype)
    for plan in ([[(0, 300)]], [[(0, n)] for n in portions(300, [150, 1, 1, 2, 97])], [[(0, 260)]] + [[(0, 1)]] * 40,
                 [[(0, n)] for n in portions(300, [6, 7, 64])]):
        check(replay(runner, {0: tokens}, plan), {0: want}, TOL[dtype], "slow state")


def test_the_first_tokens_of_a_sequence(z1):
    """Positions 0 to 4 one by one and as a portion: nothing before position 0 exists (no state, no convolved inputs, no
    keys but the token's own)."""
    folder, cfg, w = z1
    runner = open_runner(folder, "float32")
    for n in (1, 2, 3, 5):
        tokens = Z.tokens_of(cfg["vocab"], n, 90 + n)
        want = {0: P.forward(cfg, w, tokens)}
        check(replay(runner, {0: tokens}, [[(0, n)]]), want, TOL["float32"], f"{n} tokens at once")
        check(replay(runner, {0: tokens}, [[(0, 1)]] * n), want, TOL["float32"], f"{n} tokens one by one")


# --- the engine: scheduler, sampling, captured steps ------------------------------------------------------------------
@pytest.mark.parametrize("dtype, graphs, pipelined", [("float32", False, False), ("float32", True, False),
                                                      ("float32", True, True), ("bfloat16", True, True)])
@pytest.mark.parametrize("which", ["z1", "z2"])
def test_greedy_generation_through_the_engine(request, which, dtype, graphs, pipelined):
    from vipera_rs_amd import Engine

    folder, cfg, w = request.getfixturevalue(which)
    prompts = [Z.tokens_of(cfg["vocab"], n, 60 + n) for n in (5, 37, 18, 2, 23)]
    new_tokens = 24
    engine = Engine(folder, dtype=dtype, block_size=8, num_blocks=40, max_num_seqs=3, chunk_size=16,
                    max_num_batched_tokens=32, max_model_len=128, use_graphs=graphs, pipelined=pipelined)
    got = engine.generate(prompts, max_new_tokens=new_tokens)
    clear = 0
    for prompt, generation in zip(prompts, got):
        assert len(generation.tokens) == new_tokens
        logits = P.forward(cfg, w, prompt + generation.tokens[:-1])
        clear += assert_tokens_follow_plain(logits, len(prompt), generation.tokens, 2.5e-5 if dtype == "float32" else 2e-2,
                                            f"prompt of {len(prompt)}")
    assert clear >= (100 if dtype == "float32" else 30), clear
    if graphs:
        assert engine.runner.graphs.replays > 0
    assert engine.runner.cache.check() == "" and engine.runner.cache.live_requests() == 0


def test_the_command_line_generates(z2):
    """``bin/vipera generate`` on a Zeladra folder: the model is found by its configuration and run through the engine."""
    folder, cfg, w = z2
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    prompt = Z.tokens_of(cfg["vocab"], 11, 3)
    done = subprocess.run([sys.executable, os.path.join(root, "bin", "vipera"), "generate", folder, "--prompt-ids",
                           " ".join(str(t) for t in prompt), "--max-tokens", "8", "--dtype", "float32", "--json"],
                          capture_output=True, text=True, timeout=600)
    assert done.returncode == 0, done.stderr[-2000:]
    report = json.loads(done.stdout)
    assert report["prompt_tokens"] == 11 and report["generated_tokens"] == 8
    logits = P.forward(cfg, w, prompt + report["tokens"][:-1])
    assert assert_tokens_follow_plain(logits, len(prompt), report["tokens"], 2.5e-5, "command line") >= 4


def test_the_trace_runner_replays_a_schedule(tmp_path, z1):
    """``bin/trace_run`` on a Zeladra folder: four slots, pages for the live requests only."""
    folder, cfg, w = z1
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    a, b = Z.tokens_of(cfg["vocab"], 50, 1), Z.tokens_of(cfg["vocab"], 20, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:30], "want": [0, 29]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[30:32], "want": []}, {"id": "b", "tokens": b[:19], "want": [18]}], "end": []},
             {"step": 2, "entries": [{"id": "b", "tokens": b[19:], "want": [0]}, {"id": "a", "tokens": a[32:], "want": [17]}], "end": ["a", "b"]}]
    out = tmp_path / "out"
    done = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", folder, "--dtype", "float32",
                           "--out", str(out), "--max-tokens", "128"], input="\n".join(json.dumps(s) for s in steps) + "\n",
                          capture_output=True, text=True, timeout=600)
    assert done.returncode == 0, done.stderr[-2000:]
    assert [line for line in done.stdout.splitlines() if line.startswith("done")] == ["done 0", "done 1", "done 2"]
    wa, wb = P.forward(cfg, w, a), P.forward(cfg, w, b)
    rows = {0: [wa[0], wa[29]], 1: [wb[18]], 2: [wb[19], wa[49]]}
    for step, want in rows.items():
        got = np.fromfile(out / f"{step}.f32", dtype="<f4").reshape(len(want), cfg["vocab"])
        assert rel_err(got, np.stack(want)) < TOL["float32"]
