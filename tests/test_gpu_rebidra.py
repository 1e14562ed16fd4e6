"""Rebidra on the GPU against the plain implementation (``plain/rebidra_plain.py``): kernels and mechanisms alone, then
whole models through the step function (whole prompts, single tokens, portions down to two tokens, mixed batches, slots
and pages that are used again, far keys, the edges of windows and pages, the convolutions' reach across portions, passes
through the loop), and greedy generation through the engine.

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

import rebidra_helpers as Z
from helpers import assert_tokens_follow_plain, rel_err
from plain import rebidra_plain as P

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
    hold.  In bfloat16 a router's close call may fall the other way than in float64 and move one position's logits (and,
    through the keys of later layers and passes, a few after it) by more than rounding: there one position in twelve may be
    over, which a fault of a page, a slot or a state (whole runs of positions) still exceeds."""
    strict = tol < 1e-3
    over, total = [], 0
    for r in got:
        assert want[r].shape == got[r].shape
        for t in range(got[r].shape[0]):
            err = rel_err(got[r][t], want[r][t])
            total += 1
            if not err < tol:
                assert not strict, f"{label}: request {r}, position {t} of {got[r].shape[0]}: relative error {err:.3g}"
                over.append((r, t, round(err, 3)))
    assert len(over) <= total // 12, f"{label}: {len(over)} of {total} positions are over {tol}: {over[:8]}"


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
HEADS = [  # heads, kv_heads, dim, vdim, taps (0: no convolution), own values, rotated, normed
    (4, 2, 16, 16, 3, False, 16, True), (3, 1, 10, 10, 6, False, 4, True), (2, 2, 24, 24, 1, False, 0, True),
    (5, 1, 96, 96, 4, False, 64, True), (2, 1, 136, 136, 2, False, 136, True), (2, 1, 256, 256, 5, False, 130, False),
    (3, 3, 12, 20, 3, True, 12, True), (4, 2, 64, 40, 0, True, 32, True), (2, 1, 128, 128, 0, False, 128, False),
    (1, 1, 200, 200, 7, True, 6, True),
]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads, kv_heads, dim, vdim, taps, own, rot, normed", HEADS)
def test_heads_convolved_normed_rotated_and_paged(heads, kv_heads, dim, vdim, taps, own, rot, normed, dtype):
    """Entries of unequal lengths, some going on from inputs in the state, over several steps: portions around the number of
    taps, runs of eight tokens in steps of more than 512 (aligned to a page's pieces and not), steps of single tokens."""
    from vipera_rs_amd.ops import kernels

    rng = np.random.default_rng(dim * 10 + taps)
    width, block, eps, amplitude = (max(dim, vdim) + 15) // 16 * 16, 8, 1e-3, 1.3
    channels, n = (heads + kv_heads) * dim, max(taps, 1)
    values = kv_heads * vdim if own else 0
    conv = rng.standard_normal((channels, n)) / np.sqrt(n)
    qw, kw = (1 + 0.2 * rng.standard_normal(dim) for _ in range(2))
    freq = rng.uniform(0.01, 1.0, rot // 2)
    E, longest = 5, 1400
    slots = rng.permutation(E)
    state = torch.full((E + 1, (n - 1) * channels + 3), float("nan"), device="cuda")
    pages = longest // block
    table = rng.permutation(E * pages).reshape(E, pages)
    k_cache = torch.zeros((E * pages + 1, kv_heads, block, width), dtype=dtype, device="cuda")
    v_cache = torch.zeros((E * pages + 1, kv_heads, width, block), dtype=dtype, device="cuda")
    i32 = lambda a: dev(np.ascontiguousarray(a), torch.int32)
    seen = [np.zeros((0, channels + values)) for _ in range(E)]
    tol = 1e-5 if dtype == torch.float32 else 1e-2
    for sizes in ([1, 2, n, n + 1, 9], [1] * E, [600, 3, 1, 64, 24], [1] * E, [8, 16, 9, 2, 513], [1, 1, 2, 1, 1]):
        T = sum(sizes)
        starts = np.concatenate([[0], np.cumsum(sizes)])
        firsts = np.array([len(s) for s in seen])
        proj = rng.standard_normal((T, channels + values + 5))
        entry = np.repeat(np.arange(E), sizes)
        positions = np.arange(T) - starts[entry] + firsts[entry]
        angles = None
        if rot and T > 100:
            angles = kernels.rope_angles(i32(positions), dev(freq), T, amplitude)
        q = torch.full((T, heads * width), float("nan"), dtype=dtype, device="cuda")
        kernels.head_conv_prepare(dev(proj), dev(conv) if taps else None, state if n > 1 else None, i32(entry), i32(starts),
                                  i32(firsts), i32(slots), E, dev(qw), dev(kw), normed, eps, i32(positions),
                                  dev(freq) if rot else None, rot, heads, kv_heads, dim, vdim, own, width, q, k_cache, v_cache,
                                  i32(table), angles, amplitude)
        q_got = q.float().cpu().numpy().reshape(T, heads, width)
        k_all, v_all = k_cache.float().cpu().numpy(), v_cache.float().cpu().numpy()
        for e in range(E):
            seen[e] = np.concatenate([seen[e], proj[starts[e]:starts[e + 1], :channels + values]])
            y = seen[e][:, :channels]
            if taps:
                y = P.causal_conv(y, conv)
            y = y.reshape(-1, heads + kv_heads, dim)
            v_want = seen[e][:, channels:].reshape(-1, kv_heads, vdim) if own else y[:, heads:]
            if normed:
                y = P.over_rms(y, eps) * np.where(np.arange(heads + kv_heads)[:, None] < heads, qw, kw)
            if rot:
                turn = np.float64(np.float32(np.arange(len(y)))[:, None] * np.float32(freq))[:, None]
                c, s = amplitude * np.cos(turn), amplitude * np.sin(turn)
                lo, hi = y[..., :rot // 2], y[..., rot // 2:rot]
                y = np.concatenate([lo * c - hi * s, hi * c + lo * s, y[..., rot:]], axis=-1)
            new = slice(firsts[e], len(y))
            mine = q_got[starts[e]:starts[e + 1]]
            assert rel_err(mine[..., :dim], y[new, :heads]) < tol and np.all(mine[..., dim:] == 0), (sizes, e)
            at = np.arange(len(y))
            page, slot = table[e, at // block], at % block
            k_got, v_got = k_all[page, :, slot], v_all[page, :, :, slot]                 # every page, the older ones too
            assert rel_err(k_got[..., :dim], y[:, heads:]) < tol and np.all(k_got[..., dim:] == 0), (sizes, e)
            assert rel_err(v_got[..., :vdim], v_want) < tol and np.all(v_got[..., vdim:] == 0), (sizes, e)
            if n > 1:
                kept = np.concatenate([np.zeros((n - 1, channels)), seen[e][:, :channels]])[-(n - 1):]
                assert np.array_equal(state[slots[e], :(n - 1) * channels].cpu().numpy(), np.float32(kept.reshape(-1))), (sizes, e)
    assert torch.isnan(state[E]).all() and torch.isnan(state[:, (n - 1) * channels:]).all()


def route(kernels, logits, top, tile_rows):
    tokens, experts = logits.shape
    pairs = tokens * top
    ids, order = (torch.empty(pairs, dtype=torch.int32, device="cuda") for _ in range(2))
    weights = torch.empty(pairs, device="cuda")
    offsets = torch.empty(experts + 1, dtype=torch.int32, device="cuda")
    tiles = torch.full((2 * kernels.moe_max_tiles(pairs, experts, tile_rows),), -1, dtype=torch.int32, device="cuda")
    count = torch.empty(1, dtype=torch.int32, device="cuda")
    kernels.moe_route(logits, top, ids, weights, offsets, order, tiles, count, tile_rows)
    return ids, weights, offsets, order, tiles, count


@pytest.mark.parametrize("tile_rows", [16, 64, 128])
@pytest.mark.parametrize("tokens, experts, top", [(1, 1, 1), (3, 5, 2), (40, 130, 7), (300, 3, 3), (200, 64, 4), (7, 65, 64)])
def test_pairs_are_grouped_by_expert_and_cut_into_tiles(tokens, experts, top, tile_rows):
    from vipera_rs_amd.ops import kernels

    z = np.random.default_rng(tokens + experts).standard_normal((tokens, experts))
    ids, weights, offsets, order, tiles, count = route(kernels, dev(z), top, tile_rows)
    want_ids, want_weights = P.choose(z.astype(np.float32).astype(np.float64), top)
    assert np.array_equal(ids.cpu().numpy().reshape(tokens, top), want_ids)
    assert np.allclose(weights.cpu().numpy().reshape(tokens, top), want_weights, atol=1e-6)
    counts = np.bincount(want_ids.reshape(-1), minlength=experts)
    edges = np.concatenate([[0], np.cumsum(counts)])
    assert np.array_equal(offsets.cpu().numpy(), edges)
    places = order.cpu().numpy()
    for e in range(experts):
        assert sorted(places[edges[e]:edges[e + 1]]) == list(np.nonzero(want_ids.reshape(-1) == e)[0])
    listed = [(e, edges[e] + i) for e in range(experts) for i in range(0, counts[e], tile_rows)]
    assert int(count.item()) == len(listed)
    assert [tuple(t) for t in tiles.cpu().numpy().reshape(-1, 2)[:len(listed)]] == listed


@pytest.mark.parametrize("dtype, tile_rows", [(torch.float32, 64), (torch.bfloat16, 64), (torch.bfloat16, 16), (torch.bfloat16, 128)])
@pytest.mark.parametrize("plain", ["relu2", "silu", "gelu_tanh", None])
@pytest.mark.parametrize("tokens, width, ff, experts, top", [(5, 48, 24, 6, 2), (70, 136, 72, 3, 3), (1, 520, 264, 9, 4), (33, 64, 8, 1, 1)])
def test_experts_with_and_without_a_gate(tokens, width, ff, experts, top, plain, dtype, tile_rows):
    """Every form of the products: added to the residual and written, weighed in front and behind, beside a gated sum, with
    the new rows in 16 bits."""
    from vipera_rs_amd.ops import kernels

    if tile_rows == 64 and dtype == torch.bfloat16:
        width, ff = width + 1, ff + 2            # widths that leave the matrix cores
    rng = np.random.default_rng(tokens + ff)
    h, z = dev(rng.standard_normal((tokens, width)), dtype), dev(rng.standard_normal((tokens, experts)))
    gate, up = (dev(rng.standard_normal((experts, ff, width)) / np.sqrt(width), dtype) for _ in range(2))
    down = dev(rng.standard_normal((experts, width, ff)) / np.sqrt(ff), dtype)
    base, extra, side = rng.standard_normal((tokens, width)), rng.standard_normal((tokens, width)), rng.standard_normal((tokens, 3))
    f64 = lambda t: t.double().cpu().numpy()
    acts = {"relu2": lambda u: np.maximum(u, 0) ** 2, "silu": lambda u: u * P.sigmoid(u), "gelu_tanh": P.gelu_tanh}
    ids, weights = P.choose(f64(z), top)
    tol = 2e-5 if dtype == torch.float32 else 1e-2
    for weigh_input in (False, True):
        sums = np.zeros((tokens, width))
        for t in range(tokens):
            for e, share in zip(ids[t], weights[t]):
                x = f64(h)[t] * (share if weigh_input else 1.0)
                u = f64(up)[e] @ x
                if plain is None:
                    g = f64(gate)[e] @ x
                    u = g * P.sigmoid(g) * u
                else:
                    u = acts[plain](u)
                sums[t] += (1.0 if weigh_input else share) * (f64(down)[e] @ u)
        _, w, offsets, order, tiles, count = route(kernels, z, top, tile_rows)
        act = torch.full((tokens * top, ff), float("nan"), dtype=dtype, device="cuda")
        pair_out = torch.full((tokens * top, width), float("nan"), device="cuda")

        def run(residual, accumulate, **kw):
            kernels.moe_experts(h, None if plain else gate, up, down, offsets, order, tiles, count, w, top, float("inf"), 1.0, act,
                                pair_out, residual, accumulate, weigh_input, tile_rows, plain=plain, **kw)
            return residual.cpu().numpy()
        assert rel_err(run(dev(base), True), base + sums) < tol
        assert rel_err(run(dev(np.full_like(base, np.nan)), False), sums) < tol
        assert rel_err(run(dev(base), True, extra=dev(extra)), base + sums + extra) < tol
        stream = torch.empty((tokens, width), dtype=torch.bfloat16, device="cuda")
        got = run(dev(base), True, extra=dev(extra), extra_gate=dev(side)[:, 1:], stream=stream)
        want = base + sums + P.sigmoid(side[:, 1:2]) * extra
        assert rel_err(got, want) < tol and torch.equal(stream.cpu(), torch.from_numpy(got).to(torch.bfloat16))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width", [40, 50, 1000, 4096, 5000])
def test_a_norm_behind_and_a_layer_norm_in_front_in_one_launch(width, dtype):
    from vipera_rs_amd.ops import kernels

    rng = np.random.default_rng(width)
    y, x = rng.standard_normal((7, width)), rng.standard_normal((7, width)) + 3.0
    w, w2, b2 = 1 + 0.2 * rng.standard_normal(width), 1 + 0.2 * rng.standard_normal(width), rng.standard_normal(width)
    tol = 2e-5 if dtype == torch.float32 else 1e-2
    new = x + P.over_rms(y, 1e-3) * w
    for kind, bias in (("layer", None), ("layer", b2), ("rms", None)):
        stream, out = dev(x), torch.empty((7, width), dtype=dtype, device="cuda")
        kernels.rmsnorm_add(dev(y), dev(w), 1e-3, stream, out, dev(w2), 1e-2, next_kind=kind,
                            next_bias=dev(bias) if bias is not None else None)
        want = P.layer_norm(new, w2, 1e-2) + (bias if bias is not None else 0.0) if kind == "layer" else P.over_rms(new, 1e-2) * w2
        assert rel_err(stream.cpu().numpy(), new) < 1e-6 and rel_err(out.float().cpu().numpy(), want) < tol


@pytest.mark.parametrize("tokens, width, dim", [(1, 48, 8), (5, 72, 24), (17, 1032, 64), (40, 2056, 16), (3, 4104, 520), (2, 8192, 40),
                                                (256, 64, 72)])
def test_the_side_tables_step_of_few_tokens(tokens, width, dim):
    from vipera_rs_amd.ops import kernels

    rng = np.random.default_rng(width + dim)
    gate = dev(rng.standard_normal((dim, width)) / np.sqrt(width), torch.bfloat16)
    proj = dev(rng.standard_normal((width, dim)) / np.sqrt(dim), torch.bfloat16)
    x, e = np.float64(np.float32(rng.standard_normal((tokens, width)) + 0.3)), rng.standard_normal((tokens, dim + 4))
    norm, w2, b2 = 1 + 0.2 * rng.standard_normal(width), 1 + 0.2 * rng.standard_normal(width), rng.standard_normal(width)
    assert kernels.token_side_supported(dev(x), gate, proj)
    f64 = lambda t: t.double().cpu().numpy()
    z = f64(dev(x, torch.bfloat16)) @ f64(gate).T
    g = f64(dev(P.gelu_tanh(z) * e[:, 3:3 + dim], torch.bfloat16))
    new = x + P.over_rms(g @ f64(proj).T, 1e-3) * norm
    for kind, bias in ((None, None), ("layer", None), ("layer", b2), ("rms", None)):
        stream = dev(x)
        out = torch.empty((tokens, width), dtype=torch.bfloat16, device="cuda") if kind else None
        kernels.token_side(stream, dev(e)[:, 3:3 + dim], gate, proj, dev(norm), 1e-3, out, dev(w2) if kind else None, 1e-2,
                           kind or "rms", dev(bias) if bias is not None else None)
        assert rel_err(stream.cpu().numpy(), new) < 4e-3       # a number of g may be rounded the other way
        if kind:
            want = P.layer_norm(new, w2, 1e-2) + (bias if bias is not None else 0.0) if kind == "layer" else P.over_rms(new, 1e-2) * w2
            assert rel_err(out.float().cpu().numpy(), want) < 1e-2


# --- each mechanism alone, as a model of one layer -------------------------------------------------------------------
ONE_LAYER = {
    # attention: taps of one to six, odd widths, one head, as many key heads as heads, part of a head rotated, none, blended
    "window": Z.single(Z.windowed(4, 2, 16, 7, conv=3, base=300.0, scaling=Z.YARN)),
    "window_one_tap_odd": Z.single(Z.windowed(2, 2, 10, 5, conv=1, rot_dims=0, scale=0.4), width=50),
    "window_six_taps": Z.single(Z.windowed(3, 1, 24, 12, conv=6, rot_dims=10), width=48),
    "window_one_position": Z.single(Z.windowed(1, 1, 8, 1, conv=4, rot_dims=2), width=40),
    "no_window": Z.single(Z.windowed(6, 2, 32, 0, conv=2, scaling=(2.0, 16, 4.0, 4.0))),
    "window_wide": Z.single(Z.windowed(5, 5, 72, 100, conv=4, rot_dims=32), width=136),
    "window_wider_heads": Z.single(Z.windowed(2, 1, 208, 70, conv=5, rot_dims=130, scale=0.05), width=72),
    "window_many_heads_a_key": Z.single(Z.windowed(20, 1, 16, 40, conv=2), width=64),
    # the feed-forward: all experts, one expert, no shared one, odd widths, many experts
    "experts": Z.single(Z.windowed(1, 1, 8, 6), Z.moe(24, 5, 2, 40), width=48),
    "experts_all_chosen_no_shared": Z.single(Z.windowed(1, 1, 8, 6), Z.moe(33, 3, 3), width=50),
    "one_expert_odd_shared": Z.single(Z.windowed(1, 1, 8, 6), Z.moe(16, 1, 1, 35), width=56),
    "experts_many": Z.single(Z.windowed(1, 1, 8, 6), Z.moe(8, 70, 9, 8), width=40),
    "experts_wide": Z.single(Z.windowed(1, 1, 8, 6), Z.moe(136, 4, 2, 264), width=264),
    # the side table: one column, odd, wide; behind a feed-forward and without one
    "side": Z.single(Z.windowed(1, 1, 8, 6), Z.moe(24, 3, 2, 8), width=48, side=8),
    "side_one_column": Z.single(Z.windowed(1, 1, 8, 6), width=40, side=1),
    "side_wide": Z.single(Z.windowed(1, 1, 8, 6), width=72, side=136, eps=1e-2),
    # the loop: one layer in one pass, in three; constants
    "loop_once": Z.single(Z.windowed(2, 1, 8, 6), width=48, loop=(0, 1, 1), embedding_scale=3.0, logit_scale=0.25),
    "loop_three_times": Z.single(Z.windowed(2, 1, 8, 6, conv=3), Z.moe(24, 3, 1, 16), width=50, side=3, loop=(0, 1, 3), eps=1e-3),
}
LONG = {"window_wide", "no_window", "experts_wide", "window_wider_heads"}      # a prompt of 330 tokens: several tiles


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


def test_values_of_their_own_and_keys_without_a_convolution(tmp_path):
    """The options one by one, as another design may put them together: a convolution beside a value projection (of another
    width), and values that are the keys without a convolution."""
    from vipera_rs_amd.config.base import PartSpec
    from vipera_rs_amd.parts import part_class
    from vipera_rs_amd.runtime import Runtime
    from types import SimpleNamespace

    for dtype in ("float32", "bfloat16"):
        runtime, rng = Runtime("cuda:0", dtype), np.random.default_rng(5)
        T, hidden, heads, kv, dim, vdim, block = 37, 40, 4, 2, 16, 24, 8
        x = np.float64(dev(rng.standard_normal((T, hidden)), runtime.dtype).float().cpu().numpy())
        for values, taps in ((None, 3), ("keys", 0)):
            vd = dim if values else vdim
            params = {"hidden": hidden, "heads": heads, "kv_heads": kv, "head_dim": dim, "value_dim": vd, "name": "m", "values": values,
                      "conv": taps, "window": 9, "qk_norm": "head", "eps": 1e-5,
                      "tensors": {n: n for n in ("q", "k", "v", "o", "q_norm", "k_norm", "q_conv", "k_conv")}}
            spec = PartSpec("attention", params)
            kind = part_class("mixer", "attention")
            kind.check_supported(spec, runtime.dtype)
            part = kind(spec, "", runtime)
            tensors, w = {}, {}
            for t in kind.declare(spec, ""):
                value = rng.standard_normal(t.shape) / np.sqrt(t.shape[-1] if len(t.shape) > 1 else 1.0)
                tensors[t.name] = dev(value, runtime.dtype if t.role == "matrix" else torch.float32)
                w[t.name.split(".")[1]] = tensors[t.name].double().cpu().numpy()
            part.load(tensors)
            kv_spec, state_spec = kind.declare_cache(spec)
            pages = (T + block - 1) // block
            cache = SimpleNamespace(k=runtime.zeros((pages + 1, kv, block, kv_spec.head_dim)), group=0,
                                    v=runtime.zeros((pages + 1, kv, kv_spec.value_width, block)))
            state = torch.zeros((2,) + state_spec.shape, device="cuda") if state_spec else None
            i32 = lambda a: dev(np.asarray(a), torch.int32)
            batch = SimpleNamespace(num_tokens=T, num_entries=1, positions=i32(np.arange(T)), entry_of_token=i32(np.zeros(T)),
                                    entry_start=i32([0, T]), entry_first_pos=i32([0]), slots=i32([1]), shared={}, launch_plans=[],
                                    block_tables={0: i32([list(range(pages))])}, num_prefill_tiles=1, prefill_tile_tokens=128,
                                    prefill_tiles=i32([[0, 0]]), num_decode_entries=0, decode_entries=i32([]), max_tile_reach=T,
                                    sum_tile_reach=T, all_single=False)
            out = torch.zeros((T, hidden), device="cuda")
            position = part_class("position", "none")(PartSpec("none", {}), "", runtime)
            part.forward(dev(x, runtime.dtype), batch, cache, state, position, out)
            q, k = x @ w["q"].T, x @ w["k"].T
            if taps:
                q, k = P.causal_conv(q, w["q_conv"]), P.causal_conv(k, w["k_conv"])
            q, k = q.reshape(T, heads, dim), k.reshape(T, kv, dim)
            v = k if values else (x @ w["v"].T).reshape(T, kv, vd)
            o = P.sink_attention(P.over_rms(q, 1e-5) * w["q_norm"], P.over_rms(k, 1e-5) * w["k_norm"], v, dim ** -0.5,
                                 P.visible(9, T), np.full(heads, -1e9))
            assert rel_err(out.cpu().numpy(), o.reshape(T, heads * vd) @ w["o"].T) < (2e-5 if dtype == "float32" else 3e-2), (dtype, values)


def test_pages_of_two_positions_take_the_general_kernel(tmp_path):
    folder = Z.make_folder(tmp_path / "r1", Z.R1, 21)
    cfg, w = Z.load_folder(folder)
    tokens = Z.tokens_of(cfg["vocab"], 50, 3)
    runner = open_runner(folder, "float32", pages=64, page=2)
    for plan in ([[(0, 50)]], [[(0, 31)]] + [[(0, 1)]] * 19):
        check(replay(runner, {0: tokens}, plan), {0: P.forward(cfg, w, tokens)}, TOL["float32"], "pages of two")


def test_the_residual_after_every_layer(tmp_path):
    """32-bit, layer by layer in the order of the run: a fault shows in the layer or the pass that has it."""
    for name, model in (("r1", Z.R1), ("r2", Z.R2)):
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
                seen.append(x.clone())
            layer.forward = wrapped
        got = replay(runner, {0: tokens}, [[(0, 80)]])
        assert len(seen) == len(residuals) == len(P.run_order(model))
        for index, (mine, ref) in enumerate(zip(seen, residuals)):
            assert rel_err(mine.cpu().numpy(), ref) < 2e-5, f"{name}: after run {index} (layer {P.run_order(model)[index][0]})"
        check(got, {0: want}, TOL["float32"], name)


# --- whole models through the step function ------------------------------------------------------------------------
@pytest.fixture(scope="module")
def r1(tmp_path_factory):
    folder = Z.make_folder(tmp_path_factory.mktemp("r1"), Z.R1, 31)
    return (folder,) + Z.load_folder(folder)


@pytest.fixture(scope="module")
def r2(tmp_path_factory):
    folder = Z.make_folder(tmp_path_factory.mktemp("r2"), Z.R2, 32)
    return (folder,) + Z.load_folder(folder)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which", ["r1", "r2"])
def test_token_by_token_equals_the_whole_prompt(request, which, dtype):
    folder, cfg, w = request.getfixturevalue(which)
    tokens = Z.tokens_of(cfg["vocab"], 150, 7)
    want = {0: P.forward(cfg, w, tokens)}
    runner = open_runner(folder, dtype, page=4 if which == "r2" and dtype == "float32" else 8, pages=128)
    whole = replay(runner, {0: tokens}, [[(0, 150)]])
    check(whole, want, TOL[dtype], "whole")
    single = replay(runner, {0: tokens}, [[(0, 1)]] * 150)      # long decoding from the very first token
    check(single, want, TOL[dtype], "token by token")
    if dtype == "float32":   # the two ways differ by rounding only
        assert rel_err(single[0], whole[0].astype(np.float64)) < 2e-5


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("sizes", [[2], [3, 2, 17, 2, 5], [13, 1, 8], [16, 2], [64, 7], [6, 7], [65, 63, 66]])
@pytest.mark.parametrize("which", ["r1", "r2"])
def test_portions_of_a_prompt(request, which, sizes, dtype):
    """Portions cut inside pages (8), at their borders, inside windows (7, 11 and 19) and inside the convolutions' reach."""
    folder, cfg, w = request.getfixturevalue(which)
    n = 200 if max(sizes) > 20 else 83
    tokens = Z.tokens_of(cfg["vocab"], n, 9)
    want = {0: P.forward(cfg, w, tokens)}
    runner = open_runner(folder, dtype)
    plan = [[(0, size)] for size in portions(n, sizes)]
    check(replay(runner, {0: tokens}, plan), want, TOL[dtype], f"portions {sizes}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which", ["r1", "r2"])
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
def test_a_slot_and_pages_that_are_used_again_start_clean(r1, dtype):
    """One slot and few pages: every request runs in the state row and the pages the one before it left full."""
    folder, cfg, w = r1
    runner = open_runner(folder, dtype, pages=9, page=8, slots=1)
    for r, (n, cut) in enumerate([(60, [60]), (41, [5, 2, 30, 1, 1, 1, 1]), (17, [1] * 17), (64, [33, 31]), (70, [2, 68])]):
        tokens = Z.tokens_of(cfg["vocab"], n, 70 + r)
        got = replay(runner, {r: tokens}, [[(r, size)] for size in cut])
        check(got, {r: P.forward(cfg, w, tokens)}, TOL[dtype], f"request {r} in the used slot")
        assert runner.cache.slot(r) == -1 and runner.cache.free_slots() == 1


def test_state_rows_and_pages_full_of_nan_do_not_reach_a_new_request(r2):
    """A slot's row and a pool's pages may hold anything when a request takes them."""
    folder, cfg, w = r2
    runner = open_runner(folder, "float32", slots=2)
    for state in runner.storage.state:
        if state is not None:
            state.fill_(float("nan"))
    for kv in runner.storage.kv:
        kv.k.fill_(float("nan"))
        kv.v.fill_(float("nan"))
    tokens = Z.tokens_of(cfg["vocab"], 91, 4)
    want = {0: P.forward(cfg, w, tokens)}
    check(replay(runner, {0: tokens}, [[(0, 1)], [(0, 12)], [(0, 1)], [(0, 77)]]), want, TOL["float32"], "NaN rows")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", range(1, 21))
def test_configurations_drawn_at_random(tmp_path, seed, dtype):
    """Other sizes, head counts, windows, loops and constants than any other test's: whole prompts, a portion beside single
    tokens of two requests, and portions down to one token."""
    folder = Z.make_folder(tmp_path / "any", Z.random_config(seed), seed)
    cfg, w = Z.load_folder(folder)
    requests = {0: Z.tokens_of(cfg["vocab"], 90, seed), 1: Z.tokens_of(cfg["vocab"], 21, seed + 1)}
    want = {r: P.forward(cfg, w, t) for r, t in requests.items()}
    runner = open_runner(folder, dtype, pages=64, page=16 if seed % 2 else 8)
    for plan in ([[(0, 90)], [(1, 21)]], [[(0, 70), (1, 3)]] + [[(0, 1), (1, 1)]] * 18 + [[(0, 2)]],
                 [[(0, size)] for size in portions(90, [2, 7, 1, 19, 3])] + [[(1, 1)]] * 21):
        check(replay(runner, requests, plan), want, TOL[dtype], f"configuration {seed}")
    assert runner.cache.check() == "" and runner.cache.live_requests() == 0


# --- edges: windows, far keys, the sink, the convolution's reach, the loop's passes -----------------------------------
def edge_plans(n):
    return ([[(0, n)]], [[(0, n - 25)]] + [[(0, 1)]] * 25, [[(0, size)] for size in portions(n, [2, 7, 1, 19, 3])],
            [[(0, 1)]] * n)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("size", [1, 5, 8, 19])
def test_the_edges_of_a_window(tmp_path, size, dtype):
    """Attention peaked enough that the one key just inside the window carries weight and the one just outside would: in
    prompts, token by token and in portions that end on, before and behind the edge."""
    cfg = Z.single(Z.windowed(2, 1, 16, size, conv=2, rot_dims=8, scale=0.5), vocab=61)
    folder = Z.make_folder(tmp_path / "edge", cfg, 8, sharp=1.5)
    cfg, w = Z.load_folder(folder)
    tokens = Z.tokens_of(61, 70, 18)
    want = P.forward(cfg, w, tokens)
    for off in (-1, 1):
        if size + off < 1:
            continue
        other = copy.deepcopy(cfg)       # the test has teeth: a window one off moves the logits clearly
        other["layers"][0]["mixer"]["mask"]["size"] += off
        moved = P.forward(other, w, tokens)
        assert sum(rel_err(moved[t], want[t]) > 1e-2 for t in range(size, 70)) > 10, off
    runner = open_runner(folder, dtype, pages=16, page=8)
    for plan in edge_plans(70):
        check(replay(runner, {0: tokens}, plan), {0: want}, SHARP_TOL[dtype], f"window of {size}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind", ["window", "no_window", "passes"])
def test_a_far_key_among_hundreds(tmp_path, kind, dtype):
    """Peaked attention over 400 positions: a late query puts most of its weight on single keys hundreds of positions and
    many pages back; in ``passes`` within each of two passes' windows of 150; portions end on page borders, one before and
    one behind them."""
    layer = Z.windowed(2, 1, 16, {"window": 350, "no_window": 0, "passes": 150}[kind], conv=3, rot_dims=8, base=1e4, scale=0.5,
                       scaling=(4.0, 100, 8.0, 1.0))
    cfg = Z.config(61, 64, [layer], [None], loop=(0, 1, 2) if kind == "passes" else None, side=0)
    folder = Z.make_folder(tmp_path / "far", cfg, 8, sharp=3.0)
    cfg, w = Z.load_folder(folder)
    tokens = Z.tokens_of(61, 400, 17)
    want = P.forward(cfg, w, tokens)
    # the test has teeth: other tokens far back move the late positions' logits clearly
    cut = P.forward(cfg, w, tokens[:100] + Z.tokens_of(61, 100, 99) + tokens[200:])
    assert sum(rel_err(cut[t], want[t]) > 1e-2 for t in range(310, 400)) > 30
    runner = open_runner(folder, dtype, pages=60, page=16)
    for plan in ([[(0, 400)]], [[(0, 340)]] + [[(0, 1)]] * 60, [[(0, n)] for n in portions(400, [127, 2, 64, 33])],
                 [[(0, 16)], [(0, 15)], [(0, 17)], [(0, 208)]] + [[(0, 1)]] * 12 + [[(0, 132)]]):
        check(replay(runner, {0: tokens}, plan), {0: want}, SHARP_TOL[dtype], f"far key, {kind}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_the_sink_and_the_gate_weigh_in_prompts_and_in_decoding(tmp_path, dtype):
    """Sinks of either side of the scores and gates of either side of a half; without either the logits move clearly."""
    cfg = Z.single(Z.windowed(4, 2, 16, 30, conv=2, rot_dims=8), vocab=61)
    folder = Z.make_folder(tmp_path / "sink", cfg, 8, edit=lambda t: t["l0.mix.sink"].copy_(torch.tensor([-3.0, 4.0, 2.0, 6.0])))
    cfg, w = Z.load_folder(folder)
    tokens = Z.tokens_of(61, 75, 18)
    want = P.forward(cfg, w, tokens)
    for other in (dict(w, **{"l0.mix.sink": np.full(4, -1e9)}), dict(w, **{"l0.mix.g": 0 * w["l0.mix.g"]}),
                  dict(w, **{"l0.mix.sink": w["l0.mix.sink"] + np.log(2.0)})):
        moved = P.forward(cfg, other, tokens)
        assert sum(rel_err(moved[t], want[t]) > 1e-2 for t in range(75)) > 60
    runner = open_runner(folder, dtype, pages=16, page=8)
    for plan in edge_plans(75):
        check(replay(runner, {0: tokens}, plan), {0: want}, TOL[dtype], "sink")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_the_convolution_reaches_across_portions(tmp_path, dtype):
    """A tap four tokens back outweighs the others, in portions shorter and longer than its reach; an input that is lost
    or read one off between two steps moves the logits clearly."""
    def far_tap(t):
        for name in ("q", "k"):
            t[f"l0.mix.{name}.conv"][:, 0] *= 4.0
    cfg = Z.single(Z.windowed(2, 1, 16, 12, conv=5, rot_dims=8), vocab=61)
    folder = Z.make_folder(tmp_path / "taps", cfg, 8, edit=far_tap)
    cfg, w = Z.load_folder(folder)
    tokens = Z.tokens_of(61, 64, 18)
    want = P.forward(cfg, w, tokens)
    off = dict(w)
    for name in ("l0.mix.q.conv", "l0.mix.k.conv"):
        off[name] = np.roll(w[name], 1, axis=1)
    moved = P.forward(cfg, off, tokens)
    assert sum(rel_err(moved[t], want[t]) > 5e-2 for t in range(5, 64)) > 50
    runner = open_runner(folder, dtype, pages=16, page=8)
    for sizes in ([64], [1], [2], [3, 1], [4, 5, 1, 1], [6, 2, 1, 20]):
        check(replay(runner, {0: tokens}, [[(0, n)] for n in portions(64, sizes)]), {0: want}, TOL[dtype], f"portions {sizes}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("dim", [64, 96, 128])
def test_a_long_prompt_on_the_prompt_kernels_of_full_head_widths(tmp_path, dim, dtype):
    """1,300 tokens in runs, windows of hundreds, twice through the layer, then single tokens."""
    cfg = Z.config(61, 64, [Z.windowed(4, 2, dim, 300, conv=4, scaling=(4.0, 512, 32.0, 1.0))], [Z.moe(64, 4, 2, 64)], loop=(0, 1, 2))
    folder = Z.make_folder(tmp_path / "long", cfg, 12)
    cfg, w = Z.load_folder(folder)
    tokens = Z.tokens_of(61, 1300, 23)
    want = P.forward(cfg, w, tokens)
    runner = open_runner(folder, dtype, pages=90, page=16)
    for plan in ([[(0, 1300)]], [[(0, 700)], [(0, 590)]] + [[(0, 1)]] * 10, [[(0, 3)], [(0, 1297)]]):
        check(replay(runner, {0: tokens}, plan), {0: want}, TOL[dtype], "long prompt")


def test_the_first_tokens_of_a_sequence(r1):
    """Positions 0 to 4 one by one and as a portion: nothing before position 0 exists (no convolved inputs, no keys but the
    token's own and the sink)."""
    folder, cfg, w = r1
    runner = open_runner(folder, "float32")
    for n in (1, 2, 3, 5):
        tokens = Z.tokens_of(cfg["vocab"], n, 90 + n)
        want = {0: P.forward(cfg, w, tokens)}
        check(replay(runner, {0: tokens}, [[(0, n)]]), want, TOL["float32"], f"{n} tokens at once")
        check(replay(runner, {0: tokens}, [[(0, 1)]] * n), want, TOL["float32"], f"{n} tokens one by one")


# --- the engine: scheduler, sampling, captured steps ------------------------------------------------------------------
@pytest.mark.parametrize("dtype, graphs, pipelined", [("float32", False, False), ("float32", True, False),
                                                      ("float32", True, True), ("bfloat16", True, True)])
@pytest.mark.parametrize("which", ["r1", "r2"])
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


def test_the_command_line_generates(r2):
    """``bin/vipera generate`` on a Rebidra folder: the model is found by its configuration and run through the engine."""
    folder, cfg, w = r2
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


def test_the_trace_runner_replays_a_schedule(tmp_path, r1):
    """``bin/trace_run`` on a Rebidra folder: four slots, pages for the live requests only."""
    folder, cfg, w = r1
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
