"""Zeladra without a GPU: reading its configuration, the layer specs built from it, what a request keeps, declared
tensors against folders, refused configurations, the rotation's tables and reordered rows, and the plain implementation's
mechanisms against closed forms."""
import copy
import json
import math
import os
import subprocess
import sys
from types import SimpleNamespace

import numpy as np
import pytest
import torch

import vipera_rs_amd  # noqa: F401
import zeladra_helpers as Z
from plain import zeladra_plain as P
from vipera_rs_amd.config import ZeladraConfig, config_from_dict
from vipera_rs_amd.config.base import PartSpec
from vipera_rs_amd.errors import InvalidArgumentError, UnsupportedError
from vipera_rs_amd.models import check_model, declare_cache_needs, declare_model
from vipera_rs_amd.parts.rotary import RotaryNeox, blend_by_index, pairs_apart


def test_the_registry_finds_the_configuration_by_its_name():
    cfg = config_from_dict(Z.Z1)
    assert isinstance(cfg, ZeladraConfig) and (cfg.vocab, cfg.width, cfg.streams, cfg.embedding_scale) == (83, 48, 2, 1.5)
    assert config_from_dict(cfg.to_dict()).to_dict() == cfg.to_dict()


def test_layer_specs_carry_every_size_and_constant():
    specs = config_from_dict(Z.Z1).layer_specs()
    assert [s.block for s in specs] == ["hyper"] * 4 and all(s.params["streams"] == 2 for s in specs)
    space, first, window, second = (s.mixer for s in specs)
    assert space.kind == "state_space"
    assert {k: space.params[k] for k in ("heads", "vdim", "state", "groups", "norm_groups", "conv")} == \
        {"heads": 4, "vdim": 12, "state": 20, "groups": 2, "norm_groups": 2, "conv": 4}
    assert first.kind == "latent_attention" and first.params["gate"] == "head_sigmoid" and not first.params["shares_cache"]
    assert first.params["pairs"] == "interleaved" and first.params["rotary_dim"] == 8
    assert second.params["shares_cache"] and second.params["heads"] == 2 and second.params["vdim"] == 24
    assert specs[1].position.params["ramp"] == {"factor": 8.0, "original": 64.0, "fast": 8.0, "slow": 1.0}
    assert window.kind == "attention" and window.params["window"] == 11 and window.params["keep_first"] == 3
    assert "ramp" not in specs[2].position.params and specs[2].position.params["rotary_dim"] == 8
    assert specs[0].ffn.kind == "none" and specs[0].position.kind == "none"
    assert specs[1].ffn.params["intermediate"] == 40 and specs[1].ffn.params["activation"] == "silu"
    assert [e.cache_of for e in config_from_dict(Z.Z1).schedule()] == [None, None, None, 1]


def test_what_a_request_keeps():
    needs = declare_cache_needs(config_from_dict(Z.Z1))
    assert needs[0].kv is None and needs[0].state.shape == (4 * 12 * 20 + 3 * (48 + 2 * 2 * 20),)
    assert (needs[1].kv.kv_heads, needs[1].kv.head_dim, needs[1].kv.window) == (1, 32, 0)
    # kept first positions lie outside the window's bookkeeping: that layer keeps all its pages
    assert needs[2].kv.window == 0 and needs[3].owner == 1
    wide = declare_cache_needs(config_from_dict(Z.Z2))
    assert wide[1].kv.window == 7 and wide[1].kv.head_dim == 32        # values wider than keys: one padded width
    assert wide[3].owner == 0 and wide[5].owner == 5
    assert wide[2].state.shape[0] % 4 == 0 and wide[2].state.shape[0] >= 6 * 10 * 8 + 60 + 2 * 3 * 7


def test_declared_tensors_match_a_folder(tmp_path):
    from vipera_rs_amd.weights import Checkpoint

    for name, cfg in (("z1", Z.Z1), ("z2", Z.Z2)):
        folder = Z.make_folder(tmp_path / name, cfg, 3)
        specs = declare_model(config_from_dict(cfg))
        checkpoint = Checkpoint(folder)
        try:
            checkpoint.check(specs)
            assert {s.name for s in specs if not s.optional} == set(checkpoint.names())
        finally:
            checkpoint.close()
        for dtype in (torch.bfloat16, torch.float32):
            check_model(config_from_dict(cfg), dtype)


def test_refused_configurations():
    def broken(change, base=Z.Z1):
        cfg = copy.deepcopy(base)
        change(cfg)
        return cfg

    for error, change in (
            (UnsupportedError, lambda c: c["layers"][0].update(type="mamba")),
            (UnsupportedError, lambda c: c["layers"][1].update(mlp={"kind": "moe"})),
            (InvalidArgumentError, lambda c: c["layers"][2]["mixer"].update(kv_heads=3)),
            (InvalidArgumentError, lambda c: c["layers"][2]["mixer"]["rot"].update(dims=7)),
            (InvalidArgumentError, lambda c: c["layers"][2]["mixer"]["mask"].update(size=0)),
            (InvalidArgumentError, lambda c: c["layers"][3]["mixer"].update(kv_from=2)),
            (InvalidArgumentError, lambda c: c["layers"][3]["mixer"].update(kv_from=3)),
            (InvalidArgumentError, lambda c: c["layers"][3]["mixer"].update(kv_rank=32)),
            (InvalidArgumentError, lambda c: c["layers"][3]["mixer"]["rot"].update(base=501.0)),
            (InvalidArgumentError, lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].update(factor=0.0)),
            (InvalidArgumentError, lambda c: c["layers"][0]["mixer"].update(groups=3)),
            (InvalidArgumentError, lambda c: c["layers"][0]["mixer"].update(norm_groups=5)),
            (InvalidArgumentError, lambda c: c["layers"][1]["mixer"].pop("scale")),
            (InvalidArgumentError, lambda c: c.pop("norm"))):
        with pytest.raises(error):
            config_from_dict(broken(change))
    for change in (lambda c: c.update(streams=9), lambda c: c["layers"][0]["mixer"].update(state=257),
                   lambda c: [layer["mixer"].update(kv_rank=256) for layer in c["layers"] if "kv_rank" in layer["mixer"]]):
        with pytest.raises(UnsupportedError):            # no kernel takes it: said when the model is opened
            check_model(config_from_dict(broken(change)), torch.bfloat16)


# --- the rotation -------------------------------------------------------------------------------------------------------
def test_blended_frequencies_and_the_amplitude():
    rot = {"dims": 16, "base": 500.0, "scaling": {"factor": 4.0, "original": 64, "fast": 8.0, "slow": 1.0}}
    base = 500.0 ** (-np.arange(8) / 8.0)
    # the pair whose wave makes exactly n turns in 64 positions has the index log(64 / (2 pi n)) / log(500) * 8
    low = math.floor(8 * math.log(64 / (2 * math.pi * 8)) / math.log(500.0))
    high = math.ceil(8 * math.log(64 / (2 * math.pi)) / math.log(500.0))
    assert (low, high) == (0, 3)
    want = [base[0], base[1] * (2 / 3 + 1 / 12), base[2] * (1 / 3 + 2 / 12)] + list(base[3:] / 4.0)
    assert np.allclose(P.frequencies(rot), want)
    assert np.allclose(blend_by_index(base, 16, 500.0, 4.0, 64, 8.0, 1.0), want)
    assert math.isclose(P.amplitude(rot), 0.1 * math.log(4.0) + 1.0) and P.amplitude({"dims": 16}) == 1.0
    # a ramp of no width: everything from the one index on is divided
    same = blend_by_index(base, 16, 500.0, 4.0, 64, 2.0, 2.0)
    assert np.all((np.abs(same - base) < 1e-12) | (np.abs(same - base / 4.0) < 1e-12) | (np.arange(8) < 3))
    part = RotaryNeox(PartSpec("rotary_neox", {"head_dim": 16, "rotary_dim": 16, "base": 500.0, "wide_table": True,
                                               "ramp": dict(rot["scaling"])}), "", SimpleNamespace(device="cpu"))
    assert np.allclose(part.inv_freq.numpy(), want, rtol=1e-7) and math.isclose(part.amplitude, P.amplitude(rot))


def test_reordered_rows_turn_neighbouring_pairs_as_distant_ones():
    rng = np.random.default_rng(0)
    heads, dim, first, dims = 3, 14, 4, 8
    weight = rng.standard_normal((heads * dim, 5))
    moved = pairs_apart(torch.from_numpy(weight), heads, dim, first, dims).numpy().reshape(heads, dim, 5)
    plain = weight.reshape(heads, dim, 5)
    assert np.array_equal(moved[:, :first], plain[:, :first]) and np.array_equal(moved[:, first + dims:], plain[:, first + dims:])
    for i in range(dims // 2):
        assert np.array_equal(moved[:, first + i], plain[:, first + 2 * i])
        assert np.array_equal(moved[:, first + dims // 2 + i], plain[:, first + 2 * i + 1])


def test_rotation_enters_scores_by_distance_only():
    rng = np.random.default_rng(1)
    q, k = rng.standard_normal((1, 1, 12)), rng.standard_normal((1, 1, 12))
    rot = {"dims": 8, "base": 100.0}
    dots = [float(np.sum(P.rotate(q, [a], rot) * P.rotate(k, [a - 5], rot))) for a in (5, 9, 300)]
    assert np.allclose(dots, dots[0]) and not np.isclose(dots[0], float(np.sum(q * k)))
    turned = P.rotate(q, [7], rot)
    assert np.allclose(turned[..., 8:], q[..., 8:])                        # the rest passes unchanged
    assert np.allclose(turned[..., 0] ** 2 + turned[..., 1] ** 2, q[..., 0] ** 2 + q[..., 1] ** 2)      # neighbours are a pair


# --- the plain mechanisms against closed forms --------------------------------------------------------------------------
def test_masks():
    m = P.visible(3, 2, 9)
    assert [j for j in range(9) if m[8, j]] == [0, 1, 6, 7, 8] and [j for j in range(9) if m[3, j]] == [0, 1, 2, 3]
    assert [j for j in range(9) if P.visible(3, 0, 9)[8, j]] == [6, 7, 8] and np.all(P.visible(0, 0, 4) == np.tri(4, dtype=bool))


def test_layer_norm_has_no_mean_and_unit_spread():
    x = np.random.default_rng(2).standard_normal((5, 40)) * 3 + 7
    y = P.layer_norm(x, np.ones(40), np.zeros(40), 0.0)
    assert np.allclose(y.mean(axis=1), 0) and np.allclose(y.var(axis=1), 1)
    assert np.allclose(P.layer_norm(x, np.full(40, 2.0), np.full(40, 0.5), 0.0), 2 * y + 0.5)
    assert np.allclose(P.layer_norm(np.ones((1, 4)), np.ones(4), np.zeros(4), 1e-5), 0.0)


def test_the_recurrence_is_a_decayed_sum():
    rng = np.random.default_rng(3)
    T, H, V, G, N = 9, 4, 3, 2, 5
    xs, B, C = rng.standard_normal((T, H, V)), rng.standard_normal((T, G, N)), rng.standard_normal((T, G, N))
    dt, a_log, skip = rng.uniform(0.1, 2.0, (T, H)), rng.uniform(-1, 1, H), rng.standard_normal(H)
    y = P.state_space(xs, B, C, dt, a_log, skip)
    for h in range(H):
        g, rate = h // 2, math.exp(a_log[h])
        for t in range(T):
            want = sum(math.exp(-rate * dt[s + 1:t + 1, h].sum()) * dt[s, h] * (B[s, g] @ C[t, g]) * xs[s, h]
                       for s in range(t + 1)) + skip[h] * xs[t, h]
            assert np.allclose(y[t, h], want)


def test_the_gate_comes_before_the_norm_of_each_part():
    rng = np.random.default_rng(4)
    y, z, weight = rng.standard_normal((3, 12)), rng.standard_normal((3, 12)), rng.standard_normal(12)
    out = P.gated_group_norm(y, z, weight, 3, 0.0)
    v = y * P.silu(z)
    for part in range(3):
        cols = slice(4 * part, 4 * part + 4)
        assert np.allclose(out[:, cols], v[:, cols] / np.sqrt((v[:, cols] ** 2).mean(axis=1, keepdims=True)) * weight[cols])


def test_the_convolution_starts_from_zeros_and_ends_at_the_current_token():
    x = np.arange(12.0).reshape(6, 2)
    out = P.causal_conv(x, np.array([[0.0, 0.0, 1.0], [1.0, 0.0, 0.0]]), np.array([0.0, 5.0]))
    assert np.array_equal(out[:, 0], x[:, 0]) and np.array_equal(out[:, 1], [5, 5, 6, 8, 10, 12])


def test_one_stream_with_plain_weights_is_the_residual_sum():
    rng = np.random.default_rng(5)
    x = rng.standard_normal((1, 4, 6))
    w = {"c.in": np.ones(1), "c.out": np.ones(1), "c.mix": np.ones((1, 1))}
    assert np.allclose(P.hyper_connection(x, w, "c.", np.sin)[0], x[0] + np.sin(x[0]))
    # the mix matrix goes from row to column: only stream 0 reaches stream 1 here, and nothing reaches stream 0
    w = {"c.in": np.array([2.0, 0.0]), "c.out": np.array([0.0, 3.0]), "c.mix": np.array([[0.0, 1.0], [0.0, 0.0]])}
    two = rng.standard_normal((2, 4, 6))
    out = P.hyper_connection(two, w, "c.", np.sin)
    assert np.allclose(out[0], 0.0) and np.allclose(out[1], two[0] + 3.0 * np.sin(2.0 * two[0]))


def test_a_latent_layer_reads_another_layers_rows():
    """With both layers' own weights equal, the reading layer still follows the rows of the one it names."""
    w = {k: t.double().numpy() for k, t in Z.make_weights(Z.Z2, 1).items()}
    tokens = Z.tokens_of(61, 12, 3)
    want = P.forward(Z.Z2, w, tokens)
    moved = dict(w)
    moved["l0.mix.dkv"] = w["l0.mix.dkv"] + 0.05
    silent = copy.deepcopy(moved)
    silent["l0.mix.uk"], silent["l0.mix.uv"] = w["l0.mix.uk"] * 0, w["l0.mix.uv"] * 0       # layer 0 itself says nothing
    quiet = copy.deepcopy(w)
    quiet["l0.mix.uk"], quiet["l0.mix.uv"] = silent["l0.mix.uk"], silent["l0.mix.uv"]
    assert not np.allclose(P.forward(Z.Z2, moved, tokens), want)
    assert not np.allclose(P.forward(Z.Z2, silent, tokens), P.forward(Z.Z2, quiet, tokens), atol=1e-6)


def test_model_info_names_the_architecture(tmp_path):
    folder = Z.make_folder(tmp_path / "z2", Z.Z2, 5)
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    done = subprocess.run([sys.executable, os.path.join(root, "bin", "vipera"), "model-info", folder], capture_output=True,
                          text=True, timeout=300)
    assert done.returncode == 0, done.stderr[-2000:]
    assert "Zeladra" in done.stdout
    assert json.load(open(os.path.join(folder, "config.json"))) == Z.Z2
