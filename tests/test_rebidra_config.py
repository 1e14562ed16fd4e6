"""Rebidra without a GPU: reading its configuration, the layer specs and the run order built from it, what a request keeps,
declared tensors against folders, refused configurations, and the plain implementation's mechanisms against closed forms."""
import copy
import json
import math
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import vipera_rs_amd  # noqa: F401
import rebidra_helpers as Z
from plain import rebidra_plain as P
from vipera_rs_amd.config import RebidraConfig, config_from_dict
from vipera_rs_amd.errors import InvalidArgumentError, UnsupportedError
from vipera_rs_amd.models import check_model, declare_cache_needs, declare_model


def test_the_registry_finds_the_configuration_by_its_name():
    cfg = config_from_dict(Z.R1)
    assert isinstance(cfg, RebidraConfig) and (cfg.vocab, cfg.width, cfg.side_dim, cfg.loop) == (83, 48, 8, (1, 3, 2))
    for model in (Z.R1, Z.R2, Z.single(Z.windowed(2, 1, 8, 5)), Z.random_config(3)):
        cfg = config_from_dict(model)
        assert cfg.to_dict() == model and config_from_dict(cfg.to_dict()).to_dict() == model


def test_layer_specs_carry_every_size_and_constant():
    specs = config_from_dict(Z.R1).layer_specs()
    assert [s.block for s in specs] == ["prenorm"] * 4 and [s.prefix for s in specs] == ["l0.", "l1.", "l2.", "l3."]
    m = specs[2].mixer.params
    assert {k: m[k] for k in ("heads", "kv_heads", "head_dim", "window", "conv", "values", "qk_norm", "gate", "sink")} == \
        {"heads": 6, "kv_heads": 3, "head_dim": 8, "window": 19, "conv": 4, "values": "keys", "qk_norm": "head",
         "gate": "head_sigmoid", "sink": True}
    assert specs[0].position.params["ramp"] == {"factor": 8.0, "original": 64.0, "fast": 8.0, "slow": 1.0}
    assert specs[2].position.params["rotary_dim"] == 4 and "ramp" not in specs[2].position.params
    ffn = specs[2].ffn.params
    assert {k: ffn[k] for k in ("intermediate", "experts", "top", "shared", "form", "activation", "scores", "shared_gate")} == \
        {"intermediate": 32, "experts": 8, "top": 3, "shared": 16, "form": "plain", "activation": "relu2", "scores": "chosen",
         "shared_gate": "sigmoid"}
    assert [s.extras["after"].params["index"] for s in specs] == [0, 1, 2, 3]
    assert all(s.mixer_norm.params["bias"] is False for s in specs)
    other = config_from_dict(Z.R2).layer_specs()
    assert other[0].ffn.kind == "none" and other[1].ffn.params["shared"] is None and other[1].ffn.params["shared_gate"] is None
    assert other[1].position.kind == "none" and other[1].mixer.params["conv"] == 1


def test_the_run_order():
    order = [(e.layer, e.rejoins, e.cache_of) for e in config_from_dict(Z.R1).schedule()]
    assert order == [(0, False, None), (1, True, None), (2, False, None), (1, True, None), (2, False, None), (3, False, None)]
    assert [(i, enters) for i, enters, _ in order] == P.run_order(Z.R1)
    assert [e.layer for e in config_from_dict(Z.R2).schedule()] == [0, 1, 2, 1, 2, 1, 2]
    once = dict(Z.R1, loop={"start": 0, "stop": 1, "times": 1})
    assert [(e.layer, e.rejoins) for e in config_from_dict(once).schedule()] == [(0, True), (1, False), (2, False), (3, False)]
    assert config_from_dict(dict(Z.R1, loop=None)).rejoin_spec() is None
    assert not any(e.rejoins for e in config_from_dict(dict(Z.R1, loop=None)).schedule())


def test_what_a_request_keeps():
    needs = declare_cache_needs(config_from_dict(Z.R1))
    # every pass through the loop has pages and a state of its own
    assert [n.owner for n in needs] == list(range(6))
    assert [n.kv.window for n in needs] == [11, 11, 19, 11, 19, 11]
    assert (needs[2].kv.kv_heads, needs[2].kv.head_dim) == (3, 16)          # heads of 8 are padded to 16
    assert [n.state.shape for n in needs] == [(2 * 96,), (2 * 96,), (3 * 72,), (2 * 96,), (3 * 72,), (1 * 128,)]
    other = declare_cache_needs(config_from_dict(Z.R2))
    assert other[0].state.shape == (5 * 40,) and other[1].state is None      # one tap needs nothing of the past


def test_declared_tensors_match_a_folder(tmp_path):
    from vipera_rs_amd.weights import Checkpoint

    models = [("r1", Z.R1), ("r2", Z.R2), ("plain", Z.single(Z.windowed(2, 1, 8, 5), Z.moe(8, 2, 1)))]
    models += [(f"any{seed}", Z.random_config(seed)) for seed in range(6)]
    for name, cfg in models:
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
    # a layer without a feed-forward may have the norm in front of it stored all the same
    optional = {s.name for s in declare_model(config_from_dict(Z.R2)) if s.optional}
    assert optional == {"l0.norm2"}


def test_refused_configurations():
    def broken(change, base=Z.R1):
        cfg = copy.deepcopy(base)
        change(cfg)
        return cfg

    for error, change in (
            (UnsupportedError, lambda c: c["layers"][0].update(type="attention_2")),
            (UnsupportedError, lambda c: c["layers"][1].update(mlp={"kind": "dense", "ff": 8})),
            (InvalidArgumentError, lambda c: c["layers"][2]["mixer"].update(kv_heads=4)),
            (InvalidArgumentError, lambda c: c["layers"][2]["mixer"].update(vdim=16)),
            (InvalidArgumentError, lambda c: c["layers"][2]["mixer"].update(conv=0)),
            (InvalidArgumentError, lambda c: c["layers"][2]["mixer"]["mask"].update(size=0)),
            (InvalidArgumentError, lambda c: c["layers"][2]["mixer"]["rot"].update(dims=10)),
            (InvalidArgumentError, lambda c: c["layers"][2]["mixer"]["rot"].update(dims=3)),
            (InvalidArgumentError, lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("slow")),
            (InvalidArgumentError, lambda c: c["layers"][0]["mixer"].pop("scale")),
            (InvalidArgumentError, lambda c: c["layers"][0]["mlp"]["router"].update(top=6)),
            (InvalidArgumentError, lambda c: c["layers"][0]["mlp"]["shared"].update(ff=0)),
            (InvalidArgumentError, lambda c: c["loop"].update(stop=5)),
            (InvalidArgumentError, lambda c: c["loop"].update(start=3)),
            (InvalidArgumentError, lambda c: c["loop"].update(times=0)),
            (InvalidArgumentError, lambda c: c["token_side"].update(dim=0)),
            (InvalidArgumentError, lambda c: c.pop("norm"))):
        with pytest.raises(error):
            config_from_dict(broken(change))
    with pytest.raises(UnsupportedError):            # no kernel takes it: said when the model is opened
        check_model(config_from_dict(Z.single(Z.windowed(1, 1, 272, 5))), torch.bfloat16)


def test_mixers_that_take_values_from_keys_refuse_what_they_do_not_combine_with():
    from vipera_rs_amd.config.base import PartSpec
    from vipera_rs_amd.parts.attention import Attention

    base = {"hidden": 32, "heads": 2, "kv_heads": 1, "head_dim": 8, "name": "mix", "values": "keys", "conv": 3}
    Attention.check_supported(PartSpec("attention", dict(base, qk_norm="head", eps=1e-5)), torch.bfloat16)
    for extra in ({"qk_norm": "whole"}, {"qk_norm": "unit"}, {"maps": 2}, {"value_mix": "source"}, {"pairs": "interleaved"},
                  {"values": "queries"}):
        with pytest.raises(UnsupportedError):
            Attention.check_supported(PartSpec("attention", dict(base, **extra)), torch.bfloat16)
    with pytest.raises(InvalidArgumentError):
        Attention.check_supported(PartSpec("attention", dict(base, value_dim=16)), torch.bfloat16)
    names = {t.name for t in Attention.declare(PartSpec("attention", dict(base, qkv_bias=True)), "a.")}
    assert names == {"a.mix." + n for n in ("q_proj.weight", "q_proj.bias", "q_conv", "k_proj.weight", "k_proj.bias", "k_conv",
                                           "o_proj.weight")}


# --- the plain mechanisms against closed forms --------------------------------------------------------------------------
def test_masks():
    m = P.visible(3, 9)
    assert [j for j in range(9) if m[8, j]] == [6, 7, 8] and [j for j in range(9) if m[1, j]] == [0, 1]
    assert np.array_equal(P.visible(1, 4), np.eye(4, dtype=bool)) and np.array_equal(P.visible(0, 4), np.tri(4, dtype=bool))


def test_layer_norm_has_no_mean_and_unit_spread():
    x = np.random.default_rng(2).standard_normal((5, 40)) * 3 + 7
    y = P.layer_norm(x, np.ones(40), 0.0)
    assert np.allclose(y.mean(axis=1), 0) and np.allclose(y.var(axis=1), 1)
    assert np.allclose(P.layer_norm(x, np.full(40, 2.0), 0.0), 2 * y)
    assert np.allclose(P.layer_norm(np.array([[3.0, 1.0]]), np.ones(2), 3.0), [[0.5, -0.5]])        # eps inside the root


def test_the_convolution_starts_from_zeros_and_ends_at_the_current_token():
    x = np.arange(1.0, 13.0).reshape(6, 2)
    out = P.causal_conv(x, np.array([[0.0, 0.0, 1.0], [1.0, 0.0, 0.0]]))
    assert np.array_equal(out[:, 0], x[:, 0]) and np.array_equal(out[:, 1], [0, 0, 2, 4, 6, 8])
    assert np.array_equal(P.causal_conv(x, np.array([[3.0], [2.0]])), x * [3.0, 2.0])
    assert np.array_equal(P.causal_conv(x[:1], np.array([[5.0, 7.0, 1.0], [5.0, 7.0, 2.0]])), [[1.0, 4.0]])


def test_the_sink_joins_the_denominator_once_and_unscaled():
    q, k, v = np.zeros((2, 2, 4)), np.zeros((2, 1, 4)), np.ones((2, 1, 3))
    out = P.sink_attention(q, k, v, 100.0, P.visible(0, 2), np.array([0.0, math.log(2.0)]))
    # one zero score against exp(0) and 2; two against the same
    assert np.allclose(out[0, 0], 1 / 2) and np.allclose(out[0, 1], 1 / 3)
    assert np.allclose(out[1, 0], 2 / 3) and np.allclose(out[1, 1], 2 / 4)
    assert np.allclose(P.sink_attention(q, k, v, 1.0, P.visible(0, 2), np.array([900.0, -900.0]))[1], [[0.0] * 3, [1.0] * 3])


def test_blended_frequencies_and_the_amplitude():
    rot = {"dims": 16, "base": 500.0, "scaling": {"factor": 4.0, "original": 64, "fast": 8.0, "slow": 1.0}}
    base = 500.0 ** (-np.arange(8) / 8.0)
    want = [base[0], base[1] * (2 / 3 + 1 / 12), base[2] * (1 / 3 + 2 / 12)] + list(base[3:] / 4.0)
    assert np.allclose(P.frequencies(rot), want)
    assert math.isclose(P.amplitude(rot), 0.1 * math.log(4.0) + 1.0) and P.amplitude({"dims": 16}) == P.amplitude(None) == 1.0
    x = np.random.default_rng(3).standard_normal((1, 1, 20))
    turned = P.rotate(x, [7], rot)
    assert np.allclose(turned[..., 16:], x[..., 16:])                        # the rest passes unchanged
    norm2 = lambda a, i: a[..., i] ** 2 + a[..., i + 8] ** 2
    assert np.allclose(norm2(turned, 3), P.amplitude(rot) ** 2 * norm2(x, 3))  # i and i + dims / 2 are a pair
    assert np.allclose(P.rotate(x, [0], {"dims": 16, "base": 500.0}), x)


def test_values_are_the_convolved_keys_ahead_of_norm_and_rotation():
    """With one visible position the output is the token's own value, whatever its key became."""
    m = Z.windowed(2, 1, 4, 1, conv=2)["mixer"]
    rng = np.random.default_rng(4)
    w = {"q": rng.standard_normal((8, 6)), "q.b": rng.standard_normal(8), "q.conv": rng.standard_normal((8, 2)),
         "k": rng.standard_normal((4, 6)), "k.b": rng.standard_normal(4), "k.conv": rng.standard_normal((4, 2)),
         "q.norm": rng.standard_normal(4), "k.norm": rng.standard_normal(4), "sink": np.full(2, -1e9), "g": np.zeros((2, 6)),
         "o": np.eye(8)}
    x = rng.standard_normal((5, 6))
    u = x @ w["k"].T + w["k.b"]
    v = w["k.conv"][:, 1] * u
    v[1:] += w["k.conv"][:, 0] * u[:-1]
    assert np.allclose(P.attention(x, w, "", m, 1e-5), 0.5 * np.concatenate([v, v], axis=1))      # a gate of sigmoid(0)


def test_routing_weighs_the_chosen_experts_only():
    ids, weights = P.choose(np.array([[1.0, 3.0, 2.0, -5.0], [0.0, 0.0, 0.0, 0.0]]), 2)
    assert ids.tolist() == [[1, 2], [0, 1]] and np.allclose(weights[0], np.exp([3.0, 2.0]) / np.exp([3.0, 2.0]).sum())
    assert np.allclose(weights[1], 0.5)
    x = np.array([[2.0, -1.0]])
    w = {"router": np.zeros((2, 2)), "router.b": np.array([0.0, 5.0]), "shared.sg": np.array([[1.0, 2.0]])}
    for name, factor in (("e0.", 100.0), ("e1.", 1.0), ("shared.", 10.0)):
        w[name + "up"], w[name + "down"] = np.eye(2), factor * np.eye(2)
    mlp = Z.moe(2, 2, 1, 2)
    # the bias chooses expert 1; the square of relu; the shared expert at sigmoid(2 - 2) = 1/2
    assert np.allclose(P.mixture(x, w, "", mlp), [[4.0 + 0.5 * 40.0, 0.0]])
    assert np.allclose(P.mixture(x, w, "", Z.moe(2, 2, 1)), [[4.0, 0.0]])


def test_a_loop_joins_the_stream_first_and_the_embedding_second():
    w = {k: t.double().numpy() for k, t in Z.make_weights(Z.R1, 1).items()}
    tokens, width = Z.tokens_of(83, 9, 3), 48
    seen = []
    quiet = dict(w)      # silent layers: only the loop changes the stream
    for name in w:
        if name.endswith((".mix.o", ".side.norm", ".down")):
            quiet[name] = w[name] * 0.0
    P.forward(Z.R1, quiet, tokens, seen)
    x0 = w["embed"][tokens] * 1.5
    a, b = w["loop.in"][:, :width].T, w["loop.in"][:, width:].T
    once = x0 @ a + x0 @ b
    assert np.allclose(seen[0], x0) and np.allclose(seen[1], once) and np.allclose(seen[2], once)
    assert np.allclose(seen[3], once @ a + x0 @ b) and np.allclose(seen[5], seen[3]) and len(seen) == 6


def test_every_pass_reads_the_layers_own_columns_of_the_side_table():
    w = {k: t.double().numpy() for k, t in Z.make_weights(Z.R1, 1).items()}
    tokens = Z.tokens_of(83, 9, 3)
    base, moved, got, want = dict(w), dict(w), [], []
    moved["side.embed"] = w["side.embed"].copy()
    moved["side.embed"][:, 2 * 8:3 * 8] += 1.0             # layer 2's columns
    P.forward(Z.R1, moved, tokens, got)
    P.forward(Z.R1, base, tokens, want)
    assert [bool(np.allclose(a, b)) for a, b in zip(got, want)] == [True, True, False, False, False, False]


def test_a_plan_counts_a_looped_layers_weights_once_a_pass(tmp_path):
    from vipera_rs_amd.cli import plan_model
    from vipera_rs_amd.models import tensor_reads

    reads = tensor_reads(config_from_dict(Z.R1))
    assert (reads["l0.mix.q"], reads["l1.mix.q"], reads["l2.mlp.e3.up"], reads["l3.mix.o"], reads["loop.in"]) == (1, 2, 2, 1, 2)
    steps = [plan_model(Z.make_folder(tmp_path / str(times), dict(Z.R1, loop={"start": 1, "stop": 3, "times": times}), 3), 64, 1,
                        "bfloat16", 16)["decode_step_read_bytes"] for times in (1, 2, 3)]
    kept = [n for n in declare_cache_needs(config_from_dict(Z.R1))[1:3]]
    per_pass = sum(2 * math.prod(s.shape) for s in declare_model(config_from_dict(Z.R1))
                   if s.role == "matrix" and (s.name.startswith(("l1.", "l2.")) or s.name == "loop.in"))
    per_pass += sum(64 * n.kv.bytes_per_position(2) + n.state.bytes_per_slot() for n in kept)
    assert steps[1] - steps[0] == steps[2] - steps[1] == per_pass


def test_model_info_names_the_architecture(tmp_path):
    folder = Z.make_folder(tmp_path / "r2", Z.R2, 5)
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    done = subprocess.run([sys.executable, os.path.join(root, "bin", "vipera"), "model-info", folder], capture_output=True,
                          text=True, timeout=300)
    assert done.returncode == 0, done.stderr[-2000:]
    assert "Rebidra" in done.stdout
    assert json.load(open(os.path.join(folder, "config.json"))) == Z.R2
