"""Balalorn without a GPU: configuration and its refusals, the builder's tensor names, cache
groups, shared latents and state slots, and the plain model's mechanisms worked by hand."""

from __future__ import annotations

import copy
import math

import pytest
import torch

from kvforge_amd import registry
from kvforge_amd.config import BalalornConfig, ConfigError
from kvforge_amd.config.presets import PRESETS, balalorn as make_config
from kvforge_amd.models.transformer import Transformer
from kvforge_amd.parts import (GatedDelta, GatedFeedForward, LatentAttention, Mamba2, NamedRMSNorm, PostNormBlock,
                               RotaryPositions, RoutedExperts)
from kvforge_amd.weights.random_init import random_tensors
from tests.plain import balalorn as plain

SSM = dict(heads=6, vdim=20, state=24, groups=3, norm_groups=4, conv=3)
DELTA = dict(heads=6, kv_heads=2, dim=28, vdim=36, conv=5)
LAT = dict(heads=5, dim=20, rot_dim=12, vdim=28, kv_rank=44, scale=0.21, base=3000.0)


def config(**kw):
    base = dict(vocab=203, width=88, layers=[("mamba2", SSM, (24, 7, 2)), ("latent_attention", LAT, 104),
                                             ("delta", DELTA, None),
                                             ("latent_attention", dict(LAT, heads=3, dim=8, vdim=12, kv_from=1),
                                              (40, 3, 3))], eps=1e-5)
    base.update(kw)
    return make_config(**base)


def test_configuration_reads_every_key_and_writes_it_back():
    cfg = registry.config_from_dict(config())
    assert isinstance(cfg, BalalornConfig)
    assert (cfg.vocab_size, cfg.width, cfg.norm_eps, cfg.num_hidden_layers, cfg.hidden_size) == (203, 88, 1e-5, 4, 88)
    s, a, d, b = (x.mixer for x in cfg.layers)
    assert (s.heads, s.vdim, s.state, s.groups, s.norm_groups, s.conv) == (6, 20, 24, 3, 4, 3)
    assert (d.heads, d.kv_heads, d.dim, d.vdim, d.conv) == (6, 2, 28, 36, 5)
    assert (a.heads, a.dim, a.rot_dim, a.vdim, a.kv_rank, a.scale, a.kv_from) == (5, 20, 12, 28, 44, 0.21, None)
    assert (a.rot.base, a.rot.dims) == (3000.0, 12) and b.kv_from == 1 and b.heads == 3
    m = [x.mlp for x in cfg.layers]
    assert (m[0].kind, m[0].ff, m[0].experts, m[0].top) == ("moe", 24, 7, 2)
    assert (m[1].kind, m[1].ff) == ("dense", 104) and m[2] is None and m[3].top == 3
    assert registry.config_from_dict(cfg.to_dict()).to_dict() == cfg.to_dict()
    for name in ("balalorn-tiny", "balalorn-1b"):
        registry.build_spec(registry.config_from_dict(PRESETS[name]))


def test_what_a_file_may_leave_out():
    d = config()
    del d["layers"][0]["mixer"]["groups"], d["layers"][0]["mixer"]["norm_groups"]
    del d["layers"][2]["mixer"]["kv_heads"], d["layers"][2]["mixer"]["vdim"]
    cfg = registry.config_from_dict(d)
    assert (cfg.layers[0].mixer.groups, cfg.layers[0].mixer.norm_groups) == (6, 1)
    assert (cfg.layers[2].mixer.kv_heads, cfg.layers[2].mixer.vdim) == (6, 28)
    assert cfg.max_position_embeddings == 131072


@pytest.mark.parametrize("change,match", [
    (lambda d: d["layers"][0].update(type="attention"), "not supported"),
    (lambda d: d["layers"][0]["mlp"].update(kind="glu"), "not supported"),
    (lambda d: d["layers"][0]["mixer"].update(groups=4), "multiple of groups"),
    (lambda d: d["layers"][0]["mixer"].update(norm_groups=7), "multiple of norm_groups"),
    (lambda d: d["layers"][0]["mixer"].update(state=300), "256"),
    (lambda d: d["layers"][0]["mixer"].update(conv=9), "8 taps"),
    (lambda d: d["layers"][0]["mlp"]["router"].update(top=8), "exceeds the 7 experts"),
    (lambda d: d["layers"][2]["mixer"].update(kv_heads=4), "multiple of kv_heads"),
    (lambda d: d["layers"][1]["mixer"].update(kv_rank=700), "must not exceed 640"),
    (lambda d: d["layers"][1]["mixer"]["rot"].update(dims=14), "exceeds rot_dim"),
    (lambda d: d["layers"][1]["mixer"]["rot"].update(dims=7), "must be even"),
    (lambda d: d["layers"][1]["mixer"].update(scale=0.0), "positive"),
    (lambda d: d["layers"][3]["mixer"].update(kv_from=0), "latents of its own"),
    (lambda d: d["layers"][3]["mixer"].update(kv_from=3), "latents of its own"),
    (lambda d: d["layers"][3]["mixer"].update(kv_rank=48), "must equal"),
    (lambda d: d["layers"][3]["mixer"]["rot"].update(base=10.0), "must equal"),
    (lambda d: d["layers"][1]["mixer"].update(kv_from=-1), "earlier layer"),
    (lambda d: d.update(layers=[]), "at least one layer"),
    (lambda d: d.pop("norm"), "norm"),
])
def test_refusals(change, match):
    d = copy.deepcopy(config())
    change(d)
    with pytest.raises((ConfigError, KeyError), match=match):
        registry.build_spec(registry.config_from_dict(d))


def test_parts_refuse_what_their_kernels_do_not_compute():
    with pytest.raises(ValueError, match="up to 256"):
        GatedDelta("m", 32, 2, 1, 300, 16, 4, 1e-5)
    with pytest.raises(ValueError, match="divide the heads"):
        GatedDelta("m", 32, 3, 2, 16, 16, 4, 1e-5)
    with pytest.raises(ValueError, match="1 to 8 taps"):
        Mamba2("m", 32, 2, 1, 16, 16, 9, 1, 1e-5)
    with pytest.raises(ValueError, match="equal parts"):
        Mamba2("m", 32, 2, 1, 16, 16, 4, 5, 1e-5)
    with pytest.raises(ValueError, match="come together"):
        PostNormBlock(Mamba2("m", 32, 2, 1, 16, 16, 4, 1, 1e-5), NamedRMSNorm("n", 32, 1e-5),
                      GatedFeedForward("f", 32, 16))
    with pytest.raises(ValueError, match="unknown router scores"):
        RoutedExperts("f", 32, 16, 4, 2, scores="tanh")
    with pytest.raises(ValueError, match="without identity"):
        RoutedExperts("f", 32, 16, 4, 2, identity=1, weigh_input=True)
    with pytest.raises(ValueError, match="up to 640"):
        LatentAttention("a", 32, 2, 16, 16, 16, 640, None, 0.1, 1e-5)
    with pytest.raises(ValueError, match="without a scaling"):
        from kvforge_amd.config.model import RopeScaling
        RotaryPositions(8, 100.0, RopeScaling("llama3", 2.0, 1.0, 4.0, 64), rounded_once=True)


def test_tensor_names_and_parts_per_layer():
    spec = registry.build_spec(registry.config_from_dict(config()))
    names = spec.weight_specs()
    sh = lambda n: names[n].shape  # noqa: E731
    assert sh("embed") == (203, 88) and sh("head") == (203, 88) and sh("final.norm") == (88,)
    assert sh("l0.mix.in") == (120 + 120 + 72 + 72 + 6, 88) and sh("l0.mix.conv") == (264, 3)
    assert sh("l0.mix.conv.b") == (264,) and sh("l0.mix.norm") == (120,) and sh("l0.mix.o") == (88, 120)
    assert all(sh(f"l0.mix.{n}") == (6,) for n in ("dt_bias", "A_log", "D"))
    assert sh("l0.mlp.router") == (7, 88) and "l0.mlp.correction" not in names
    assert sh("l0.mlp.e6.gate") == (24, 88) and sh("l0.mlp.e6.down") == (88, 24) and "l0.mlp.e7.up" not in names
    assert sh("l1.mix.q") == (160, 88) and sh("l1.mix.dkv") == (56, 88) and sh("l1.mix.dkv.norm") == (44,)
    assert sh("l1.mix.uk") == (100, 44) and sh("l1.mix.uv") == (140, 44) and sh("l1.mix.g") == (5, 88)
    assert sh("l1.mix.o") == (88, 140) and sh("l1.mlp.gate") == (104, 88)
    assert sh("l2.mix.q") == (56, 88) and sh("l2.mix.k.conv") == (56, 5) and sh("l2.mix.v.conv") == (216, 5)
    assert sh("l2.mix.g") == (216, 88) and sh("l2.mix.a") == (6, 88) and sh("l2.mix.b") == (6, 88)
    assert sh("l2.mix.norm") == (36,) and "l2.norm2" not in names and "l2.norm1" in names
    assert sh("l3.mix.q") == (60, 88) and "l3.mix.dkv" not in names and sh("l3.mix.uk") == (24, 44)
    b = spec.blocks
    assert all(isinstance(x, PostNormBlock) and isinstance(x.norm, NamedRMSNorm) for x in b)
    assert [type(x.mixer) for x in b] == [Mamba2, LatentAttention, GatedDelta, LatentAttention]
    assert isinstance(b[0].ffn, RoutedExperts) and isinstance(b[1].ffn, GatedFeedForward) and b[2].ffn is None
    assert b[1].mixer.rotary is b[3].mixer.rotary and len(spec.positions) == 1         # equal rotations share tables
    assert [c.cache_of for c in spec.run_order()] == [None, None, None, 1]


def test_one_layers_pages_serve_both_latent_layers_and_memories_have_slots():
    model = Transformer(registry.build_spec(registry.config_from_dict(config())), torch.float32, "cpu")
    assert len(model.cache_groups) == 1 and model.cache_groups[0].layers == (1,)
    assert [p.shape for p in model.cache_groups[0].pages] == [(1, "block", 64), (1, 64, "block")]
    assert sorted(model.state_specs) == [0, 2]
    assert model.state_specs[0].shape == (6 * 24 * 20 + 2 * (120 + 2 * 72),)
    assert model.state_specs[2].shape == (6 * 28 * 36 + 4 * (2 * 56 + 216),)


def test_frequencies_are_rounded_once():
    r = RotaryPositions(12, 70000.0, interleaved=True, rounded_once=True)
    want = torch.tensor([70000.0 ** (-2.0 * i / 12) for i in range(6)], dtype=torch.float64).float()
    assert torch.equal(r.inv_freq, want)


# ---------------------------------------------------------------------------- mechanisms by hand
def sig(z):
    return 1.0 / (1.0 + math.exp(-z))


def test_convolution_looks_back_and_its_last_column_meets_the_token():
    x = torch.tensor([[1.0, 10.0], [2.0, 20.0], [4.0, 40.0]])
    taps = torch.tensor([[0.5, 0.0, 1.0], [0.0, 0.1, 0.0]])
    y = plain.short_conv(x, taps, torch.tensor([0.25, 0.0]))
    for t, pre in enumerate([(1.25, 0.0), (2.25, 1.0), (4.0 + 0.5 + 0.25, 2.0)]):
        for c in range(2):
            assert abs(float(y[t, c]) - pre[c] * sig(pre[c])) < 1e-6


def test_two_tokens_of_the_delta_rule():
    q = torch.tensor([[[1.0, 2.0]], [[3.0, -1.0]]])
    k = torch.tensor([[[0.6, 0.8]], [[1.0, 0.0]]])
    v = torch.tensor([[[1.0, 10.0]], [[2.0, 0.0]]])
    g, beta = torch.tensor([[0.5], [0.25]]), torch.tensor([[0.5], [0.8]])
    o = plain.delta_scan(q, k, v, g, beta)
    # S_0 = k_0 (beta_0 v_0)^T; the read-out sees the token's own write
    torch.testing.assert_close(o[0, 0], (1.0 * 0.6 + 2.0 * 0.8) * 0.5 * v[0, 0])
    # the memory has decayed before it answers to k_1: g_1 S_0^T k_1 = 0.25 * 0.6 * 0.5 v_0
    u = 0.8 * (v[1, 0] - 0.25 * 0.6 * 0.5 * v[0, 0])
    want = (3.0 * 0.6 - 1.0 * 0.8) * 0.25 * 0.5 * v[0, 0] + 3.0 * u
    torch.testing.assert_close(o[1, 0], want)


def test_two_tokens_of_the_state_space_memory():
    C = torch.tensor([[[1.0, 2.0]], [[3.0, -1.0]]])
    B = torch.tensor([[[0.5, 1.0]], [[2.0, 0.0]]])
    x = torch.tensor([[[1.0, 10.0], [3.0, 0.0]], [[2.0, 0.0], [1.0, 1.0]]])     # two heads over one group
    a, dt = torch.tensor([[0.9, 0.9], [0.5, 0.1]]), torch.tensor([[0.2, 1.0], [0.4, 2.0]])
    y = plain.ssd_scan(C, B, x, a, dt)
    torch.testing.assert_close(y[0, 0], 2.5 * 0.2 * x[0, 0])
    torch.testing.assert_close(y[1, 0], 0.5 * 0.2 * 0.5 * x[0, 0] + 0.4 * 6.0 * x[1, 0])
    torch.testing.assert_close(y[1, 1], 0.5 * 1.0 * 0.1 * x[0, 1] + 2.0 * 6.0 * x[1, 1])


def test_unit_vectors_and_softplus():
    torch.testing.assert_close(plain.unit(torch.tensor([[3.0, 4.0]])), torch.tensor([[0.6, 0.8]]))
    assert float(plain.unit(torch.zeros(1, 3)).abs().max()) == 0.0
    torch.testing.assert_close(plain.softplus(torch.tensor([0.0, 30.0, -30.0])),
                               torch.tensor([math.log(2.0), 30.0, math.exp(-30.0)]))


def test_the_norm_of_the_gated_row_is_taken_part_by_part():
    w = {"m.in": torch.zeros(4 + 4 + 2 + 2 + 2, 3), "m.conv": torch.ones(8, 1), "m.conv.b": torch.zeros(8),
         "m.dt_bias": torch.full((2,), -40.0), "m.A_log": torch.zeros(2), "m.D": torch.tensor([1.0, 2.0]),
         "m.norm": torch.tensor([1.0, 2.0, 3.0, 4.0]), "m.o": torch.eye(4)}
    w["m.in"][0:4, 0] = torch.tensor([1.0, 2.0, 3.0, 4.0])          # z
    w["m.in"][4:8, 1] = torch.tensor([1.0, -1.0, 0.5, 2.0])         # x
    m = dict(heads=2, vdim=2, state=2, groups=1, norm_groups=2)
    y = plain.mamba2_mixer(torch.tensor([[1.0, 1.0, 0.0]]), w, "m.", m, 1e-6)[0]
    # the step size is all but zero: what is left is D x; silu on x and on z, two parts of two elements
    xs = [v * sig(v) for v in (1.0, -1.0, 0.5, 2.0)]
    u = [d * x * z * sig(z) for d, x, z in zip((1.0, 1.0, 2.0, 2.0), xs, (1.0, 2.0, 3.0, 4.0))]
    for i in range(4):
        lo = i // 2 * 2
        r = math.sqrt((u[lo] ** 2 + u[lo + 1] ** 2) / 2 + 1e-6)
        assert abs(float(y[i]) - u[i] / r * (i + 1)) < 1e-4


def test_the_gate_of_a_head_and_a_layers_latents():
    torch.manual_seed(0)
    T, W = 4, 6
    m = dict(heads=2, dim=3, rot_dim=2, vdim=2, kv_rank=5, scale=0.7, rot={"base": 100.0, "dims": 2})
    h = torch.randn(T, W)
    w = {"m.q": torch.randn(10, W), "m.dkv": torch.randn(7, W), "m.dkv.norm": torch.rand(5) + 0.5, "m.uk": torch.randn(6, 5),
         "m.uv": torch.randn(4, 5), "m.g": torch.randn(2, W), "m.o": torch.eye(4)}
    c, kr = plain.latents(h, w, "m.", m, 1e-6)
    y = plain.latent_mixer(h, w, "m.", m, c, kr)
    raw = h @ w["m.dkv"].T
    torch.testing.assert_close(c, raw[:, :5] / torch.sqrt(raw[:, :5].pow(2).mean(1, keepdim=True) + 1e-6) * w["m.dkv.norm"])
    for t in range(T):
        ang = torch.tensor(float(t))
        u, v = raw[t, 5], raw[t, 6]
        torch.testing.assert_close(kr[t], torch.stack([u * ang.cos() - v * ang.sin(), v * ang.cos() + u * ang.sin()]))
    t, i = 3, 1
    q = (h[t] @ w["m.q"].T).view(2, 5)[i]
    ang = torch.tensor(float(t))
    qr = torch.stack([q[3] * ang.cos() - q[4] * ang.sin(), q[4] * ang.cos() + q[3] * ang.sin()])
    s = torch.stack([(q[:3] @ (w["m.uk"].view(2, 3, 5)[i] @ c[j]) + qr @ kr[j]) * 0.7 for j in range(t + 1)])
    o = (torch.softmax(s, 0)[:, None] * torch.stack([w["m.uv"].view(2, 2, 5)[i] @ c[j] for j in range(t + 1)])).sum(0)
    torch.testing.assert_close(y[t, 2:], o * torch.sigmoid(h[t] @ w["m.g"][1]), atol=1e-5, rtol=1e-5)


def test_the_score_weighs_an_experts_input():
    torch.manual_seed(1)
    h = torch.randn(3, 4)
    w = {f"f.e{e}.{n}": torch.randn(*s) for e in range(4) for n, s in (("gate", (5, 4)), ("up", (5, 4)), ("down", (4, 5)))}
    w["f.router"] = torch.randn(4, 4)
    got = plain.routed_ff(h, w, "f.", {"router": {"experts": 4, "top": 2}})
    for t in range(3):
        s = [sig(float(h[t] @ w["f.router"][e])) for e in range(4)]
        best = sorted(range(4), key=lambda e: -s[e])[:2]
        want = sum(plain.gated_ff(s[e] * h[t:t + 1], w, f"f.e{e}.")[0] for e in best)
        torch.testing.assert_close(got[t], want, atol=1e-5, rtol=1e-5)


def test_the_plain_model_runs_and_its_layers_matter():
    d = PRESETS["balalorn-tiny"]
    spec = registry.build_spec(registry.config_from_dict(d))
    w = {k: v.float() * (40.0 if k == "embed" else 3.0 if v.dim() == 2 else 1.0) for k, v in random_tensors(spec, 1).items()}
    toks = [5, 9, 200, 31, 7, 7, 100, 2] * 6
    layers = []
    logits = plain.forward(d, w, toks, layers_out=layers)
    assert logits.shape == (48, 304) and len(layers) == 4 and bool(torch.isfinite(logits).all())
    other = plain.forward(d, w, [6] + toks[1:])
    assert float((logits[-1] - other[-1]).abs().max()) > 1e-6         # memories and latents carry the first token on
    assert len(plain.greedy(d, w, toks[:5], 3)) == 3
