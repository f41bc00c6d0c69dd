"""Balalorn on the GPU: each mechanism's kernels alone against the plain functions, then whole
models (other sizes in every test than anywhere else) through the engine's runner, cache and
state slots: whole prompts, the stream after every layer, token-by-token decoding, portions down
to two tokens, unequal requests in one batch, pages and slots that come back, a marked key far
away among hundreds (also through another layer's latents), memories that carry a token for
hundreds of steps, models drawn at random, and greedy generation through the engine and its
scheduler."""

from __future__ import annotations

import math
import os
import random

import numpy as np
import pytest
import torch
from safetensors.torch import load_file, save_file

import kvforge_amd
from kvforge_amd.config.presets import balalorn as make_config
from kvforge_amd.engine.batch import StepEntry
from tests import replay_util as ru
from tests.plain import balalorn as plain
from tests.test_fogorax_gpu import in_portions, make_runner, prompts_for, replay, replay_all
from tests.test_kernels_gpu import Paged, prefill_work
from tests.test_rudorax_gpu import close_to_truth, jittered

pytestmark = pytest.mark.gpu
DEV = "cuda"
DTYPES = [torch.float32, torch.bfloat16]
NAME = {torch.float32: "float32", torch.bfloat16: "bfloat16"}


def ops():
    from kvforge_amd.kernels import ops as o
    return o


def tol(dtype):
    return dict(atol=3e-5, rtol=3e-5) if dtype == torch.float32 else dict(atol=2e-2, rtol=2e-2)


def rand(*shape, seed=0, scale=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed)) * scale


def i32(values):
    return torch.tensor(values, dtype=torch.int32, device=DEV)


# ======================================================================= mechanisms alone
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("taps", range(1, 9))
@pytest.mark.parametrize("G,dk,other,bias", [(0, 0, 70, True), (2, 24, 300, False), (5, 100, 9, False), (1, 256, 0, True),
                                             (3, 7, 16, False)])
def test_convolution_over_runs_steps_and_slots(dtype, taps, G, dk, other, bias):
    """Runs of every length around the taps and the kernel's tile, each continued from what the
    step before left in its slot (single tokens, runs shorter than the taps); a slot that held
    another's inputs starts from zeros at position 0; a sequence without a slot keeps nothing.
    The first channels are heads made unit vectors, the first half of them scaled."""
    unit, C = 2 * G * dk, 2 * G * dk + other
    lens = [1, 2, 16, 17, 40, 3]
    more = [5, 1, 2, 33, 1, 1]
    w, b = rand(C, taps, seed=taps, scale=0.6), rand(C, seed=2) if bias else None
    xs = [rand(n + m, C, seed=10 + i).to(dtype).float() for i, (n, m) in enumerate(zip(lens, more))]

    def want(x):
        y = plain.short_conv(x, w, b)
        if G:
            qk = plain.unit(y[:, :unit].reshape(-1, 2, G, dk))
            qk[:, 0] *= 0.3
            y = torch.cat([qk.reshape(-1, unit), y[:, unit:]], dim=1)
        return y

    wants = [want(x) for x in xs]
    off = 5
    state = torch.full((7, off + (taps - 1) * C + 2), 5.0, device=DEV)
    slots = [3, 0, 6, 2, 5, -1]

    def step(parts):
        rows = torch.cat([xs[s][a:e] for s, a, e in parts])
        wide = torch.cat([torch.full((len(rows), 3), 9.0), rows, torch.full((len(rows), 4), 9.0)], dim=1).to(dtype).to(DEV)
        out = torch.full((len(rows), C), 7.0, device=DEV)
        ops().ssm_conv(wide, 3, w.to(DEV), b.to(DEV) if bias else None, i32([0] + list(np.cumsum([e - a for _, a, e in parts]))),
                       i32([p for _, a, e in parts for p in range(a, e)]), i32([slots[s] for s, _, _ in parts]), state, off,
                       out, len(parts), max(e - a for _, a, e in parts), unit=unit, key_dim=dk, q_scale=0.3)
        return out.cpu()

    first = step([(s, 0, n) for s, n in enumerate(lens)])
    at = 0
    for s, n in enumerate(lens):
        torch.testing.assert_close(first[at:at + n], wants[s][:n], atol=2e-5, rtol=2e-5)
        at += n
    second = step([(s, lens[s], lens[s] + more[s]) for s in range(5)])       # the one without a slot does not go on
    at = 0
    for s in range(5):
        torch.testing.assert_close(second[at:at + more[s]], wants[s][lens[s]:], atol=2e-5, rtol=2e-5)
        at += more[s]
    assert float((state[1] - 5.0).abs().max()) == 0.0 and float((state[4] - 5.0).abs().max()) == 0.0
    assert float((state[:, :off] - 5.0).abs().max()) == 0.0 and float((state[:, -2:] - 5.0).abs().max()) == 0.0


def run_memory(delta, q, k, v, za, zb, neg_a, dt_bias, skip, runs, state, slots, positions, H, G, dk, dv):
    """The kernels over the runs of one step; rows of q, k, v in 32-bit."""
    o = ops()
    n = q.shape[0]
    rows = torch.cat([q, k, v, torch.full((n, 3), 9.0)], dim=1).to(DEV)
    gates = torch.cat([torch.full((n, 2), 9.0), za, zb], dim=1).to(DEV)
    chunks, rr = o.ssm_plan(runs, dk)
    multi = None
    if chunks:
        multi = {"chunks": i32(chunks).view(-1, 4), "runs": i32(rr).view(-1, 3)}
        for name, (shape, dt) in o.ssm_scratch(n, len(chunks) // 4, H, dk, dv, delta).items():
            multi[name] = torch.full(shape, 7.0, dtype=dt, device=DEV)
    out = torch.full((n, H * dv), 7.0, device=DEV)
    o.ssm_scan(rows, 0, G * dk, 2 * G * dk, gates, 2, 2 + H if delta else None, neg_a.to(DEV), dt_bias.to(DEV),
               skip.to(DEV) if skip is not None else None, i32([0] + list(np.cumsum(runs))), i32(positions), i32(slots),
               state, out, len(runs), H, G, dk, dv, multi=multi, short_runs=any(r < o.SSM_CHUNK_FROM for r in runs))
    return out.cpu()


@pytest.mark.parametrize("delta", [True, False])
@pytest.mark.parametrize("H,G,dk,dv", [(2, 1, 16, 16), (6, 3, 24, 40), (2, 2, 64, 130), (3, 1, 100, 72), (2, 1, 256, 64),
                                       (4, 2, 8, 200), (2, 1, 128, 128), (1, 1, 1, 1), (2, 1, 33, 65)])
def test_the_memory_over_runs_steps_and_slots(delta, H, G, dk, dv):
    """Sequences of every kind in one step: a few tokens (token by token), lengths on both sides of
    the chunks' first and of their edges, a single token; then each goes on from its slot the
    other way.  Log decays from all but nothing to gates that close; a slot that held another's
    memory starts from zeros at position 0; a sequence without a slot keeps nothing."""
    lens = [9, 150, 1, 64, 23, 24, 65]
    more = [70, 3, 20, 1, 64, 63, 40]
    g = torch.Generator().manual_seed(dk + dv)
    neg_a = -torch.exp(torch.randn(H, generator=g))
    dt_bias = torch.randn(H, generator=g)
    skip = None if delta else torch.randn(H, generator=g)
    seqs = []
    for n in (a + b for a, b in zip(lens, more)):
        q, k = torch.randn(n, G, dk, generator=g), torch.randn(n, G, dk, generator=g)
        if delta:
            q, k = plain.unit(q), plain.unit(k)
        else:
            q, k = q * dk ** -0.5, k * dk ** -0.5
        v = torch.randn(n, H, dv, generator=g)
        za, zb = torch.randn(n, H, generator=g) * 2.0 - 2.0, torch.randn(n, H, generator=g) * 2.0
        za[torch.rand(n, H, generator=g) < 0.03] = 40.0                        # a gate that closes
        seqs.append((q, k, v, za, zb))

    def truth(q, k, v, za, zb):
        q, k, v, za, zb = (t.double() for t in (q, k, v, za, zb))
        dt = plain.softplus(za + dt_bias)
        a = torch.exp(neg_a * dt)
        if delta:
            return plain.delta_scan(q, k, v, a, torch.sigmoid(zb)).float()
        return (plain.ssd_scan(q, k, v, a, dt) + skip[:, None] * v).float()

    want = [truth(*s) for s in seqs]
    size = max(float(w.abs().max()) for w in want)
    close = dict(atol=2e-5 * size, rtol=2e-4)
    state = torch.full((9, H * dk * dv + 3), 5.0, device=DEV)          # leftovers of others in every slot
    slots = [2, 0, 3, 8, 5, 6, 1]

    def step(parts):
        cat = lambda i: torch.cat([seqs[s][i][a:b].reshape(b - a, -1) for s, a, b in parts])  # noqa: E731
        pos = [p for _, lo, hi in parts for p in range(lo, hi)]
        return run_memory(delta, cat(0), cat(1), cat(2), cat(3), cat(4), neg_a, dt_bias, skip,
                          [hi - lo for _, lo, hi in parts], state, [slots[s] for s, _, _ in parts], pos, H, G, dk, dv)

    def compare(got, parts):
        at = 0
        for s, lo, hi in parts:
            torch.testing.assert_close(got[at:at + hi - lo].view(-1, H, dv), want[s][lo:hi], **close,
                                       msg=lambda m: f"sequence {s}, tokens {lo} to {hi}: {m}")
            at += hi - lo

    first = [(s, 0, n) for s, n in enumerate(lens)]
    compare(step(first), first)
    second = [(s, n, n + m) for s, (n, m) in enumerate(zip(lens, more))]
    compare(step(second), second)
    # token by token from the middle of a long one's memory
    again = [(1, 0, 148)]
    compare(step(again), again)
    for t in range(148, 153):
        compare(step([(1, t, t + 1)]), [(1, t, t + 1)])
    # without a slot
    slots[0] = -1
    before = state.clone()
    alone = [(0, 0, 70)]
    compare(step(alone), alone)
    assert torch.equal(before, state) and float((state[:, -3:] - 5.0).abs().max()) == 0.0


def test_writes_that_repeat_a_key_replace_what_it_answers():
    """With beta near one and no decay, the delta rule's memory answers a key with the last value
    written under it, however often it was overwritten, also across chunks."""
    H, dk, dv, n = 1, 16, 16, 130
    which = [i % 4 for i in range(n)]
    keys = torch.linalg.qr(rand(dk, dk, seed=2))[0][:4]       # four orthogonal unit vectors
    kk = torch.stack([keys[i] for i in which])
    v = rand(n, dv, seed=3)
    za, zb = torch.full((n, H), -60.0), torch.full((n, H), 40.0)
    q = torch.stack([keys[(i + 1) % 4] for i in which])       # asks for the key written three tokens ago
    state = torch.zeros(1, dk * dv, device=DEV)
    got = run_memory(True, q, kk, v, za, zb, torch.tensor([-1.0]), torch.zeros(1), None, [n], state, [0], list(range(n)),
                     H, 1, dk, dv)
    torch.testing.assert_close(got[3:], v[:-3], atol=1e-4, rtol=1e-4)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("inner,parts", [(24, 1), (120, 4), (96, 96), (2048, 2), (5000, 1)])
def test_gate_and_norm_in_parts(dtype, inner, parts):
    y, z = rand(5, inner, seed=1, scale=3.0), rand(5, inner + 8, seed=2, scale=2.0).to(dtype)
    y[2] = 0.0
    w = 1.0 + rand(inner, seed=3, scale=0.3)
    out = torch.zeros(5, inner, dtype=dtype, device=DEV)
    ops().ssm_gate_norm(y.to(DEV), z.to(DEV)[:, 8:], w.to(DEV), 1e-3, parts, out)
    u = y * plain.silu(z.float()[:, 8:])
    want = plain.rms(u.view(5, parts, inner // parts), 1e-3).reshape(5, inner) * w
    torch.testing.assert_close(out.float().cpu(), want, **tol(dtype))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("h", [1, 30, 88, 1024, 2052, 4096, 5000])
def test_a_normed_row_joins_the_stream_and_the_sum_is_copied(dtype, h):
    x, y, w = rand(3, h, seed=1, scale=4.0), rand(3, h, seed=2, scale=0.1), 1.0 + rand(h, seed=3, scale=0.3)
    dx, out = x.clone().to(DEV), torch.zeros(3, h, dtype=dtype, device=DEV)
    ops().rms_add_cast(dx, y.to(DEV), w.to(DEV), 1e-4, out)
    want = x + plain.norm(y, w, 1e-4)
    torch.testing.assert_close(dx.cpu(), want, atol=2e-5, rtol=2e-5)
    assert torch.equal(out.cpu(), dx.cpu().to(dtype))


@pytest.mark.parametrize("R,top", [(1, 1), (8, 1), (8, 3), (70, 16), (512, 5)])
def test_router_scores_by_sigmoid(R, top):
    z = rand(9, R + 3, seed=R, scale=3.0).to(DEV)
    chosen = torch.full((9, top), -5, dtype=torch.int32, device=DEV)
    weights = torch.full((9, top), -5.0, device=DEV)
    for renormalize in (False, True):
        ops().moe_topk(z[:, :R], None, chosen, weights, "sigmoid", renormalize)
        s = torch.sigmoid(z[:, :R].float().cpu())
        v, i = torch.topk(s, top)
        assert torch.equal(chosen.cpu().long(), i)
        torch.testing.assert_close(weights.cpu(), v / v.sum(1, keepdim=True) if renormalize else v, atol=1e-6, rtol=1e-5)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("E,top,ff,width,n", [(5, 2, 32, 64, 7), (4, 1, 24, 40, 40), (8, 3, 64, 104, 400), (3, 3, 16, 30, 5)])
@pytest.mark.parametrize("fresh", [True, False])
def test_experts_whose_inputs_are_weighed(dtype, E, top, ff, width, n, fresh):
    """The layer alone, on the grouped kernels and on the products over all experts, added to rows
    that hold something and written to fresh ones."""
    from kvforge_amd.engine.batch import Step, Workspace
    from kvforge_amd.parts import RoutedExperts

    part = RoutedExperts("f", width, ff, E, top, scores="sigmoid", renormalize=False, correct=False, weigh_input=True)
    w = {k: rand(*v.shape, seed=i, scale=0.3).to(dtype) for i, (k, v) in enumerate(sorted(part.weight_specs().items()))}
    # scores that no rounding reorders: the rows' first elements name them
    x = rand(n, width, seed=40)
    levels = torch.linspace(-2.0, 2.0, E)
    g = torch.Generator().manual_seed(3)
    for t in range(n):
        x[t, :E] = levels[torch.randperm(E, generator=g)]
    w["f.router"] = torch.eye(E, width).to(dtype)
    x = x.to(dtype)
    part.load({k: v.to(DEV) for k, v in w.items()})
    part.seal()
    step = Step()
    step.ws, step.act_dtype, step.n_tokens = Workspace(DEV), dtype, n
    rows = rand(n, width, seed=50).to(DEV)
    base = torch.zeros(n, width) if fresh else rows.cpu().clone()
    if fresh:
        step.fresh = rows
    part.forward(x.to(DEV), step, rows)
    step.settle()
    assert step.fresh is None
    want = base + plain.routed_ff(x.float(), {k: v.float() for k, v in w.items()}, "f.", {"router": {"experts": E, "top": top}})
    spread = float((want - base).std())       # the outputs' own size: a bf16 engine rounds activations and outputs
    torch.testing.assert_close(rows.cpu(), want, rtol=1e-4,
                               atol=(1e-5 if dtype == torch.float32 else 3e-2) * spread)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,O,I,n", [(1, 16, 8, 3), (5, 28, 44, 70), (4, 64, 192, 300), (3, 12, 30, 9), (2, 64, 512, 300)])
def test_a_gate_per_head_where_the_values_are_read_out(dtype, H, O, I, n):
    x, w, g = rand(n, H * I, seed=1).to(dtype), rand(H, O, I, seed=2, scale=I ** -0.5).to(dtype), rand(n, H + 4, seed=3, scale=2.0).to(dtype)
    out = torch.zeros(n, H * O, dtype=dtype, device=DEV)
    ops().head_product(x.to(DEV), I, w.to(DEV), out, O, gate=g.to(DEV)[:, 4:])
    want = torch.einsum("nhi,hoi->nho", x.float().view(n, H, I), w.float()) * torch.sigmoid(g.float()[:, 4:])[:, :, None]
    torch.testing.assert_close(out.float().cpu(), want.reshape(n, H * O), **tol(dtype))


@pytest.mark.parametrize("dtype", DTYPES)
def test_queries_alone_for_another_layers_keys(dtype):
    n, H, dim, rot, rank, d = 4, 3, 10, 6, 20, 32
    proj = rand(n, H * (dim + rot) + 5, seed=1).to(dtype).to(DEV)
    qkv = torch.full((n, H * d), 9.0, dtype=dtype, device=DEV)
    ops().latent_split(proj, qkv, None, 1e-5, H, dim, rot, rank, d)
    q = qkv.view(n, H, d)
    assert torch.equal(q[:, :, :rot], proj[:, :H * (dim + rot)].view(n, H, dim + rot)[:, :, dim:])
    assert float((q[:, :, rot:rot + rank].float() - 9.0).abs().max()) == 0.0 and float(q[:, :, rot + rank:].abs().max()) == 0.0


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,KV,d,bs", [(4, 1, 272, 16), (11, 1, 576, 16), (2, 2, 640, 6)])
def test_attention_over_heads_of_more_than_256_elements(dtype, H, KV, d, bs):
    """Query runs and single tokens, one cut of the key range and several."""
    scale = 1 / math.sqrt(d)
    for seq_lens, q_lens in (([90, 33, 70, 5], [40, 33, 2, 5]), ([7, 90, 1, 300], [1, 1, 1, 1])):
        paged = Paged(seq_lens, KV, d, bs, dtype, seed=d)
        n = sum(q_lens)
        buf = rand(n, H * d, seed=d + 1, scale=1.5).to(dtype)
        cu, ctx = i32([0] + list(np.cumsum(q_lens))), i32(seq_lens)
        want, off = [], 0
        for s, (m, ql) in enumerate(zip(seq_lens, q_lens)):
            k, v = (t[s].float().repeat_interleave(H // KV, dim=1) for t in (paged.keys, paged.values))
            sc = torch.einsum("qhd,khd->hqk", buf[off:off + ql].float().view(ql, H, d), k) * scale
            sc = sc.masked_fill(torch.arange(m)[None, None, :] > torch.arange(m - ql, m)[None, :, None], float("-inf"))
            want.append(torch.einsum("hqk,khd->qhd", torch.softmax(sc, -1), v).reshape(ql, H * d))
            off += ql
        want = torch.cat(want)
        args = (buf.to(DEV), paged.k.to(DEV), paged.v.to(DEV), paged.table.to(DEV))
        if max(q_lens) > 1:
            out = torch.zeros(n, H * d, dtype=dtype, device=DEV)
            ops().attn_prefill(*args, cu, ctx, prefill_work(q_lens, H // KV, dtype, d, bs).to(DEV), out, H, KV, d, scale)
            torch.testing.assert_close(out.float().cpu(), want, **tol(dtype))
            continue
        for splits in (1, 3):
            out = torch.zeros(n, H * d, dtype=dtype, device=DEV)
            ws = (torch.empty(n * H * splits * d, device=DEV), torch.empty(n * H * splits * 2, device=DEV))
            ops().attn_decode(*args, None, n, cu, ctx, out, H, KV, d, scale, 0, splits, ws)
            torch.testing.assert_close(out.float().cpu(), want, **tol(dtype))


# ======================================================================= whole models
def shape_a():
    """All mixers and both feed-forwards, latents used by a later layer; sizes that no kernel's
    tiles divide."""
    return make_config(vocab=203, width=88, layers=[
        ("mamba2", dict(heads=6, vdim=20, state=24, groups=3, norm_groups=4, conv=3), (24, 7, 2)),
        ("latent_attention", dict(heads=5, dim=20, rot_dim=12, vdim=28, kv_rank=44, scale=0.21, base=3000.0), 104),
        ("delta", dict(heads=6, kv_heads=2, dim=28, vdim=36, conv=5), None),
        ("latent_attention", dict(heads=3, dim=8, rot_dim=12, vdim=12, kv_rank=44, scale=0.3, base=3000.0, kv_from=1),
         (40, 3, 3))], eps=1e-5, max_positions=2048)


def shape_b():
    """What a model may make equal or one: one head everywhere, as many q/k heads as memories, one
    group, one part, one tap, one expert of one, no plain query part, two layers over one layer's
    latents and latents of their own again."""
    lat = dict(heads=1, dim=16, rot_dim=16, vdim=16, kv_rank=16, scale=1.0, base=100.0)
    return make_config(vocab=64, width=32, layers=[
        ("latent_attention", lat, None),
        ("delta", dict(heads=1, kv_heads=1, dim=16, vdim=16, conv=1), (16, 1, 1)),
        ("latent_attention", dict(lat, kv_from=0), 32),
        ("mamba2", dict(heads=1, vdim=32, state=16, groups=1, norm_groups=1, conv=1), None),
        ("latent_attention", dict(lat, dim=0, kv_from=0), None),
        ("delta", dict(heads=2, kv_heads=2, dim=16, vdim=16, conv=2), (16, 3, 3)),
        ("latent_attention", dict(lat, rot_dim=2, scale=0.5), 16)], eps=1e-6, max_positions=512)


def shape_c():
    """Layers wide enough for the kernels that serving a real model takes: latents on the matrix
    cores, memories wider than a wave's rows, experts on the grouped kernels, a feed-forward deep
    enough for a down projection cut in two halves of K elsewhere, a vocabulary that ends inside
    a group of 16 columns."""
    lat = dict(heads=6, dim=64, rot_dim=32, vdim=64, kv_rank=128, scale=0.1, base=100000.0)
    return make_config(vocab=1000, width=384, layers=[
        ("delta", dict(heads=4, kv_heads=2, dim=128, vdim=128, conv=4), 4096),
        ("latent_attention", lat, (128, 8, 2)),
        ("mamba2", dict(heads=8, vdim=64, state=128, groups=2, norm_groups=2, conv=4), (64, 8, 1)),
        ("latent_attention", dict(lat, kv_from=1), 512)], eps=1e-5, max_positions=2048)


def shape_d():
    """A latent row beyond the matrix-core kernels' heads, memories of 256-element keys."""
    lat = dict(heads=3, dim=32, rot_dim=24, vdim=40, kv_rank=300, scale=0.15, base=5000.0)
    return make_config(vocab=150, width=64, layers=[
        ("latent_attention", lat, (32, 4, 2)), ("delta", dict(heads=2, kv_heads=1, dim=256, vdim=24, conv=8), 48),
        ("mamba2", dict(heads=3, vdim=16, state=200, groups=1, norm_groups=3, conv=4), None),
        ("latent_attention", dict(lat, heads=9, kv_from=0), None)], eps=1e-4, max_positions=512)


SHAPE = {"a": shape_a, "b": shape_b, "c": shape_c, "d": shape_d}


def liven(folder: str, cfg: dict, seed: int = 0) -> None:
    """Random weights of std 0.02 give flat attention, closed convolutions and memories that hardly
    turn.  Scaled so that attention is peaked, gates swing and the first layers have something to
    read.  The routers read a few coordinates of the stream that the embedding alone fills (the
    norms' weights are zero there) with levels evenly spaced and shuffled per token, so that every
    token has its own experts and scores and no rounding can reorder them."""
    path = os.path.join(folder, "model.safetensors")
    w = load_file(path)
    routed = [l["mlp"]["router"]["experts"] for l in cfg["layers"] if l["mlp"] and l["mlp"]["kind"] == "moe"]
    E = max(routed, default=0)
    g = torch.Generator().manual_seed(seed)
    for k in list(w):
        f = 1.0
        if k == "embed":
            f = 40.0
        elif k.endswith((".q", ".dkv")):
            f = 6.0
        elif k.endswith((".uk", ".uv", ".g", ".in", ".k", ".v", ".a", ".b")) and ".mix" in k:
            f = 8.0
        elif k.endswith((".o", ".down", ".up", ".gate")):
            f = 4.0
        elif k == "head":
            f = 3.0
        if f != 1.0:
            w[k] = (w[k].float() * f).to(w[k].dtype)
    if E:
        for k in list(w):
            if k.endswith((".norm1", ".norm2")):
                w[k][:E] = 0.0
        levels = torch.linspace(-2.0, 2.0, E) if E > 1 else torch.zeros(1)
        for t in range(w["embed"].shape[0]):
            w["embed"][t, :E] = levels[torch.randperm(E, generator=g)].to(w["embed"].dtype)
        for i, layer in enumerate(cfg["layers"]):
            if layer["mlp"] and layer["mlp"]["kind"] == "moe":
                r = w[f"l{i}.mlp.router"]
                r[:] = torch.eye(*r.shape).to(r.dtype)[torch.randperm(r.shape[0], generator=g)]
    save_file(w, path, metadata={"format": "pt"})


_MODELS: dict = {}


def model_folder(tmp_path_factory, name: str, dtype):
    key = (name, dtype)
    if key not in _MODELS:
        folder = str(tmp_path_factory.mktemp(f"balalorn_{name}_{NAME[dtype]}"))
        cfg = SHAPE[name]()
        kvforge_amd.write_random_model(folder, cfg, seed=len(name) + 19, dtype=NAME[dtype])
        liven(folder, cfg)
        _MODELS[key] = (folder, cfg, load_file(os.path.join(folder, "model.safetensors")))
    return _MODELS[key]


_WANT: dict = {}


def plain_logits(cfg, w, toks, dtype):
    """(the truth, plain runs with the roundings of ``dtype``): the plain model in 64-bit, and in
    32-bit (for a 32-bit engine) or in 32-bit with every trip through memory that a bfloat16
    engine may make rounded to bfloat16: as the weights are, and twice with them moved by half a
    bfloat16 step, which shows the rows where the design multiplies rounding (a memory head is
    divided by its own size, so a head whose query all but misses its memory is rounding through
    and through)."""
    key = (id(w), tuple(toks), dtype)
    if key not in _WANT:
        truth = plain.forward(cfg, w, toks, dtype=torch.float64).float()
        if dtype == torch.bfloat16:
            runs = [plain.forward(cfg, w, toks, store=torch.bfloat16)]
            runs += [plain.forward(cfg, jittered(w, s), toks, store=torch.bfloat16) for s in range(1, 3)]
        else:
            runs = [plain.forward(cfg, w, toks)]
        _WANT[key] = (truth, runs)
    return _WANT[key]


def check(got, cfg, w, toks, dtype, what=""):
    truth, plain_runs = plain_logits(cfg, w, toks, dtype)
    close_to_truth(got, truth, plain_runs, dtype, what)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(SHAPE))
def test_whole_prompts_and_their_first_tokens(tmp_path_factory, name, dtype):
    folder, cfg, w = model_folder(tmp_path_factory, name, dtype)
    runner = make_runner(folder, dtype)
    seqs = prompts_for(cfg, [1, 2, 3, 70, 150], 1)
    got = replay(runner, seqs, [[(r, 0, len(t))] for r, t in seqs.items()])
    for r, t in seqs.items():
        check(got[r], cfg, w, t, dtype, f"{name} {r}")
    assert runner.cache.num_free_blocks == 64 and runner.cache.slots.num_free == 4


@pytest.mark.parametrize("name", sorted(SHAPE))
def test_the_stream_after_every_layer(tmp_path_factory, name):
    """In 32-bit, so that a fault names its layer."""
    folder, cfg, w = model_folder(tmp_path_factory, name, torch.float32)
    runner = make_runner(folder, torch.float32)
    toks = prompts_for(cfg, [60], 2)["r0"]
    want, truth = [], []
    plain.forward(cfg, w, toks, layers_out=want)
    plain.forward(cfg, w, toks, dtype=torch.float64, layers_out=truth)
    runner.cache.allocate("x", 0)
    runner.cache.append_slots("x", len(toks), 0)
    step, _ = runner.build_step([StepEntry("x", toks, 0, "all")])
    model = runner.model
    assert len(model.order) == len(want) == len(cfg["layers"])
    with torch.inference_mode():
        residual = model.embed(step)
        for i, (call, ls) in enumerate(zip(model.order, model.layer_states)):
            model.spec.blocks[call.layer].forward(residual, step, ls)
            step.settle()
            own = float((want[i].double() - truth[i]).abs().max())
            torch.testing.assert_close(residual.cpu().double(), truth[i], atol=max(3e-4, 8.0 * own), rtol=3e-4,
                                       msg=lambda m: f"layer {i} ({cfg['layers'][i]['type']}): {m}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(SHAPE))
def test_decoding_token_by_token_equals_the_prompt_read_at_once(tmp_path_factory, name, dtype):
    """From the first token on, and from a prompt's end for 119 tokens."""
    folder, cfg, w = model_folder(tmp_path_factory, name, dtype)
    runner = make_runner(folder, dtype)
    seqs = prompts_for(cfg, [90, 160], 3)
    plan = [[("r0", i, i + 1)] for i in range(90)]
    plan += [[("r1", 0, 41)]] + [[("r1", i, i + 1)] for i in range(41, 160)]
    got = replay(runner, seqs, plan)
    for r, t in seqs.items():
        check(got[r], cfg, w, t, dtype, f"{name} {r}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(SHAPE))
@pytest.mark.parametrize("sizes", [(2,), (7, 2, 5, 3, 2, 11), (13, 1, 8, 40, 3), (64, 9), (23, 24, 25)])
def test_prompts_in_portions(tmp_path_factory, name, dtype, sizes):
    folder, cfg, w = model_folder(tmp_path_factory, name, dtype)
    runner = make_runner(folder, dtype)
    seqs = prompts_for(cfg, [101], 4)
    got = replay(runner, seqs, in_portions("r0", 101, sizes))
    check(got["r0"], cfg, w, seqs["r0"], dtype, f"{name} {sizes}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(SHAPE))
def test_unequal_requests_in_one_batch_against_each_alone(tmp_path_factory, name, dtype):
    """Portions of some requests beside single tokens of others; four slots and so few pages
    that both are used again by later requests; a request left out of a step goes on later."""
    folder, cfg, w = model_folder(tmp_path_factory, name, dtype)
    seqs = prompts_for(cfg, [83, 40, 7, 120, 33, 58], 5)
    plan = [
        [("r0", 0, 30), ("r1", 0, 1)],
        [("r0", 30, 31), ("r1", 1, 40), ("r2", 0, 2)],
        [("r2", 2, 7), ("r0", 31, 64), ("r3", 0, 50)],
        [("r3", 50, 51), ("r4", 0, 9)],                        # r0 is left out here
        [("r0", 64, 83), ("r3", 51, 52), ("r4", 9, 10), ("r5", 0, 16)],
        [("r3", 52, 118), ("r4", 10, 33), ("r5", 16, 17)],
        [("r3", 118, 119), ("r5", 17, 58)],
        [("r3", 119, 120)],
    ]
    runner = make_runner(folder, dtype, block_size=8, num_blocks=29, seqs=4)     # 118 + 33 + 58 tokens at the most
    together = replay(runner, seqs, plan)
    assert runner.cache.num_free_blocks == 29 and runner.cache.slots.num_free == 4
    for r, t in seqs.items():
        check(together[r], cfg, w, t, dtype, f"{name} {r} in the batch")
        alone = replay(runner, {r: t}, [[(r, 0, len(t))]])[r]
        check(alone, cfg, w, t, dtype, f"{name} {r} alone")
        truth, plain_runs = plain_logits(cfg, w, t, dtype)
        close_to_truth(together[r], alone, [p + (alone - truth) for p in plain_runs], dtype,
                       f"{name} {r} against itself alone")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["a", "c"])
def test_a_prompt_of_a_thousand_tokens(tmp_path_factory, name, dtype):
    """More than a dozen chunks of the memories, latents over many pages: whole, in large and
    small portions, and its last tokens one by one."""
    folder, cfg, w = model_folder(tmp_path_factory, name, dtype)
    runner = make_runner(folder, dtype, block_size=16, num_blocks=80, tokens=1200)
    toks = prompts_for(cfg, [1100], 11)["r0"]
    for plan in ([[("r0", 0, 1100)]], in_portions("r0", 1100, (300, 64, 65, 7, 129, 2)),
                 [[("r0", 0, 1050)]] + [[("r0", i, i + 1)] for i in range(1050, 1100)]):
        got = replay(runner, {"r0": toks}, plan)["r0"]
        check(got, cfg, w, toks, dtype, f"{name}, {len(plan)} steps")


def marked_model(tmp_path, dtype, shared: bool):
    """A model in which token 1 is marked: its embedding lies along one axis that no other token
    uses, element 0 of its latent is all there is of it, every query has a constant that meets
    that element, the values carry it on.  So the marked token scores far above all others for
    every query.  ``shared``: the layer that looks is the second one and uses the first one's
    latents; the first one's own head is closed by its gate."""
    V, W, rank, H = 50, 32, 24, 2
    lat = dict(heads=H, dim=16, rot_dim=8, vdim=16, kv_rank=rank, scale=1.0, base=1000.0)
    layers = [("latent_attention", lat, None)]
    if shared:
        layers.append(("latent_attention", dict(lat, kv_from=0), None))
    cfg = make_config(vocab=V, width=W, layers=layers, eps=1e-6, max_positions=2048)
    folder = str(tmp_path / f"m_{shared}")
    kvforge_amd.write_random_model(folder, cfg, seed=5, dtype=NAME[dtype])
    path = os.path.join(folder, "model.safetensors")
    w = load_file(path)
    e = rand(V, W, seed=1, scale=0.3)
    e[:, 0] = 0.0
    e[:, 1] = 1.0                       # a constant every token has: the queries' handle
    e[1] = 0.0
    e[1, 0] = 6.0
    dkv = rand(rank + 8, W, seed=2, scale=0.3)
    dkv[:, 0] = 0.0
    dkv[0] = 0.0
    dkv[0, 0] = 1.0                     # only the marked token has this element, and nothing else
    look = 1 if shared else 0
    wq = torch.zeros(H * 24, W)
    wq[0, 1] = wq[24, 1] = 3.0
    uk = rand(H * 16, rank, seed=3, scale=0.1)
    uk[0] = uk[16] = 0.0
    uk[0, 0] = uk[16, 0] = 1.0
    uv = rand(H * 16, rank, seed=4, scale=0.1)
    uv[:, 0] = rand(H * 16, seed=5, scale=1.5)
    # the stream's first two axes stay what the embedding made them
    new = {"embed": e, "l0.mix.dkv": dkv, "l0.mix.dkv.norm": torch.ones(rank), f"l{look}.mix.q": wq,
           f"l{look}.mix.uk": uk, f"l{look}.mix.uv": uv, f"l{look}.mix.g": rand(H, W, seed=6, scale=0.1),
           f"l{look}.mix.o": rand(W, H * 16, seed=7, scale=0.5)}
    if shared:
        shut = torch.zeros(H, W)
        shut[:, 1] = -60.0
        shut[:, 0] = -10.0
        new["l0.mix.g"] = shut
    for k, t in new.items():
        assert w[k].shape == t.shape, k
        w[k] = t.to(w[k].dtype)
    for k in w:
        if k.endswith(".norm1"):
            w[k][:2] = 0.0
    save_file(w, path, metadata={"format": "pt"})
    return folder, cfg, load_file(path)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shared", [False, True])
@pytest.mark.parametrize("bs", [8, 16])
def test_one_key_among_hundreds(tmp_path, dtype, shared, bs):
    """The logits follow the marked token from hundreds of tokens away, wherever it lies: first,
    in the middle of a page, a page's last and first, a portion's last; read whole, in portions
    and token by token."""
    folder, cfg, w = marked_model(tmp_path, dtype, shared)
    runner = make_runner(folder, dtype, block_size=bs, num_blocks=-(-700 // bs), tokens=640)
    g = torch.Generator().manual_seed(bs)
    for at in (0, 7, bs - 1, bs, 12 * bs - 1, 200):
        n = at + 320
        toks = torch.randint(2, 50, (n,), generator=g).tolist()
        toks[at] = 1
        want = plain.forward(cfg, w, toks)
        blind = plain.forward(cfg, w, [t if i != at else 2 for i, t in enumerate(toks)])
        assert float((want[-1] - blind[-1]).abs().max()) > 0.3 * float(want.std())      # seen from the end
        if at:
            assert float((want[at - 1] - blind[at - 1]).abs().max()) == 0.0
        for plan in ([[("x", 0, n)]], in_portions("x", n, (at + 1, 2, 31)),
                     [[("x", 0, n - 40)]] + [[("x", i, i + 1)] for i in range(n - 40, n)]):
            got = replay(runner, {"x": toks}, plan)["x"]
            check(got, cfg, w, toks, dtype, f"marked at {at}, pages of {bs}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["delta", "mamba2"])
def test_memory_carries_a_token_from_the_far_past(tmp_path, dtype, kind):
    """A model of memories that hardly fade and are hardly written to after the first tokens: what
    token 0 was still shows in the logits hundreds of tokens later, through portions and single
    tokens and through a slot that others have used."""
    mix = (dict(heads=2, kv_heads=1, dim=32, vdim=16, conv=4) if kind == "delta"
           else dict(heads=2, vdim=24, state=32, groups=1, norm_groups=1, conv=4))
    cfg = make_config(vocab=40, width=48, layers=[(kind, mix, None), (kind, mix, 24)], eps=1e-6, max_positions=512)
    folder = str(tmp_path / "m")
    kvforge_amd.write_random_model(folder, cfg, seed=6, dtype=NAME[dtype])
    liven(folder, cfg)
    path = os.path.join(folder, "model.safetensors")
    w = load_file(path)
    for k in list(w):
        if k.endswith(".A_log"):
            w[k] = torch.full_like(w[k], -9.0)
        elif k.endswith(".dt_bias"):
            w[k] = torch.full_like(w[k], -3.0)
        elif k.endswith(".b"):                             # beta small, except under token 0's embedding
            w[k] = (w[k].float() * 0.0).to(w[k].dtype)
            if not k.endswith("conv.b"):
                w[k][:, 0] = 2.0
        elif k == "embed":
            w[k][:, 0] = -3.0
            w[k][0, 0] = w[k][1, 0] = 3.0
        elif k.endswith((".norm1", ".norm2")):
            w[k][0] = 0.0
        elif k.endswith(".in"):
            w[k][-2:] = 0.0
            w[k][-2:, 0] = 1.5                             # the step size likewise
    save_file(w, path, metadata={"format": "pt"})
    w = load_file(path)
    runner = make_runner(folder, dtype, block_size=8, num_blocks=16, seqs=2, tokens=512)
    assert len(runner.model.state_specs) == 2
    toks = [0] + [t + 2 if t < 2 else t for t in prompts_for(cfg, [399], 7)["r0"]]
    other = [1] + toks[1:]
    a, b = plain.forward(cfg, w, toks), plain.forward(cfg, w, other)
    assert float((a[-1] - b[-1]).abs().max()) > 0.05 * float(a.std())     # the first token still matters
    plan = in_portions("x", 300, (64, 3, 2, 50)) + [[("x", i, i + 1)] for i in range(300, 400)]
    for seq in (toks, other):
        got = replay(runner, {"x": seq}, plan)["x"]
        check(got, cfg, w, seq, dtype, "far past")


def random_shape(seed: int) -> dict:
    """A model whose every size, count, constant and layer order is drawn."""
    rng = random.Random(seed)
    width = rng.choice([24, 40, 56, 64, 88, 104, 128])

    def mlp():
        kind = rng.choice(["none", "dense", "moe", "moe"])
        if kind == "none":
            return None
        if kind == "dense":
            return rng.choice([8, 24, 40, 64, 136])
        experts = rng.choice([1, 2, 3, 5, 8, 12])
        return (rng.choice([8, 16, 32, 40, 64]), experts, rng.randint(1, min(experts, 4)))

    layers, latent_at = [], []
    for i in range(rng.randint(2, 6)):
        kind = rng.choice(["mamba2", "delta", "latent_attention"])
        if kind == "mamba2":
            g = rng.choice([1, 2, 3])
            heads, vdim = g * rng.choice([1, 2, 4]), rng.choice([4, 8, 16, 24, 40, 70])
            parts = rng.choice([p for p in (1, 2, 3, 4, g) if heads * vdim % p == 0])
            m = dict(heads=heads, vdim=vdim, state=rng.choice([4, 16, 24, 40, 64, 96, 144]), groups=g, norm_groups=parts,
                     conv=rng.choice([1, 2, 3, 4, 6]))
        elif kind == "delta":
            kv = rng.choice([1, 2, 3])
            m = dict(heads=kv * rng.choice([1, 2, 3]), kv_heads=kv, dim=rng.choice([4, 16, 20, 32, 48, 64, 72, 136]),
                     vdim=rng.choice([8, 16, 24, 40, 64, 100]), conv=rng.choice([1, 2, 3, 4, 5, 8]))
        else:
            src = rng.choice(latent_at) if latent_at and rng.random() < 0.6 else None
            rank, rot = rng.choice([8, 16, 40, 96, 130]), rng.choice([2, 8, 12, 16, 32])
            base = rng.choice([100.0, 10000.0, 1000000.0])
            if src is not None:
                rank, rot, base = (layers[src][1][k] for k in ("kv_rank", "rot_dim", "base"))
            m = dict(heads=rng.choice([1, 2, 3, 5, 8]), dim=rng.choice([8, 16, 20, 32, 48]), rot_dim=rot,
                     vdim=rng.choice([8, 16, 20, 32, 48]), kv_rank=rank, scale=rng.choice([0.05, 0.125, 0.3]), base=base)
            if src is not None:
                m["kv_from"] = src
            else:
                latent_at.append(i)
        layers.append((kind, m, mlp()))
    return make_config(vocab=rng.choice([17, 64, 100, 257, 512]), width=width, layers=layers,
                       eps=rng.choice([1e-6, 1e-5, 1e-3, 0.1]), max_positions=256)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("seed", range(14))
def test_models_drawn_at_random(tmp_path, seed, dtype):
    """Whole, token by token, in portions and in a batch with pages and slots used again."""
    cfg = random_shape(seed)
    folder = str(tmp_path / "model")
    kvforge_amd.write_random_model(folder, cfg, seed=seed, dtype=NAME[dtype])
    liven(folder, cfg, seed)
    w = load_file(os.path.join(folder, "model.safetensors"))
    bs = [4, 8, 16, 24][seed % 4]
    seqs = prompts_for(cfg, [90, 41, 2, 64, 33], seed)
    runner = make_runner(folder, dtype, block_size=bs, num_blocks=-(-300 // bs), seqs=3)
    plan = ([[("r0", 0, 90)]] + [[("r1", i, i + 1)] for i in range(41)] + in_portions("r3", 64, (5, 2, 17, 3))
            + [[("r0", 0, 40), ("r2", 0, 1)], [("r2", 1, 2), ("r0", 40, 41), ("r4", 0, 20)],
               [("r0", 41, 90), ("r4", 20, 21), ("r1", 0, 30)], [("r4", 21, 33), ("r1", 30, 41)]])
    got = replay_all(runner, seqs, plan)
    for r, t in seqs.items():
        for k, logits in enumerate(got[r]):
            check(logits, cfg, w, t, dtype, f"seed {seed}, {r}, pass {k}: {cfg}")
    if runner.model.state_specs:
        assert runner.cache.slots.num_free == 3
    if runner.model.cache_groups:
        assert runner.cache.num_free_blocks == -(-300 // bs)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["a", "c"])
def test_greedy_generation_through_the_engine(tmp_path_factory, name, dtype):
    """The framework's own entry point and scheduler: prompts admitted in portions under a small
    token budget, decode steps replayed from captured graphs (the memories advance on the
    device), three slots for five requests."""
    folder, cfg, w = model_folder(tmp_path_factory, name, dtype)
    engine = kvforge_amd.InferenceEngine.from_folder(
        folder, kvforge_amd.EngineConfig(
            cache=kvforge_amd.CacheConfig(block_size=8, num_blocks=60), dtype=dtype,
            scheduler=kvforge_amd.SchedulerConfig(max_num_seqs=3, max_num_batched_tokens=24, max_model_len=256)))
    prompts = list(prompts_for(cfg, [30, 2, 11, 45, 1], 7).values())
    outs = engine.generate(prompts, kvforge_amd.SamplingParams(max_tokens=40, temperature=0.0, ignore_eos=True))
    margin = 1e-3 if dtype == torch.float32 else 0.25
    followed, missed = 0, []
    for p, o in zip(prompts, outs):
        assert len(o.output_token_ids) == 40
        logits = plain.forward(cfg, w, p + o.output_token_ids)
        for i, tok in enumerate(o.output_token_ids):
            row = logits[len(p) - 1 + i]
            if float(row.max() - row[tok]) > margin * float(row.std()):
                missed.append((len(p), i, tok))
        followed += o.output_token_ids != plain.greedy(cfg, w, p[-1:], 40)
    assert len(missed) <= (0 if dtype == torch.float32 else 6), missed
    assert followed >= 4          # what comes out depends on more than the last token
    assert engine.cache.slots.num_free == 3 and engine.cache.num_free_blocks == 60
    if engine.runner.use_graphs:
        assert engine.runner.num_graph_replays > 0


def test_a_request_that_loses_its_pages_and_slot_is_read_again_from_its_first_token(tmp_path_factory):
    """Three requests outgrow the pool: the scheduler takes one's pages and state slot away and
    feeds it again later, prompt and generated tokens, into a slot and pages that others have
    used; its memories and convolutions start from zeros again."""
    folder, cfg, w = model_folder(tmp_path_factory, "b", torch.float32)
    engine = kvforge_amd.InferenceEngine.from_folder(
        folder, kvforge_amd.EngineConfig(
            cache=kvforge_amd.CacheConfig(block_size=8, num_blocks=20, watermark=0.0), dtype=torch.float32,
            scheduler=kvforge_amd.SchedulerConfig(max_num_seqs=3, max_num_batched_tokens=32, max_model_len=128)))
    prompts = list(prompts_for(cfg, [30, 26, 33], 10).values())
    outs = engine.generate(prompts, kvforge_amd.SamplingParams(max_tokens=40, temperature=0.0, ignore_eos=True))
    assert engine.scheduler.num_preemptions > 0
    for p, o in zip(prompts, outs):
        assert len(o.output_token_ids) == 40
        logits = plain.forward(cfg, w, p + o.output_token_ids)
        for i, tok in enumerate(o.output_token_ids):
            row = logits[len(p) - 1 + i]
            assert float(row.max() - row[tok]) <= 1e-3 * float(row.std()), (i, tok)
    assert engine.cache.slots.num_free == 3 and engine.cache.num_free_blocks == 20


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_replay_in_a_process_of_its_own(tmp_path_factory, tmp_path, dtype):
    """``bin/trace_run`` as a user runs it: whole, token by token, in portions and mixed, with
    a pool of exactly the peak of live tokens and four state slots."""
    td = torch.float32 if dtype == "float32" else torch.bfloat16
    folder, cfg, w = model_folder(tmp_path_factory, "a", td)
    prompts = prompts_for(cfg, [37, 81, 100, 53], 8)
    tb = ru.TraceBuilder()
    for rid, toks in prompts.items():
        for mode, fn in (("w", ru.whole), ("d", ru.decode_tail), ("p", ru.portions)):
            fn(tb, f"{rid}#{mode}", toks)
    ru.mixed(tb, {f"{rid}#m": toks for rid, toks in prompts.items()}, 9)
    out = str(tmp_path / "out")
    ru.run_trace(folder, dtype, tb, out)
    want = {rid: plain_logits(cfg, w, toks, td) for rid, toks in prompts.items()}
    for sid, rows in enumerate(tb.expect):
        if not rows:
            continue
        got = torch.from_numpy(np.fromfile(os.path.join(out, f"{sid}.f32"), dtype="<f4").reshape(-1, cfg["vocab"]).copy())
        truth = torch.stack([want[rid.split("#")[0]][0][pos] for rid, pos in rows])
        runs = [torch.stack([want[rid.split("#")[0]][1][k][pos] for rid, pos in rows])
                for k in range(len(next(iter(want.values()))[1]))]
        close_to_truth(got, truth, runs, td, f"step {sid}")
