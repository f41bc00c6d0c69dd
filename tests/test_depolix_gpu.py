"""Depolix on the GPU: each mechanism's kernels alone against the plain functions, then whole
models (other sizes in every test than anywhere else) through the engine's runner, cache and
state slots: whole prompts, the stream after every layer, token-by-token decoding, portions down
to two tokens, unequal requests in one batch, pages and slots that come back, keys just inside and
just outside a window and among its kept first keys, a marked key far away among hundreds,
memories that carry a token for hundreds of steps, models drawn at random, and greedy generation
through the engine and its scheduler."""

from __future__ import annotations

import math
import os
import random

import numpy as np
import pytest
import torch
from safetensors.torch import load_file, save_file

import kvforge_amd
from kvforge_amd.config.presets import depolix as make_config
from kvforge_amd.engine.batch import StepEntry
from tests import replay_util as ru
from tests.plain import depolix as plain
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
@pytest.mark.parametrize("H,KV,d,dk,bs", [(2, 1, 16, 9, 4), (6, 3, 48, 40, 8), (5, 5, 80, 80, 16), (1, 1, 256, 200, 32),
                                          (8, 2, 64, 64, 12), (3, 1, 128, 100, 24)])
def test_convolved_q_k_and_v_over_runs_steps_and_slots(dtype, taps, H, KV, d, dk, bs):
    """Runs of every length around the taps and the kernel's tiles from positions on and off their
    borders, each continued from what the step before left in its slot; a slot that held
    another's rows starts from zeros at position 0; a sequence without a slot keeps nothing; a
    token without a page is not stored."""
    C = (H + 2 * KV) * d
    lens, more, third = [1, 2, 16, 17, 40, 3], [5, 1, 2, 33, 1, 1], [9, 1, 7, 2, 20, 1]
    totals = [a + b + c for a, b, c in zip(lens, more, third)]
    w = rand(C, taps, seed=taps, scale=0.6)
    real = torch.zeros(C, dtype=torch.bool).view(H + 2 * KV, d)
    real[:, :dk] = True                                        # the others are padding: zero rows and weights
    real = real.view(-1)
    w[~real] = 0.0
    xs = [(rand(n, C, seed=10 + i) * real).to(dtype).float() for i, n in enumerate(totals)]
    eps = 1e-3
    weights = (1.0 + rand(dk, seed=5, scale=0.3), 1.0 + rand(dk, seed=6, scale=0.3)) if taps == 3 else None

    def want(x):
        y = plain.short_conv(x, w).view(-1, H + 2 * KV, d)
        for lo, hi, nw in ((0, H, 0), (H, H + KV, 1)):
            y[:, lo:hi, :dk] = plain.rms(y[:, lo:hi, :dk], eps) * (weights[nw] if weights else 1.0)
        return y[:, :H], y[:, H:H + KV], y[:, H + KV:]

    wants = [want(x) for x in xs]
    n_seqs = len(lens)
    width = max(-(-n // bs) for n in totals)
    nb = n_seqs * width + 1
    order = torch.randperm(nb, generator=torch.Generator().manual_seed(3))[:n_seqs * width].view(n_seqs, width)
    table = order.to(torch.int32)
    table[3, 0] = -1                                             # given back
    k_pages = torch.full((nb, KV, bs, d), 7.0, dtype=dtype, device=DEV)
    v_pages = torch.full((nb, KV, d, bs), 7.0, dtype=dtype, device=DEV)
    pad = (-(taps - 1) * C) % 4
    state = torch.full((7, 4 + (taps - 1) * C + pad + 4), 5.0, device=DEV)
    slots = [3, 0, 6, 2, 5, -1]

    def step(parts):
        rows = torch.cat([xs[s][a:e] for s, a, e in parts])
        wide = torch.cat([rows, torch.full((len(rows), 8), 9.0)], dim=1).to(dtype).to(DEV)
        q = torch.full((len(rows), H * d), 7.0, dtype=dtype, device=DEV)
        ops().conv_norm_kvwrite(wide, w.t().contiguous().to(DEV), i32([0] + list(np.cumsum([e - a for _, a, e in parts]))),
                                i32([p for _, a, e in parts for p in range(a, e)]), i32([slots[s] for s, _, _ in parts]),
                                state[:, 4:4 + (taps - 1) * C] if taps > 1 else None,
                                table[[s for s, _, _ in parts]].contiguous().to(DEV), q, k_pages, v_pages, H, KV, d,
                                len(parts), max(e - a for _, a, e in parts), norm_dim=dk, eps=eps,
                                q_weight=weights[0].to(DEV) if weights else None,
                                k_weight=weights[1].to(DEV) if weights else None)
        at = 0
        for s, a, e in parts:
            got = q[at:at + e - a].float().cpu().view(-1, H, d)
            torch.testing.assert_close(got, wants[s][0][a:e], **tol(dtype), msg=lambda m: f"q of {s}, {a} to {e}: {m}")
            at += e - a

    step([(s, 0, n) for s, n in enumerate(lens)])
    step([(s, lens[s], lens[s] + more[s]) for s in range(5)])       # the one without a slot does not go on
    for i in range(max(third)):                                    # and single tokens
        step([(s, totals[s] - third[s] + i, totals[s] - third[s] + i + 1) for s in range(5) if i < third[s]])
    kc, vc = k_pages.float().cpu(), v_pages.float().cpu()
    for s in range(n_seqs):
        for p in range(lens[s] if s == 5 else totals[s]):
            page, off = int(table[s, p // bs]), p % bs
            if page < 0:
                continue
            torch.testing.assert_close(kc[page, :, off], wants[s][1][p], **tol(dtype), msg=lambda m: f"k {s}, {p}: {m}")
            torch.testing.assert_close(vc[page, :, :, off], wants[s][2][p], **tol(dtype), msg=lambda m: f"v {s}, {p}: {m}")
    untouched = [p for p in range(nb) if p not in table.flatten().tolist()]
    assert float((k_pages[untouched] - 7.0).abs().max()) == 0.0 and float((v_pages[untouched] - 7.0).abs().max()) == 0.0
    assert float((state[[1, 4]] - 5.0).abs().max()) == 0.0 and float((state[:, :4] - 5.0).abs().max()) == 0.0
    assert float((state[:, 4 + (taps - 1) * C:] - 5.0).abs().max()) == 0.0


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,KV,d,bs,window,keep,far", [
    (4, 2, 16, 8, 0, 0, 3), (6, 1, 48, 16, 33, 5, 20), (8, 2, 64, 16, 40, 37, 150), (3, 3, 80, 8, 64, 0, 64),
    (20, 1, 32, 16, 17, 3, 40), (2, 1, 208, 16, 50, 9, 90), (16, 1, 128, 16, 0, 0, 2000), (2, 2, 256, 24, 31, 2, 45),
    (4, 1, 64, 6, 20, 4, 30)])
def test_attention_with_a_bias_by_distance(dtype, H, KV, d, bs, window, keep, far):
    """Query runs and single tokens, one cut of the key range and several; tables shorter and longer
    than the contexts, and too long for LDS; a window's kept first keys lie at distances of
    their own."""
    scale = 1.0 / math.sqrt(d)
    table = rand(H, far, seed=far, scale=2.0)
    for seq_lens, q_lens in (([90, 33, 150, 5], [40, 33, 2, 5]), ([7, 90, 1, 300], [1, 1, 1, 1])):
        paged = Paged(seq_lens, KV, d, bs, dtype, seed=d)
        n = sum(q_lens)
        buf = rand(n, H * d, seed=d + 1, scale=1.5).to(dtype)
        cu, ctx = i32([0] + list(np.cumsum(q_lens))), i32(seq_lens)
        want, off = [], 0
        for s, (m, ql) in enumerate(zip(seq_lens, q_lens)):
            k, v = (t[s].float().repeat_interleave(H // KV, dim=1) for t in (paged.keys, paged.values))
            sc = torch.einsum("qhd,khd->hqk", buf[off:off + ql].float().view(ql, H, d), k) * scale
            i, j = torch.arange(m - ql, m)[:, None], torch.arange(m)[None, :]
            sc = sc + table[:, (i - j).clamp(0, far - 1)]
            seen = j <= i
            if window:
                seen = seen & ((i - j < window) | (j < keep))
            sc = sc.masked_fill(~seen[None], float("-inf"))
            want.append(torch.einsum("hqk,khd->qhd", torch.softmax(sc, -1), v).reshape(ql, H * d))
            off += ql
        want = torch.cat(want)
        args = (buf.to(DEV), paged.k.to(DEV), paged.v.to(DEV), paged.table.to(DEV))
        dt = table.to(DEV)
        if max(q_lens) > 1:
            for tiles in (1, 2):
                per = ops().prefill_rows_per_item(dtype, d, bs, tiles)
                if tiles == 2 and per == ops().prefill_rows_per_item(dtype, d, bs, 1):
                    continue
                rows = [(s, i, -1) for s, q in enumerate(q_lens) for i in range(-(-q * (H // KV) // per))]
                out = torch.zeros(n, H * d, dtype=dtype, device=DEV)
                ops().attn_prefill(*args, cu, ctx, i32(rows), out, H, KV, d, scale, window, rows_per_item=per,
                                   keep_first=keep, dist=dt)
                torch.testing.assert_close(out.float().cpu(), want, **tol(dtype))
            continue
        for splits in (1, 3):
            out = torch.zeros(n, H * d, dtype=dtype, device=DEV)
            ws = (torch.empty(n * H * splits * d, device=DEV), torch.empty(n * H * splits * 2, device=DEV))
            ops().attn_decode(*args, None, n, cu, ctx, out, H, KV, d, scale, window, splits, ws, keep_first=keep, dist=dt)
            torch.testing.assert_close(out.float().cpu(), want, **tol(dtype))


def test_a_bias_by_distance_goes_with_nothing_else_on_the_matrix_cores():
    from kvforge_amd.kernels.ops import KernelError
    paged = Paged([20], 1, 16, 8, torch.bfloat16, seed=1)
    q = torch.zeros(20, 32, dtype=torch.bfloat16, device=DEV)
    args = (q, paged.k.to(DEV), paged.v.to(DEV), paged.table.to(DEV), i32([0, 20]), i32([20]),
            prefill_work([20], 2, torch.bfloat16, 16, 8).to(DEV), torch.zeros_like(q), 2, 1, 16, 0.3)
    dist = torch.zeros(2, 5, device=DEV)
    for kw in (dict(slopes=torch.ones(2, device=DEV)), dict(sinks=torch.ones(2, device=DEV)), dict(score_cap=3.0),
               dict(chunk=8)):
        with pytest.raises(KernelError, match="biases by distance"):
            ops().attn_prefill(*args, dist=dist, **kw)


def run_memory(q, k, v, za, zb, neg_a, dt_bias, runs, state, slots, positions, H, G, dk, dv):
    """The kernels over the runs of one step; rows of q, k, v in 32-bit."""
    o = ops()
    n = q.shape[0]
    rows = torch.cat([q, k, v, torch.full((n, 3), 9.0)], dim=1).to(DEV)
    decay = torch.cat([torch.full((n, 2), 9.0), za], dim=1).to(DEV)
    steps = torch.cat([torch.full((n, 1), 9.0), zb], dim=1).to(DEV)
    chunks, rr = o.ssm_plan(runs, dk, o.CHDELTA_CHUNK_FROM)
    multi = None
    if chunks:
        multi = {"chunks": i32(chunks).view(-1, 4), "runs": i32(rr).view(-1, 3)}
        for name, (shape, dt) in o.chdelta_scratch(n, len(chunks) // 4, H, dk, dv).items():
            multi[name] = torch.full(shape, float("nan"), dtype=dt, device=DEV)
    out = torch.full((n, H * dv), 7.0, device=DEV)
    o.chdelta_scan(rows, 0, G * dk, 2 * G * dk, decay, 2, steps, 1, neg_a.to(DEV), dt_bias.to(DEV),
                   i32([0] + list(np.cumsum(runs))), i32(positions), i32(slots), state, out, len(runs), H, G, dk, dv,
                   multi=multi, short_runs=any(r < o.CHDELTA_CHUNK_FROM for r in runs))
    return out.cpu()


@pytest.mark.parametrize("H,G,dk,dv", [(2, 1, 16, 16), (6, 3, 24, 40), (2, 2, 64, 130), (3, 1, 100, 72), (2, 1, 256, 64),
                                       (4, 2, 8, 200), (2, 1, 128, 128), (1, 1, 1, 1), (2, 1, 33, 65), (1, 1, 150, 20)])
def test_the_memory_over_runs_steps_and_slots(H, G, dk, dv):
    """Sequences of every kind in one step: a few tokens (token by token), lengths on both sides of
    the chunks' first and of their edges, a single token; then each goes on from its slot the
    other way.  Decays per channel from all but none to gates that close (for one token, and for a
    channel throughout); a slot that held another's memory starts from zeros at position 0; a sequence
    without a slot keeps nothing.  Slots are a block of columns of wider ones."""
    lens = [9, 150, 1, 64, 23, 24, 65]
    more = [70, 3, 20, 1, 64, 63, 40]
    g = torch.Generator().manual_seed(dk + dv)
    neg_a = -torch.exp(torch.randn(H, generator=g))
    dt_bias = torch.randn(H * dk, generator=g)
    seqs = []
    for n in (a + b for a, b in zip(lens, more)):
        q, k = plain.unit(torch.randn(n, G, dk, generator=g)), plain.unit(torch.randn(n, G, dk, generator=g))
        v = torch.randn(n, H, dv, generator=g)
        za, zb = torch.randn(n, H, dk, generator=g) * 2.0 - 2.0, torch.randn(n, H, generator=g) * 2.0
        za[torch.rand(n, H, dk, generator=g) < 0.03] = 60.0                       # gates that close
        za[:, :, 0] = 25.0 if dk > 1 else -1.0
        if dk > 3:
            za[:, :, 3] = -30.0                                                  # and one that never does
        seqs.append((q, k, v, za, zb))

    def truth(q, k, v, za, zb):
        q, k, v, za, zb = (t.double() for t in (q, k, v, za, zb))
        a = torch.exp(neg_a[:, None] * plain.softplus(za + dt_bias.view(H, dk)))
        return plain.channel_delta_scan(plain.of_group(q, H), plain.of_group(k, H), v, a, torch.sigmoid(zb)).float()

    want = [truth(*s) for s in seqs]
    size = max(float(w.abs().max()) for w in want)
    close = dict(atol=2e-5 * size, rtol=2e-4)
    floats = H * dk * dv
    wide = torch.full((9, floats + 7), 5.0, device=DEV)                # leftovers of others in every slot
    state = wide[:, 4:4 + floats]
    slots = [2, 0, 3, 8, 5, 6, 1]

    def step(parts):
        cat = lambda i: torch.cat([seqs[s][i][a:b].reshape(b - a, -1) for s, a, b in parts])  # noqa: E731
        pos = [p for _, lo, hi in parts for p in range(lo, hi)]
        return run_memory(cat(0), cat(1), cat(2), cat(3), cat(4), neg_a, dt_bias, [hi - lo for _, lo, hi in parts], state,
                          [slots[s] for s, _, _ in parts], pos, H, G, dk, dv)

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
    before = wide.clone()
    alone = [(0, 0, 70)]
    compare(step(alone), alone)
    assert torch.equal(before, wide)
    assert float((wide[:, :4] - 5.0).abs().max()) == 0.0 and float((wide[:, -3:] - 5.0).abs().max()) == 0.0


def test_channels_that_are_kept_and_channels_that_are_dropped():
    """With beta near one, keys along single channels and no decay but on some channels, a query for a
    kept channel's key gets the last value written under it, across chunks, and one for a dropped
    channel's key gets nothing."""
    dk, dv, n = 16, 16, 130
    which = [i % 4 for i in range(n)]                          # channels 0 to 3 in turn; channel 2 is dropped at once
    k = torch.eye(dk)[which]
    v = rand(n, dv, seed=3)
    za = torch.full((n, 1, dk), -60.0)
    za[:, :, 2] = 60.0
    q = torch.eye(dk)[[(i + 1) % 4 for i in range(n)]]          # asks for the key written three tokens ago
    state = torch.zeros(1, dk * dv, device=DEV)
    got = run_memory(q, k, v, za.view(n, dk), torch.full((n, 1), 40.0), torch.tensor([-1.0]), torch.zeros(dk), [n], state, [0],
                     list(range(n)), 1, 1, dk, dv)
    for t in range(3, n):
        want = torch.zeros(dv) if (t + 1) % 4 == 2 else v[t - 3]
        torch.testing.assert_close(got[t], want, atol=1e-4, rtol=1e-4)


@pytest.mark.parametrize("runs", [[400], [20] * 20])
def test_decays_are_exact_enough_to_hold_over_hundreds_of_tokens(runs):
    """One channel per head, written once and left to fade: what is left after t tokens is the decay to the power
    of t, for pre-activations from channels that all but never fade to ones that are gone at once; chunk by chunk and
    token by token."""
    H, n = 61, sum(runs)
    z = torch.linspace(-18.0, 12.0, H)
    neg_a = -torch.exp(torch.linspace(-3.0, 1.0, H))[torch.randperm(H, generator=torch.Generator().manual_seed(1))]
    q, k, v = torch.ones(n, H, 1), torch.ones(n, H, 1), torch.ones(n, H, 1)
    zb = torch.full((n, H), -200.0)
    zb[0] = 200.0
    state = torch.zeros(1, H, device=DEV)
    got, at = [], 0
    for r in runs:
        part = slice(at, at + r)
        got.append(run_memory(q[part].view(r, H), k[part].view(r, H), v[part].view(r, H), z.expand(r, H).contiguous(), zb[part],
                              neg_a, torch.zeros(H), [r], state, [0], list(range(at, at + r)), H, H, 1, 1))
        at += r
    rate = neg_a.double() * plain.softplus(z.double())
    want = torch.exp(torch.arange(n, dtype=torch.float64)[:, None] * rate[None, :])
    # a relative error of 3e-7 (and of the exponent's own rounding) a token
    allowed = 1e-6 + torch.arange(n)[:, None] * (3e-7 + 3e-7 * rate.abs()[None, :]) * want
    err = (torch.cat(got).double() - want).abs()
    assert bool((err <= allowed + 1e-30).all()), (float((err / allowed).max()), int((err / allowed).amax(0).argmax()))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("paired", [True, False])
@pytest.mark.parametrize("bias", [True, False])
@pytest.mark.parametrize("inter", [6, 40, 1024])
def test_limited_pairs(dtype, paired, bias, inter):
    gu = rand(5, 2 * inter, seed=1, scale=3.0).to(dtype)
    bg, bu = (rand(inter, seed=2), rand(inter, seed=3)) if bias else (None, None)
    out = torch.zeros(5, inter, dtype=dtype, device=DEV)
    ops().gated_act(gu.to(DEV), out, "limited", paired, bg.to(DEV) if bias else None, bu.to(DEV) if bias else None, limit=1.7,
                    scale=0.6)
    g, u = (gu.float().view(5, inter, 2).unbind(-1)) if paired else gu.float().split(inter, dim=1)
    want = plain.limited_gate(g + (bg if bias else 0.0), u + (bu if bias else 0.0), 1.7) * 0.6
    torch.testing.assert_close(out.float().cpu(), want, **tol(dtype))
    with pytest.raises(Exception, match="limit"):
        ops().gated_act(gu.to(DEV), out, "limited", paired)


@pytest.mark.parametrize("m", [1, 3, 17, 40])
@pytest.mark.parametrize("bias", [True, False])
def test_limited_pairs_in_the_store_of_the_product(m, bias):
    k, inter = 64, 48
    a, w = rand(m, k, seed=1).bfloat16(), rand(2 * inter, k, seed=2, scale=0.4).bfloat16()
    bg, bu = (rand(inter, seed=3), rand(inter, seed=4)) if bias else (None, None)
    out = torch.zeros(m, inter, dtype=torch.bfloat16, device=DEV)
    ops().gemm_gated(a.to(DEV), ops().streamed(w.to(DEV)), out, "limited", bg.to(DEV) if bias else None,
                     bu.to(DEV) if bias else None, limit=0.9, scale=1.3)
    g, u = (a.float() @ w.float().T).view(m, inter, 2).unbind(-1)
    want = plain.limited_gate(g + (bg if bias else 0.0), u + (bu if bias else 0.0), 0.9) * 1.3
    torch.testing.assert_close(out.float().cpu(), want, **tol(torch.bfloat16))


@pytest.mark.parametrize("R,top", [(1, 1), (8, 1), (8, 3), (70, 16), (512, 5)])
def test_router_weights_by_the_softmax_over_the_chosen_logits(R, top):
    z, b = rand(9, R + 3, seed=R, scale=3.0), rand(R, seed=R + 1, scale=4.0)
    z[3] *= 40.0                                                  # far apart: the softmax over all would vanish
    chosen = torch.full((9, top), -5, dtype=torch.int32, device=DEV)
    weights = torch.full((9, top), -5.0, device=DEV)
    for bias in (None, b):
        ops().moe_topk(z.to(DEV)[:, :R], None, chosen, weights, "chosen", bias=bias.to(DEV) if bias is not None else None,
                       scale=0.7)
        v, i = torch.topk(z[:, :R] + (bias if bias is not None else 0.0), top)
        assert torch.equal(chosen.cpu().long(), i)
        torch.testing.assert_close(weights.cpu(), 0.7 * torch.softmax(v, -1), atol=1e-6, rtol=1e-5)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("E,top,ff,width,n", [(5, 2, 32, 64, 7), (4, 1, 24, 40, 40), (8, 3, 64, 104, 400), (3, 3, 16, 30, 5)])
def test_experts_with_limited_pairs_and_a_router_bias(dtype, E, top, ff, width, n):
    """The layer alone, on the grouped kernels and on the products over all experts."""
    from kvforge_amd.engine.batch import Step, Workspace
    from kvforge_amd.parts import RoutedExperts

    part = RoutedExperts("f", width, ff, E, top, scores="chosen", correct=False, router_bias=True, form="limited", limit=0.8,
                         out_scale=0.6)
    w = {k: rand(*v.shape, seed=i, scale=0.3).to(dtype) for i, (k, v) in enumerate(sorted(part.weight_specs().items()))}
    # logits that no rounding reorders: the rows' first elements name them
    x = rand(n, width, seed=40)
    levels = torch.linspace(-2.0, 2.0, E)
    g = torch.Generator().manual_seed(3)
    for t in range(n):
        x[t, :E] = levels[torch.randperm(E, generator=g)]
    w["f.router"] = torch.eye(E, width).to(dtype)
    w["f.router.b"] = torch.zeros(E).to(dtype)
    w["f.router.b"][0] = -16.0 if top < E else 0.5
    x = x.to(dtype)
    part.load({k: v.to(DEV) for k, v in w.items()})
    part.seal()
    step = Step()
    step.ws, step.act_dtype, step.n_tokens = Workspace(DEV), dtype, n
    rows = rand(n, width, seed=50).to(DEV)
    base = rows.cpu().clone()
    part.forward(x.to(DEV), step, rows)
    step.settle()
    mlp = {"router": {"experts": E, "top": top}, "expert": {"limit": 0.8}}
    want = base + 0.6 * plain.routed_ff(x.float(), {k: v.float() for k, v in w.items()}, "f.", mlp)
    spread = float((want - base).std())       # the outputs' own size: a bf16 engine rounds activations and outputs
    torch.testing.assert_close(rows.cpu(), want, rtol=1e-4, atol=(1e-5 if dtype == torch.float32 else 3e-2) * spread)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n", [3, 90])
def test_a_dense_layers_bias_stays_owed_until_the_next_norm(dtype, n):
    """The stream as the next norm leaves it, and as settling leaves it."""
    from kvforge_amd.engine.batch import Step, Workspace
    from kvforge_amd.parts import GatedFeedForward, OnePlusRMSNorm
    from kvforge_amd.parts.block import norm_rows

    width, ff = 56, 40
    part = GatedFeedForward("f", width, ff, "limited", bias=True, names={"gate": "gate", "up": "up", "down": "down"},
                            bias_suffix=".b", limit=1.1, out_scale=0.7)
    w = {k: rand(*v.shape, seed=i, scale=0.4).to(dtype) for i, (k, v) in enumerate(sorted(part.weight_specs().items()))}
    part.load({k: v.to(DEV) for k, v in w.items()})
    part.seal()
    norm = OnePlusRMSNorm("n", width, 1e-5)
    nw = rand(width, seed=9, scale=0.2)
    norm.load({"n": nw.to(DEV)})
    x, rows = rand(n, width, seed=20).to(dtype), rand(n, width, seed=21)
    want = rows + 0.7 * plain.dense_ff(x.float(), {k: v.float() for k, v in w.items()}, "f.", 1.1)
    for settle in (False, True):
        step = Step()
        step.ws, step.act_dtype, step.n_tokens = Workspace(DEV), dtype, n
        stream, out = rows.to(DEV), torch.zeros(n, width, dtype=dtype, device=DEV)
        part.forward(x.to(DEV), step, stream)
        assert step.owed_bias is not None
        if settle:
            step.settle()
        norm_rows(norm, stream, out, step)
        assert step.owed_bias is None and step.owed is None
        torch.testing.assert_close(stream.cpu(), want, **tol(dtype))
        torch.testing.assert_close(out.float().cpu(), plain.one_plus_norm(want, nw, 1e-5), **tol(dtype))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("h", [30, 88, 2048])
@pytest.mark.parametrize("rows", [False, True])
def test_a_norm_adds_a_bias_owed_to_every_row(dtype, h, rows):
    x, d, b, w = (rand(*s, seed=i) for i, s in enumerate(((4, h), (4, h), (h,), (h,))))
    d = d.to(dtype)
    for add in (None, d):
        dx, out = x.clone().to(DEV), torch.zeros(2 if rows else 4, h, dtype=dtype, device=DEV)
        ops().rmsnorm(dx, w.to(DEV), 1e-4, out, i32([3, 1]) if rows else None, add.to(DEV) if add is not None else None,
                      b.to(DEV))
        want = x + b + (d.float() if add is not None else 0.0)
        torch.testing.assert_close(dx.cpu(), x if rows else want, atol=1e-6, rtol=1e-6)
        y = plain.norm(want, w, 1e-4)
        torch.testing.assert_close(out.float().cpu(), y[[3, 1]] if rows else y, **tol(dtype))


@pytest.mark.parametrize("h", [1, 30, 88, 1024, 2052, 4096, 5000, 9000])
def test_two_normed_rows_join_the_stream(h):
    x, a, b = rand(3, h, seed=1, scale=4.0), rand(3, h, seed=2, scale=0.1), rand(3, h, seed=4, scale=7.0)
    wa, wb = 1.0 + rand(h, seed=3, scale=0.3), rand(h, seed=5)
    b[1] = 0.0
    dx = x.clone().to(DEV)
    ops().rms_add_two(dx, a.to(DEV), wa.to(DEV), b.to(DEV), wb.to(DEV), 1e-4)
    torch.testing.assert_close(dx.cpu(), x + plain.norm(a, wa, 1e-4) + plain.norm(b, wb, 1e-4), atol=2e-5, rtol=2e-5)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,O,I,n", [(1, 16, 8, 3), (5, 28, 44, 70), (4, 64, 192, 300), (3, 12, 30, 9), (2, 64, 512, 300),
                                     (3, 70, 128, 290)])
def test_a_gate_per_output_where_the_values_are_read_out(dtype, H, O, I, n):
    x, w, g = rand(n, H * I, seed=1).to(dtype), rand(H, O, I, seed=2, scale=I ** -0.5).to(dtype), rand(n, H * O + 5, seed=3, scale=2.0).to(dtype)
    out = torch.zeros(n, H * O, dtype=dtype, device=DEV)
    for lead in (0, 5):
        gate = g.to(DEV)[:, lead:lead + H * O]
        ops().head_product(x.to(DEV), I, w.to(DEV), out, O, gate=gate, gate_outputs=True, scale=0.7)
        want = torch.einsum("nhi,hoi->nho", x.float().view(n, H, I), w.float()).reshape(n, H * O)
        want = want * torch.sigmoid(g.float()[:, lead:lead + H * O]) * 0.7
        torch.testing.assert_close(out.float().cpu(), want, **tol(dtype))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rank,lead", [(1, 0), (30, 3), (96, 8), (768, 0), (2500, 1), (4096, 16)])
def test_the_norm_of_a_block_of_columns(dtype, rank, lead):
    x, w = rand(5, lead + rank + 8, seed=1, scale=2.0).to(dtype), 1.0 + rand(rank, seed=2, scale=0.3)
    out = torch.zeros(5, rank, dtype=dtype, device=DEV)
    ops().latent_norm(x.to(DEV)[:, lead:lead + rank], w.to(DEV), 1e-3, out)
    torch.testing.assert_close(out.float().cpu(), plain.norm(x.float()[:, lead:lead + rank], w, 1e-3), **tol(dtype))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,dv", [(1, 1), (3, 20), (4, 128)])
def test_head_norm_under_a_sigmoid_gate(dtype, H, dv):
    o, g, w = rand(6, H * dv, seed=1, scale=3.0), rand(6, H * dv + 4, seed=2, scale=2.0), 1.0 + rand(dv, seed=3, scale=0.3)
    out = torch.zeros(6, H * dv, dtype=dtype, device=DEV)
    ops().linmem_out(o.to(DEV), g.to(DEV)[:, 4:], w.to(DEV), 1e-3, out, H, dv, sigmoid=True)
    want = (plain.rms(o.view(6, H, dv), 1e-3) * w).reshape(6, H * dv) * torch.sigmoid(g[:, 4:])
    torch.testing.assert_close(out.float().cpu(), want, **tol(dtype))


# ======================================================================= whole models
def shape_a():
    """Both mixers and both feed-forwards; sizes that no kernel's tiles divide."""
    lat = dict(heads=5, dim=20, rot_dim=12, vdim=28, q_rank=36, kv_rank=44, scale=0.21, base=3000.0,
               scaling=(2.5, 40, 8.0, 1.0))
    return make_config(vocab=203, width=88, layers=[
        ("parallel", dict(left=dict(heads=6, kv_heads=3, dim=20, vdim=12, scale=0.4, conv=4, bias_max=50, buckets=10,
                                    window=37, keep_first=5),
                          right=dict(heads=6, kv_heads=2, dim=28, vdim=36, conv=5, a_rank=7, g_rank=9)), (24, 2.5, 7, 2)),
        ("latent_attention", lat, (104, 1.5)),
        ("parallel", dict(left=dict(heads=4, kv_heads=4, dim=12, vdim=28, scale=0.5, conv=2, bias_max=300, buckets=24,
                                    window=9),
                          right=dict(heads=3, kv_heads=3, dim=20, vdim=16, conv=3, a_rank=16, g_rank=4)), None),
        ("latent_attention", dict(lat, heads=3, dim=8, vdim=12, q_rank=24, kv_rank=20), (40, 0.9, 3, 3))],
        eps=1e-5, embed_scale=9.4, residual_mult=0.6, logit_scale=0.8, max_positions=2048)


def shape_b():
    """What a model may make equal or one: one head everywhere, as many q/k heads as memories, one tap, one
    expert of one, no plain query part, no rotation, no window, ranks of one, every constant one."""
    lat = dict(heads=1, dim=16, rot_dim=16, vdim=16, q_rank=16, kv_rank=16, scale=1.0, base=100.0)
    left = dict(heads=1, kv_heads=1, dim=16, vdim=16, scale=1.0, conv=1, bias_max=2, buckets=2)
    right = dict(heads=1, kv_heads=1, dim=16, vdim=16, conv=1, a_rank=1, g_rank=1)
    return make_config(vocab=64, width=32, layers=[
        ("latent_attention", lat, None), ("parallel", dict(left=left, right=right), (16, 1.0, 1, 1)),
        ("latent_attention", dict(lat, dim=0), (32, 1.0)),
        ("parallel", dict(left=dict(left, conv=2, buckets=4, bias_max=7, window=1, keep_first=1),
                          right=dict(right, heads=2, kv_heads=2, conv=2)), (16, 1.0, 3, 3)),
        ("latent_attention", dict(lat, rot_dim=0, scale=0.5, q_rank=1), (16, 1.0))], eps=1e-6, max_positions=512)


def shape_c():
    """Layers wide enough for the kernels that serving a real model takes: latents on the matrix cores,
    memories wider than a wave's rows, experts on the grouped kernels, a deep feed-forward, a vocabulary that
    ends inside a group of 16 columns."""
    lat = dict(heads=6, dim=64, rot_dim=32, vdim=64, q_rank=160, kv_rank=128, scale=0.1, base=100000.0,
               scaling=(8.0, 256, 32.0, 1.0))
    par = dict(left=dict(heads=8, kv_heads=2, dim=128, vdim=96, scale=0.09, conv=4, bias_max=128, buckets=32, window=200,
                         keep_first=16),
               right=dict(heads=4, kv_heads=2, dim=128, vdim=128, conv=4, a_rank=64, g_rank=48))
    return make_config(vocab=1000, width=384, layers=[
        ("latent_attention", lat, (4096, 4.0)), ("parallel", par, (128, 3.0, 8, 2)), ("latent_attention", lat, (64, 3.0, 8, 1)),
        ("parallel", par, (512, 7.0))], eps=1e-5, embed_scale=12.0, residual_mult=0.5, logit_scale=2.5, max_positions=2048)


def shape_d():
    """A latent row beyond the matrix-core kernels' heads, memories of 256-element keys, a wide head."""
    lat = dict(heads=3, dim=32, rot_dim=24, vdim=40, q_rank=50, kv_rank=300, scale=0.15, base=5000.0)
    return make_config(vocab=150, width=64, layers=[
        ("latent_attention", lat, (32, 2.0, 4, 2)),
        ("parallel", dict(left=dict(heads=2, kv_heads=1, dim=40, vdim=250, scale=0.2, conv=8, bias_max=1000, buckets=40,
                                    window=64, keep_first=40),
                          right=dict(heads=2, kv_heads=1, dim=256, vdim=24, conv=8, a_rank=20, g_rank=20)), (48, 1.2))],
        eps=1e-4, embed_scale=3.0, residual_mult=1.3, logit_scale=1.5, max_positions=512)


SHAPE = {"a": shape_a, "b": shape_b, "c": shape_c, "d": shape_d}


def liven(folder: str, cfg: dict, seed: int = 0) -> None:
    """Random weights of std 0.02 give flat attention and memories that hardly turn.  Scaled so that attention
    is peaked and gates swing.  The routers read a few coordinates of the stream that the embedding alone
    fills (nothing is added to them, and their norm weights are one) with levels evenly spaced and shuffled per
    token, so that every token has its own experts and no rounding can reorder them; one expert's bias keeps it
    from being chosen."""
    path = os.path.join(folder, "model.safetensors")
    w = load_file(path)
    routed = [l["mlp"]["router"]["experts"] for l in cfg["layers"] if l["mlp"] and l["mlp"]["kind"] == "moe"]
    E = max(routed, default=0)
    g = torch.Generator().manual_seed(seed)
    embed_std = 2.0 / cfg["embedding"]["scale"]
    for k in list(w):
        f = 1.0
        if k == "embed":
            f = embed_std / 0.02
        elif k.endswith((".uq", ".dkv")):
            f = 6.0
        elif k.endswith((".dq", ".uk", ".uv", ".g", ".q", ".k", ".v", ".b", ".a1", ".g1")) and ".mix" in k:
            f = 8.0
        elif k.endswith((".a2", ".g2")):
            f = 20.0
        elif k.endswith((".o", ".down", ".up", ".gate")):
            f = 6.0
        elif k.endswith((".gate.b", ".up.b", ".down.b")):
            f = 20.0
        elif k == "head":
            f = 3.0
        if f != 1.0:
            w[k] = (w[k].float() * f).to(w[k].dtype)
        if k.endswith(".right.dt_bias"):
            w[k] = (w[k].float() - 2.0).to(w[k].dtype)
    if E:
        for k in list(w):
            if k.endswith(".norm1"):
                w[k][:E] = 0.0                          # (stored around zero)
            elif k.endswith((".left.out", ".right.out", ".down.b", ".mix.o")) or (k.endswith(".down") and ".mlp." in k):
                w[k][:E] = 0.0
        levels = torch.linspace(-2.0, 2.0, E) if E > 1 else torch.zeros(1)
        for t in range(w["embed"].shape[0]):
            w["embed"][t, :E] = (levels[torch.randperm(E, generator=g)] * embed_std).to(w["embed"].dtype)
        for i, layer in enumerate(cfg["layers"]):
            if layer["mlp"] and layer["mlp"]["kind"] == "moe":
                r = w[f"l{i}.mlp.router"]
                r[:] = torch.eye(*r.shape).to(r.dtype)[torch.randperm(r.shape[0], generator=g)]
                w[f"l{i}.mlp.router.b"][:] = 0.0
                if layer["mlp"]["router"]["top"] < r.shape[0]:
                    w[f"l{i}.mlp.router.b"][r.shape[0] // 2] = -40.0
    save_file(w, path, metadata={"format": "pt"})


_MODELS: dict = {}


def model_folder(tmp_path_factory, name: str, dtype):
    key = (name, dtype)
    if key not in _MODELS:
        folder = str(tmp_path_factory.mktemp(f"depolix_{name}_{NAME[dtype]}"))
        cfg = SHAPE[name]()
        kvforge_amd.write_random_model(folder, cfg, seed=len(name) + 23, dtype=NAME[dtype])
        liven(folder, cfg)
        _MODELS[key] = (folder, cfg, load_file(os.path.join(folder, "model.safetensors")))
    return _MODELS[key]


_WANT: dict = {}


def plain_logits(cfg, w, toks, dtype):
    """(the truth, plain runs with the roundings of ``dtype``): the plain model in 64-bit, and in
    32-bit (for a 32-bit engine) or in 32-bit with every trip through memory that a bfloat16
    engine may make rounded to bfloat16: as the weights are, and twice with them moved by half a
    bfloat16 step, which shows the rows where the design multiplies rounding."""
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
    """More than a dozen chunks of the memories, latents over many pages, many windows: whole, in large and
    small portions, and its last tokens one by one."""
    folder, cfg, w = model_folder(tmp_path_factory, name, dtype)
    runner = make_runner(folder, dtype, block_size=16, num_blocks=80, tokens=1200)
    toks = prompts_for(cfg, [1100], 11)["r0"]
    for plan in ([[("r0", 0, 1100)]], in_portions("r0", 1100, (300, 64, 65, 7, 129, 2)),
                 [[("r0", 0, 1050)]] + [[("r0", i, i + 1)] for i in range(1050, 1100)]):
        got = replay(runner, {"r0": toks}, plan)["r0"]
        check(got, cfg, w, toks, dtype, f"{name}, {len(plan)} steps")


def marked_latent_model(tmp_path, dtype):
    """Token 1 is marked: its embedding lies along one axis that no other token uses, element 0 of its latent is
    all there is of it, every query has a constant that meets that element, the values carry it on.  So the
    marked token scores far above all others for every query."""
    V, W, rank, qr, H = 50, 32, 24, 8, 2
    lat = dict(heads=H, dim=16, rot_dim=8, vdim=16, q_rank=qr, kv_rank=rank, scale=1.0, base=1000.0,
               scaling=(4.0, 128, 16.0, 1.0))
    cfg = make_config(vocab=V, width=W, layers=[("latent_attention", lat, None)], max_positions=2048)
    folder = str(tmp_path / "marked")
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
    dq = torch.zeros(qr, W)
    dq[0, 1] = 1.0
    dq[1:] = rand(qr - 1, W, seed=8, scale=0.05)
    uq = torch.zeros(H * 24, qr)
    uq[0, 0] = uq[24, 0] = 1.0
    uk = rand(H * 16, rank, seed=3, scale=0.1)
    uk[0] = uk[16] = 0.0
    uk[0, 0] = uk[16, 0] = 1.0
    uv = rand(H * 16, rank, seed=4, scale=0.1)
    uv[:, 0] = rand(H * 16, seed=5, scale=1.5)
    new = {"embed": e, "l0.mix.dkv": dkv, "l0.mix.dkv.norm": torch.ones(rank), "l0.mix.dq": dq, "l0.mix.dq.norm": torch.ones(qr),
           "l0.mix.uq": uq, "l0.mix.uk": uk, "l0.mix.uv": uv, "l0.mix.g": rand(H * 16, W, seed=6, scale=0.1),
           "l0.mix.o": rand(W, H * 16, seed=7, scale=0.5), "l0.norm1": torch.zeros(W)}
    for k, t in new.items():
        assert w[k].shape == t.shape, k
        w[k] = t.to(w[k].dtype)
    save_file(w, path, metadata={"format": "pt"})
    return folder, cfg, load_file(path)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("bs", [8, 16])
def test_one_latent_among_hundreds(tmp_path, dtype, bs):
    """The logits follow the marked token from hundreds of tokens away, wherever it lies: first,
    in the middle of a page, a page's last and first, a portion's last; read whole, in portions
    and token by token."""
    folder, cfg, w = marked_latent_model(tmp_path, dtype)
    runner = make_runner(folder, dtype, block_size=bs, num_blocks=-(-700 // bs), tokens=640)
    g = torch.Generator().manual_seed(bs)
    for at in (0, 7, bs - 1, bs, 12 * bs - 1, 200):
        n = at + 320
        toks = torch.randint(2, 50, (n,), generator=g).tolist()
        toks[at] = 1
        want = plain.forward(cfg, w, toks)
        blind = plain.forward(cfg, w, [t if i != at else 2 for i, t in enumerate(toks)])
        assert float((want[-1] - blind[-1]).abs().max()) > 0.3 * float(want.std())      # seen from the end
        for plan in ([[("x", 0, n)]], in_portions("x", n, (at + 1, 2, 31)),
                     [[("x", 0, n - 40)]] + [[("x", i, i + 1)] for i in range(n - 40, n)]):
            got = replay(runner, {"x": toks}, plan)["x"]
            check(got, cfg, w, toks, dtype, f"marked at {at}, pages of {bs}")


def marked_window_model(tmp_path, dtype, window: int, keep: int):
    """One layer of two mixers side by side in which the left one looks: token 1 is marked by an axis of its own, which
    alone makes the keys' first element, and every query has a large first element.  The memory is closed (its
    output has weight zero)."""
    V, W = 50, 32
    left = dict(heads=2, kv_heads=1, dim=16, vdim=16, scale=0.6, conv=2, bias_max=30, buckets=8, window=window, keep_first=keep)
    right = dict(heads=1, kv_heads=1, dim=16, vdim=16, conv=2, a_rank=4, g_rank=4)
    cfg = make_config(vocab=V, width=W, layers=[("parallel", dict(left=left, right=right), None)], max_positions=1024)
    folder = str(tmp_path / f"w{window}_{keep}")
    kvforge_amd.write_random_model(folder, cfg, seed=5, dtype=NAME[dtype])
    path = os.path.join(folder, "model.safetensors")
    w = load_file(path)
    e = rand(V, W, seed=1, scale=0.3)
    e[:, 0] = 0.0
    e[:, 1] = 1.0
    e[1, 0] = 5.0
    q = torch.zeros(32, W)
    q[0, 1] = q[16, 1] = 1.0
    k = rand(16, W, seed=2, scale=0.05)
    k[0] = 0.0
    k[:, 0] = 0.0
    k[0, 0] = 1.0
    k[1, 1] = 1.0                       # the others' keys point elsewhere
    v = rand(16, W, seed=3, scale=0.1)
    v[:, 0] = rand(16, seed=4, scale=1.0)
    tap = lambda rows: torch.tensor([0.0, 1.0]).expand(rows, 2)  # noqa: E731
    new = {"embed": e, "l0.norm1": torch.zeros(W), "l0.mix.left.q": q, "l0.mix.left.k": k, "l0.mix.left.v": v,
           "l0.mix.left.q.conv": tap(32), "l0.mix.left.k.conv": tap(16), "l0.mix.left.v.conv": tap(16),
           "l0.mix.left.rel": rand(8, 2, seed=6, scale=0.5), "l0.mix.left.g": rand(2, W, seed=7, scale=0.1),
           "l0.mix.left.o": rand(W, 32, seed=8, scale=0.5), "l0.mix.left.out": torch.ones(W),
           "l0.mix.right.out": torch.zeros(W)}
    for key, t in new.items():
        assert w[key].shape == t.shape, key
        w[key] = t.to(w[key].dtype).contiguous()
    save_file(w, path, metadata={"format": "pt"})
    return folder, cfg, load_file(path)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window,keep", [(24, 5), (33, 0), (16, 16), (7, 20), (64, 3)])
def test_keys_just_inside_and_just_outside_the_window_and_its_kept_first_keys(tmp_path, dtype, window, keep):
    """The marked key is the last that a window holds, the first it has lost, the last kept one and the first
    that is not; read whole, in portions cut at the edge, and with the edge passing over decoded tokens."""
    folder, cfg, w = marked_window_model(tmp_path, dtype, window, keep)
    runner = make_runner(folder, dtype, block_size=8, num_blocks=40, tokens=300)
    g = torch.Generator().manual_seed(window)
    for at in sorted({0, max(keep - 1, 0), keep, keep + 1, 50}):
        n = at + window + 30
        toks = torch.randint(2, 50, (n,), generator=g).tolist()
        toks[at] = 1
        want = plain.forward(cfg, w, toks)
        blind = plain.forward(cfg, w, [t if i != at else 2 for i, t in enumerate(toks)])
        seen = (want - blind).abs().amax(1)
        spread = float(want.std())
        assert float(seen[at + window - 1]) > 0.1 * spread                   # the window's last
        if at >= keep:
            assert float(seen[at + window:].max()) < 1e-4 * spread            # and gone behind it
        else:
            assert float(seen[at + window]) > 0.1 * spread and float(seen[-1]) > 0.1 * spread
        for plan in ([[("x", 0, n)]], in_portions("x", n, (at + window, 2, 3)), in_portions("x", n, (at + 1, window - 1 or 1, 1, 5)),
                     [[("x", 0, at + 2)]] + [[("x", i, i + 1)] for i in range(at + 2, n)]):
            got = replay(runner, {"x": toks}, plan)["x"]
            check(got, cfg, w, toks, dtype, f"marked at {at}, window {window}, kept {keep}")


@pytest.mark.parametrize("dtype", DTYPES)
def test_memory_carries_a_token_from_the_far_past(tmp_path, dtype):
    """A model of memories that hardly fade and are hardly written to after the first tokens: what
    token 0 was still shows in the logits hundreds of tokens later, through portions and single
    tokens and through a slot that others have used."""
    par = dict(left=dict(heads=2, kv_heads=1, dim=16, vdim=16, scale=0.3, conv=3, bias_max=20, buckets=8, window=10),
               right=dict(heads=2, kv_heads=1, dim=32, vdim=16, conv=4, a_rank=4, g_rank=4))
    cfg = make_config(vocab=40, width=48, layers=[("parallel", par, None), ("parallel", par, (24, 2.0))], max_positions=512)
    folder = str(tmp_path / "m")
    kvforge_amd.write_random_model(folder, cfg, seed=6, dtype=NAME[dtype])
    liven(folder, cfg)
    path = os.path.join(folder, "model.safetensors")
    w = load_file(path)
    for k in list(w):
        if k.endswith(".A_log"):
            w[k] = torch.full_like(w[k], -9.0)
        elif k.endswith(".right.b"):                       # beta small, except under token 0's embedding
            w[k] = (w[k].float() * 0.0).to(w[k].dtype)
            w[k][:, 0] = 2.0
        elif k == "embed":
            w[k][:, 0] = -3.0
            w[k][0, 0] = w[k][1, 0] = 3.0
        elif k.endswith((".left.out", ".right.out", ".norm1", ".down.b")) or (k.endswith(".down") and ".mlp." in k):
            w[k][0] = 0.0
    save_file(w, path, metadata={"format": "pt"})
    w = load_file(path)
    runner = make_runner(folder, dtype, block_size=8, num_blocks=60, seqs=2, tokens=512)
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
        limit = rng.choice([0.5, 1.0, 3.0, 7.0])
        if kind == "none":
            return None
        if kind == "dense":
            return rng.choice([8, 24, 40, 64, 136]), limit
        experts = rng.choice([1, 2, 3, 5, 8, 12])
        return rng.choice([8, 16, 32, 40, 64]), limit, experts, rng.randint(1, min(experts, 4))

    layers = []
    for i in range(rng.randint(2, 5)):
        if rng.random() < 0.5:
            G = rng.choice([1, 2, 3])
            buckets = rng.choice([2, 4, 8, 16, 32])
            left = dict(heads=G * rng.choice([1, 2, 3, 5]), kv_heads=G, dim=rng.choice([4, 16, 20, 32, 48, 64]),
                        vdim=rng.choice([4, 12, 16, 40, 64]), scale=rng.choice([0.1, 0.25, 0.6]), conv=rng.choice([1, 2, 3, 4, 6, 8]),
                        bias_max=rng.choice([20, 47, 90, 400]), buckets=buckets)
            if rng.random() < 0.8:
                left.update(window=rng.choice([1, 5, 16, 23, 40]), keep_first=rng.choice([0, 1, 4, 9, 30]))
            kv = rng.choice([1, 2, 3])
            right = dict(heads=kv * rng.choice([1, 2, 3]), kv_heads=kv, dim=rng.choice([4, 16, 20, 32, 48, 64, 72, 136]),
                         vdim=rng.choice([8, 16, 24, 40, 64, 100]), conv=rng.choice([1, 2, 3, 4, 5, 8]),
                         a_rank=rng.choice([1, 5, 16, 24, 40]), g_rank=rng.choice([1, 5, 16, 24, 40]))
            layers.append(("parallel", dict(left=left, right=right), mlp()))
        else:
            m = dict(heads=rng.choice([1, 2, 3, 5, 8]), dim=rng.choice([0, 8, 16, 20, 32]), rot_dim=rng.choice([2, 8, 12, 16, 32]),
                     vdim=rng.choice([8, 16, 20, 32, 48]), q_rank=rng.choice([8, 20, 48, 100]), kv_rank=rng.choice([8, 16, 40, 96, 130]),
                     scale=rng.choice([0.05, 0.125, 0.3]), base=rng.choice([100.0, 10000.0, 1000000.0]))
            if rng.random() < 0.7:
                m["scaling"] = (rng.choice([1.5, 4.0, 16.0]), rng.choice([16, 100, 1024]), rng.choice([8.0, 32.0]),
                                rng.choice([0.5, 1.0, 2.0]))
            layers.append(("latent_attention", m, mlp()))
    return make_config(vocab=rng.choice([17, 64, 100, 257, 512]), width=width, layers=layers,
                       eps=rng.choice([1e-6, 1e-5, 1e-3, 0.1]), embed_scale=rng.choice([0.5, 1.0, 6.3, 11.0]),
                       residual_mult=rng.choice([0.3, 0.55, 1.0, 1.4]), logit_scale=rng.choice([0.25, 1.0, 3.0]), max_positions=256)


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


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["a", "c"])
def test_greedy_generation_through_the_engine(tmp_path_factory, name, dtype):
    """The framework's own entry point and scheduler: prompts admitted in portions under a small
    token budget, decode steps replayed from captured graphs (memories and convolutions advance on the
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
    assert engine.cache.slots.num_free == 3
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
    assert engine.cache.slots.num_free == 3


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
