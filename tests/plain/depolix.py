"""A plain, slow Depolix decoder: whole sequences, no cache, no carried state, one function per
mechanism, torch on the CPU in 32-bit (or 64-bit, for a truth all but free of rounding).  It is
the oracle the engine's Depolix model is held to and shares no code with ``kvforge_amd``: it reads
``config.json`` dictionaries and ``{checkpoint name: tensor}`` dicts itself.

The design in this file's notation (``T`` tokens of one sequence, positions ``0..T-1``):

* stream ``x_t = a embed[token_t]`` with ``a = embedding.scale``;
* a layer: ``h = N1(x)``, ``x += m (mixer(h) + ff(h))`` with ``m = residual_mult`` (``ff`` may be missing);
  ``N1(y) = y / sqrt(mean(y^2) + eps) * (1 + w)``;
* mixer ``latent_attention``: the queries are read out of a normed latent of their own; keys and
  values of all heads out of one normed latent per token; one rotated key part that the heads share
  (halves turned against each other, frequencies stretched); the heads' outputs are gated
  element by element;
* mixer ``parallel``: ``(N(left(h)) + N'(right(h))) / 2``, norms over the width with plain weights.
  *left*: grouped attention whose q, k and v pass a short convolution first; q and k of every head
  are divided by their root mean square; scores get a learned bias by distance bucket; a window with
  kept first keys; one gate per head.  *right*: a matrix memory written by the delta rule whose key
  rows decay each by a gate of its own, behind short convolutions with silu;
* feed-forward: ``down(g sigmoid(1.702 g) (u + 1))`` with ``g = min(gate, L)``, ``u = clamp(up, -L, L)``, dense with
  biases on all three projections, or the ``top`` experts of largest router logit, weighted by the
  softmax over those logits;
* logits ``= logit_scale * head @ N(x)``.
"""

from __future__ import annotations

import math

import torch


def stored(x: torch.Tensor, store: torch.dtype | None) -> torch.Tensor:
    """``x`` after a trip through memory in type ``store`` (rounded and widened again), or
    unchanged for ``None``."""
    return x if store is None else x.to(store).to(x.dtype)


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """``x`` divided by its root mean square over the last axis, eps inside the root."""
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return rms(x, eps) * w


def one_plus_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return rms(x, eps) * (1.0 + w)


# ---------------------------------------------------------------------------------- convolution
def short_conv(x: torch.Tensor, taps: torch.Tensor) -> torch.Tensor:
    """``y_t[c] = sum_j taps[c, j] x_(t - (n - 1) + j)[c]`` for ``n`` taps; inputs before the first token are
    zeros."""
    n = taps.shape[1]
    before = torch.cat([x.new_zeros(n - 1, x.shape[1]), x])
    return torch.stack([(taps.T * before[t:t + n]).sum(0) for t in range(x.shape[0])])


def silu(x: torch.Tensor) -> torch.Tensor:
    return x / (1.0 + torch.exp(-x))


def softplus(z: torch.Tensor) -> torch.Tensor:
    return torch.logaddexp(z, torch.zeros_like(z))


def unit(x: torch.Tensor) -> torch.Tensor:
    return x / torch.sqrt(x.pow(2).sum(-1, keepdim=True) + 1e-6)


def of_group(x: torch.Tensor, heads: int) -> torch.Tensor:
    """``x [T, G, n]`` as ``[T, heads, n]``: head ``h`` gets group ``h // (heads / G)``'s."""
    return x.repeat_interleave(heads // x.shape[1], dim=1)


# ---------------------------------------------------------------------------------- rotation
def frequencies(rot: dict) -> tuple[torch.Tensor, float]:
    """(angle per position of every pair, what cosine and sine are multiplied by)."""
    d, base = int(rot["dims"]), float(rot["base"])
    f = [base ** (-2.0 * i / d) for i in range(d // 2)]
    s = rot.get("scaling")
    if not s:
        return torch.tensor(f, dtype=torch.float64), 1.0
    where = lambda turns: d * math.log(s["original"] / (2 * math.pi * turns)) / (2 * math.log(base))  # noqa: E731
    lo, hi = max(math.floor(where(s["fast"])), 0), min(math.ceil(where(s["slow"])), d - 1)
    out = []
    for i, fi in enumerate(f):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / s["factor"] * r + fi * (1.0 - r))
    return torch.tensor(out, dtype=torch.float64), 0.1 * math.log(s["factor"]) + 1.0


def turn_halves(x: torch.Tensor, rot: dict | None) -> torch.Tensor:
    """``x [T, heads, n]``: element ``i`` of the first ``dims`` turned against element ``i + dims / 2`` by the
    position's angle (formed in 32-bit)."""
    if not rot:
        return x
    half = int(rot["dims"]) // 2
    f, mag = frequencies(rot)
    a = torch.arange(x.shape[0], dtype=torch.float32)[:, None] * f.to(torch.float32)[None, :]
    cos, sin = ((t * mag).to(x.dtype)[:, None, :] for t in (a.cos(), a.sin()))
    u, v = x[..., :half], x[..., half:2 * half]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, x[..., 2 * half:]], dim=-1)


# ---------------------------------------------------------------------------------- attention
def softmax_rows(s: torch.Tensor, seen: torch.Tensor) -> torch.Tensor:
    s = s.masked_fill(~seen, float("-inf"))
    e = (s - s.max(-1, keepdim=True).values).exp()
    return e / e.sum(-1, keepdim=True)


def latent_mixer(h: torch.Tensor, w: dict, p: str, m: dict, eps: float, store: torch.dtype | None = None) -> torch.Tensor:
    """Keys and values are read out of every token's latent as the equations have it; nothing is
    taken through the queries."""
    T = h.shape[0]
    H, d, rot, dv, rank = (int(m[n]) for n in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
    cq = stored(norm(stored(h @ w[p + "dq"].T, store), w[p + "dq.norm"], eps), store)
    q = stored(cq @ w[p + "uq"].T, store).view(T, H, d + rot)
    qr = stored(turn_halves(q[..., d:], m.get("rot")), store)
    down = stored(h @ w[p + "dkv"].T, store)
    c = stored(norm(down[:, :rank], w[p + "dkv.norm"], eps), store)
    kr = stored(turn_halves(down[:, None, rank:], m.get("rot"))[:, 0], store)
    k, v = (c @ w[p + "uk"].T).view(T, H, d), (c @ w[p + "uv"].T).view(T, H, dv)
    seen = torch.arange(T)[:, None] >= torch.arange(T)[None, :]
    out = h.new_zeros(T, H, dv)
    for i in range(H):
        s = (q[:, i, :d] @ k[:, i].T + qr[:, i] @ kr.T) * float(m["scale"])
        out[:, i] = softmax_rows(s, seen) @ v[:, i]
    out = out.reshape(T, H * dv) * torch.sigmoid(stored(h @ w[p + "g"].T, store))
    return stored(out, store) @ w[p + "o"].T


def distance_bucket(n: int, buckets: int, far: float) -> int:
    half = buckets // 2
    if n < half:
        return n
    return min(buckets - 1, half + math.floor(math.log(n / half) / math.log(far / half) * (buckets - half)))


def distance_bias(table: torch.Tensor, T: int, far: float) -> torch.Tensor:
    """``[heads, T, T]``: what the score of key ``j`` for query ``i`` gets (zero above the diagonal)."""
    buckets, heads = table.shape
    rows = torch.tensor([distance_bucket(n, buckets, far) for n in range(T)])
    out = table.new_zeros(heads, T, T)
    for i in range(T):
        out[:, i, :i + 1] = table[rows[:i + 1].flip(0)].T
    return out


def window_mask(T: int, mask: dict | None) -> torch.Tensor:
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    seen = j <= i
    if mask:
        seen = seen & ((i - j < int(mask["size"])) | (j < int(mask.get("keep_first") or 0)))
    return seen


def bias_attention(h: torch.Tensor, w: dict, p: str, m: dict, eps: float, store: torch.dtype | None = None) -> torch.Tensor:
    T = h.shape[0]
    H, G, d, dv = (int(m[n]) for n in ("heads", "kv_heads", "dim", "vdim"))
    q, k, v = (short_conv(stored(h @ w[p + n].T, store), w[p + n + ".conv"]) for n in ("q", "k", "v"))
    q = stored(rms(q.view(T, H, d), eps), store)
    k = of_group(stored(rms(k.view(T, G, d), eps), store), H)
    v = of_group(stored(v, store).view(T, G, dv), H)
    bias, seen = distance_bias(w[p + "rel"], T, float(m["bias_max"])), window_mask(T, m.get("mask"))
    gate = torch.sigmoid(h @ w[p + "g"].T)
    out = h.new_zeros(T, H, dv)
    for i in range(H):
        out[:, i] = softmax_rows(q[:, i] @ k[:, i].T * float(m["scale"]) + bias[i], seen) @ v[:, i]
    out = out * gate[:, :, None]
    return stored(out.reshape(T, H * dv), store) @ w[p + "o"].T


# ---------------------------------------------------------------------------------- memory
def channel_delta_scan(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, g: torch.Tensor, beta: torch.Tensor
                       ) -> torch.Tensor:
    """``q, k, g [T, H, dk]``, ``v [T, H, dv]``, ``beta [T, H]``: every key row of ``S`` decays by its own ``g``,
    then the memory's answer to the key is brought towards the value."""
    T, H, dv = v.shape
    S = v.new_zeros(H, k.shape[2], dv)
    out = v.new_zeros(T, H, dv)
    for t in range(T):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out


def delta_mixer(h: torch.Tensor, w: dict, p: str, m: dict, eps: float, store: torch.dtype | None = None) -> torch.Tensor:
    T = h.shape[0]
    H, G, dk, dv = (int(m[n]) for n in ("heads", "kv_heads", "dim", "vdim"))
    q, k, v = (silu(short_conv(stored(h @ w[p + n].T, store), w[p + n + ".conv"])) for n in ("q", "k", "v"))
    q, k = of_group(unit(q.view(T, G, dk)) * dk ** -0.5, H), of_group(unit(k.view(T, G, dk)), H)
    beta = torch.sigmoid(h @ w[p + "b"].T)
    z = stored(h @ w[p + "a1"].T, store) @ w[p + "a2"].T + w[p + "dt_bias"]
    g = torch.exp(-torch.exp(w[p + "A_log"])[:, None] * softplus(z).view(T, H, dk))
    o = rms(channel_delta_scan(q, k, v.view(T, H, dv), g, beta), eps) * w[p + "norm"]
    gate = stored(stored(h @ w[p + "g1"].T, store) @ w[p + "g2"].T, store)
    return stored(o.reshape(T, H * dv) * torch.sigmoid(gate), store) @ w[p + "o"].T


def parallel_mixer(h: torch.Tensor, w: dict, p: str, m: dict, eps: float, store: torch.dtype | None = None) -> torch.Tensor:
    a = bias_attention(h, w, p + "left.", m["left"], eps, store)
    b = delta_mixer(h, w, p + "right.", m["right"], eps, store)
    return 0.5 * (norm(a, w[p + "left.out"], eps) + norm(b, w[p + "right.out"], eps))


# ---------------------------------------------------------------------------------- feed-forward
def limited_gate(g: torch.Tensor, u: torch.Tensor, limit: float) -> torch.Tensor:
    g, u = g.clamp(max=limit), u.clamp(-limit, limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1.0)


def dense_ff(h: torch.Tensor, w: dict, p: str, limit: float, store: torch.dtype | None = None) -> torch.Tensor:
    g, u = h @ w[p + "gate"].T + w[p + "gate.b"], h @ w[p + "up"].T + w[p + "up.b"]
    return stored(limited_gate(g, u, limit), store) @ w[p + "down"].T + w[p + "down.b"]


def routed_ff(h: torch.Tensor, w: dict, p: str, mlp: dict, store: torch.dtype | None = None) -> torch.Tensor:
    z = h @ w[p + "router"].T + w[p + "router.b"]
    limit, top = float(mlp["expert"]["limit"]), int(mlp["router"]["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        best = torch.topk(z[t], top)
        share = torch.softmax(best.values, dim=-1)
        for s, e in zip(share, best.indices.tolist()):
            pe, r = f"{p}e{e}.", h[t:t + 1]
            y = stored(limited_gate(r @ w[pe + "gate"].T, r @ w[pe + "up"].T, limit), store) @ w[pe + "down"].T
            out[t] += s * stored(y, store)[0]
    return out


# ---------------------------------------------------------------------------------- the model
MIXERS = {"latent_attention": latent_mixer, "parallel": parallel_mixer}


def forward(config: dict, weights: dict, tokens, dtype: torch.dtype = torch.float32,
            store: torch.dtype | None = None, layers_out: list | None = None) -> torch.Tensor:
    """Logits ``[T, vocab]`` of one whole sequence.  ``dtype``: the arithmetic (float32 or
    float64); ``store``: what an engine may keep in 16 bits between operations is rounded to
    this.  ``layers_out``: a list that receives the stream after every layer."""
    w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in weights.items()}
    eps, mult = float(config["norm"]["eps"]), float(config["residual_mult"])
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)] * float(config["embedding"]["scale"])
    for i, layer in enumerate(config["layers"]):
        p = f"l{i}."
        h = stored(one_plus_norm(x, w[p + "norm1"], eps), store)
        y = MIXERS[layer["type"]](h, w, p + "mix.", layer["mixer"], eps, store)
        mlp = layer.get("mlp")
        if mlp and mlp["kind"] == "dense":
            y = y + dense_ff(h, w, p + "mlp.", float(mlp["limit"]), store)
        elif mlp and mlp["kind"] == "moe":
            y = y + routed_ff(h, w, p + "mlp.", mlp, store)
        elif mlp:
            raise ValueError(f"unknown feed-forward {mlp['kind']!r}")
        x = x + mult * y
        if layers_out is not None:
            layers_out.append(x.clone())
    h = stored(one_plus_norm(x, w["final.norm"], eps), store)
    return h @ w["head"].T * float(config["logit_scale"])


def greedy(config: dict, weights: dict, prompt, n: int, dtype: torch.dtype = torch.float32) -> list[int]:
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(forward(config, weights, toks, dtype)[-1].argmax()))
    return toks[len(prompt):]
