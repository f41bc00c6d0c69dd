"""A plain, slow Balalorn decoder: whole sequences, no cache, no carried state, one function per
mechanism, torch on the CPU in 32-bit (or 64-bit, for a truth all but free of rounding).  It is
the oracle the engine's Balalorn model is held to and shares no code with ``kvforge_amd``: it
reads ``config.json`` dictionaries and ``{checkpoint name: tensor}`` dicts itself.

The design in this file's notation (``T`` tokens of one sequence, positions ``0..T-1``):

* stream ``x_t = embed[token_t]``;
* a layer: ``x += N1(mixer(x))``, then, where the layer has a feed-forward, ``x += N2(ff(x))``: the
  sublayers read the stream itself, ``N(y) = y / sqrt(mean(y^2) + eps) * w`` is taken of what
  they give;
* mixer ``mamba2``: one projection into ``z``, ``x``, ``B``, ``C``, ``dt``; x, B and C through a short
  causal convolution with bias and silu; per head a matrix ``S [state, vdim]`` with
  ``S_t = exp(-exp(A) dt_t) S_(t-1) + dt_t B_t x_t^T``, ``y_t = S_t^T C_t + D x_t``; gated by
  ``silu(z)``, then normalised in equal parts of the row;
* mixer ``delta``: q, k, v through a short causal convolution and silu, q and k made unit vectors;
  ``S <- g_t S``, ``S <- S + k_t (beta_t (v_t - S^T k_t))^T``, ``o_t = S^T q_t``; head norm with a
  weight, silu gate;
* mixer ``latent_attention``: keys and values of all heads read out of one latent per token, one
  rotated key part shared by the heads, one sigmoid gate per head; a layer may use an earlier
  layer's latents and rotated key parts (``kv_from``);
* feed-forward ``dense``: ``W_down (silu(W_gate x) * W_up x)``; ``moe``: the ``top`` experts of largest
  ``s = sigmoid(W_r x)``, each applied to ``s x``;
* logits ``= head @ N(x)``.
"""

from __future__ import annotations

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


def silu(x: torch.Tensor) -> torch.Tensor:
    return x / (1.0 + torch.exp(-x))


# ---------------------------------------------------------------------------------- convolution
def short_conv(x: torch.Tensor, taps: torch.Tensor, bias: torch.Tensor | None) -> torch.Tensor:
    """``y_t[c] = silu(sum_j taps[c, j] x_(t - (n - 1) + j)[c] + bias[c])`` for ``n`` taps, the last of
    which meets the token itself; inputs before the first token are zeros."""
    n = taps.shape[1]
    before = torch.cat([x.new_zeros(n - 1, x.shape[1]), x])
    y = torch.stack([(taps.T * before[t:t + n]).sum(0) for t in range(x.shape[0])])
    if bias is not None:
        y = y + bias
    return silu(y)


def unit(x: torch.Tensor) -> torch.Tensor:
    return x / torch.sqrt(x.pow(2).sum(-1, keepdim=True) + 1e-6)


# ---------------------------------------------------------------------------------- memories
def of_group(x: torch.Tensor, heads: int) -> torch.Tensor:
    """``x [T, G, n]`` as ``[T, heads, n]``: head ``h`` gets group ``h // (heads / G)``'s."""
    return x.repeat_interleave(heads // x.shape[1], dim=1)


def delta_scan(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, g: torch.Tensor, beta: torch.Tensor) -> torch.Tensor:
    """``q, k [T, G, dk]`` (head ``h`` uses ``h // (H / G)``), ``v [T, H, dv]``, ``g, beta [T, H]``."""
    T, H, dv = v.shape
    q, k = of_group(q, H), of_group(k, H)
    S = v.new_zeros(H, q.shape[2], dv)
    out = v.new_zeros(T, H, dv)
    for t in range(T):
        S = g[t][:, None, None] * S
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out


def ssd_scan(C: torch.Tensor, B: torch.Tensor, x: torch.Tensor, a: torch.Tensor, dt: torch.Tensor) -> torch.Tensor:
    """``C, B [T, G, N]`` (head ``h`` uses group ``h // (H / G)``), ``x [T, H, dv]``, decays ``a`` and
    step sizes ``dt [T, H]``: ``S_t = a_t S_(t-1) + dt_t B_t x_t^T``, ``y_t = S_t^T C_t``."""
    T, H, dv = x.shape
    B, C = of_group(B, H), of_group(C, H)
    S = x.new_zeros(H, B.shape[2], dv)
    out = x.new_zeros(T, H, dv)
    for t in range(T):
        S = a[t][:, None, None] * S + dt[t][:, None, None] * B[t][:, :, None] * x[t][:, None, :]
        out[t] = (S * C[t][:, :, None]).sum(1)
    return out


def softplus(z: torch.Tensor) -> torch.Tensor:
    return torch.logaddexp(z, torch.zeros_like(z))


def delta_mixer(h: torch.Tensor, w: dict, p: str, m: dict, eps: float, store: torch.dtype | None = None) -> torch.Tensor:
    T = h.shape[0]
    H, G, dk, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    q, k, v = (short_conv(stored(h @ w[p + n].T, store), w[p + n + ".conv"], None) for n in ("q", "k", "v"))
    q = unit(q.view(T, G, dk)) * dk ** -0.5
    k = unit(k.view(T, G, dk))
    beta = torch.sigmoid(h @ w[p + "b"].T)
    g = torch.exp(-torch.exp(w[p + "A_log"]) * softplus(h @ w[p + "a"].T + w[p + "dt_bias"]))
    o = rms(delta_scan(q, k, v.view(T, H, dv), g, beta), eps) * w[p + "norm"]
    y = o.reshape(T, H * dv) * silu(stored(h @ w[p + "g"].T, store))
    return stored(y, store) @ w[p + "o"].T


def mamba2_mixer(h: torch.Tensor, w: dict, p: str, m: dict, eps: float, store: torch.dtype | None = None) -> torch.Tensor:
    T = h.shape[0]
    H, dv, N, G = int(m["heads"]), int(m["vdim"]), int(m["state"]), int(m["groups"])
    inner, gn = H * dv, G * N
    rows = h @ w[p + "in"].T
    z, xbc = stored(rows[:, :inner], store), stored(rows[:, inner:2 * inner + 2 * gn], store)
    dt = softplus(rows[:, 2 * inner + 2 * gn:] + w[p + "dt_bias"])
    xbc = short_conv(xbc, w[p + "conv"], w[p + "conv.b"])
    x = xbc[:, :inner].reshape(T, H, dv)
    B, C = xbc[:, inner:inner + gn].reshape(T, G, N), xbc[:, inner + gn:].reshape(T, G, N)
    y = ssd_scan(C, B, x, torch.exp(-torch.exp(w[p + "A_log"]) * dt), dt) + w[p + "D"][:, None] * x
    y = y.reshape(T, inner) * silu(z)
    parts = int(m["norm_groups"])
    y = rms(y.view(T, parts, inner // parts), eps).reshape(T, inner) * w[p + "norm"]
    return stored(y, store) @ w[p + "o"].T


# ---------------------------------------------------------------------------------- latent attention
def turn(x: torch.Tensor, positions: torch.Tensor, dims: int, base: float) -> torch.Tensor:
    """``x [T, heads, dim]``: pairs ``(2i, 2i+1)`` of the first ``dims`` elements of every head turned
    by the angle ``position * base^(-2i/dims)`` (formed in 32-bit)."""
    i = torch.arange(dims // 2, dtype=torch.float64)
    f = base ** (-2.0 * i / dims)
    a = positions.to(torch.float32)[:, None] * f.to(torch.float32)[None, :]
    cos, sin = a.cos().to(x.dtype)[:, None, :], a.sin().to(x.dtype)[:, None, :]
    out = x.clone()
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2] = u * cos - v * sin
    out[..., 1:dims:2] = v * cos + u * sin
    return out


def latents(h: torch.Tensor, w: dict, p: str, m: dict, eps: float, store: torch.dtype | None = None
            ) -> tuple[torch.Tensor, torch.Tensor]:
    """(latents ``c [T, kv_rank]``, rotated key parts ``[T, rot_dim]``): all that later tokens, and a
    later layer that uses this one's, need of a token."""
    rank, rot = int(m["kv_rank"]), int(m["rot_dim"])
    rows = stored(h @ w[p + "dkv"].T, store)
    c = stored(norm(rows[:, :rank], w[p + "dkv.norm"], eps), store)
    kr = rows[:, rank:rank + rot]
    r = m["rot"]
    kr = turn(kr[:, None, :], torch.arange(h.shape[0]), int(r["dims"]), float(r["base"]))[:, 0]
    return c, stored(kr, store)


def latent_mixer(h: torch.Tensor, w: dict, p: str, m: dict, c: torch.Tensor, kr: torch.Tensor,
                 store: torch.dtype | None = None) -> torch.Tensor:
    """Keys and values are read out of every token's latent as the equations have it; nothing is
    taken through the queries."""
    T = h.shape[0]
    H, d, rot, dv = int(m["heads"]), int(m["dim"]), int(m["rot_dim"]), int(m["vdim"])
    r = m["rot"]
    q = stored(h @ w[p + "q"].T, store).view(T, H, d + rot)
    qr = stored(turn(q[..., d:], torch.arange(T), int(r["dims"]), float(r["base"])), store)
    k = (c @ w[p + "uk"].T).view(T, H, d)
    v = (c @ w[p + "uv"].T).view(T, H, dv)
    gate = torch.sigmoid(h @ w[p + "g"].T)
    mask = torch.arange(T)[:, None] >= torch.arange(T)[None, :]
    out = h.new_zeros(T, H, dv)
    for i in range(H):
        s = (q[:, i, :d] @ k[:, i].T + qr[:, i] @ kr.T) * float(m["scale"])
        s = s.masked_fill(~mask, float("-inf"))
        e = (s - s.max(-1, keepdim=True).values).exp()
        out[:, i] = (e / e.sum(-1, keepdim=True)) @ v[:, i]
    out = out * gate[:, :, None]
    return stored(out, store).reshape(T, H * dv) @ w[p + "o"].T


# ---------------------------------------------------------------------------------- feed-forward
def gated_ff(h: torch.Tensor, w: dict, p: str, store: torch.dtype | None = None) -> torch.Tensor:
    g, u = h @ w[p + "gate"].T, h @ w[p + "up"].T
    return stored(silu(g) * u, store) @ w[p + "down"].T


def routed_ff(h: torch.Tensor, w: dict, p: str, mlp: dict, store: torch.dtype | None = None) -> torch.Tensor:
    """Every chosen expert reads its weight times the token's row."""
    s = torch.sigmoid(h @ w[p + "router"].T)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e in torch.topk(s[t], int(mlp["router"]["top"])).indices.tolist():
            out[t] += stored(gated_ff(s[t, e] * h[t:t + 1], w, f"{p}e{e}.", store)[0], store)
    return out


# ---------------------------------------------------------------------------------- the model
def forward(config: dict, weights: dict, tokens, dtype: torch.dtype = torch.float32,
            store: torch.dtype | None = None, layers_out: list | None = None) -> torch.Tensor:
    """Logits ``[T, vocab]`` of one whole sequence.  ``dtype``: the arithmetic (float32 or
    float64); ``store``: what an engine may keep in 16 bits between operations is rounded to
    this.  ``layers_out``: a list that receives the stream after every layer."""
    w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in weights.items()}
    eps = float(config["norm"]["eps"])
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    x = w["embed"][tokens]
    kept: dict[int, tuple[torch.Tensor, torch.Tensor]] = {}
    for i, layer in enumerate(config["layers"]):
        p = f"l{i}."
        h = stored(x, store)
        kind, m = layer["type"], layer["mixer"]
        if kind == "mamba2":
            y = mamba2_mixer(h, w, p + "mix.", m, eps, store)
        elif kind == "delta":
            y = delta_mixer(h, w, p + "mix.", m, eps, store)
        elif kind == "latent_attention":
            if m.get("kv_from") is None:
                kept[i] = latents(h, w, p + "mix.", m, eps, store)
            y = latent_mixer(h, w, p + "mix.", m, *kept[i if m.get("kv_from") is None else int(m["kv_from"])], store)
        else:
            raise ValueError(f"unknown layer type {kind!r}")
        x = x + norm(y, w[p + "norm1"], eps)
        mlp = layer.get("mlp")
        if mlp:
            h = stored(x, store)
            if mlp["kind"] == "dense":
                y = gated_ff(h, w, p + "mlp.", store)
            elif mlp["kind"] == "moe":
                y = routed_ff(h, w, p + "mlp.", mlp, store)
            else:
                raise ValueError(f"unknown feed-forward {mlp['kind']!r}")
            x = x + norm(y, w[p + "norm2"], eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    h = stored(norm(x, w["final.norm"], eps), store)
    return h @ w["head"].T


def greedy(config: dict, weights: dict, prompt, n: int, dtype: torch.dtype = torch.float32) -> list[int]:
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(forward(config, weights, toks, dtype)[-1].argmax()))
    return toks[len(prompt):]
