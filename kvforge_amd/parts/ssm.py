"""State-space layers: matrix memories with one decay per head and token behind a short causal
convolution, as mixers with per-request state.

Per head a memory ``S [dk, dv]`` that starts at zero; for a token with rows ``q, k`` (heads that
several memories may share) and ``v``, a step ``dt = softplus(z_a + dt_bias)`` and the decay
``a = exp(-exp(A_log) dt)``::

    Mamba2        S <- a S + dt k v^T;                              y = S^T q + D v
    GatedDelta    S <- a S;   S <- S + k (beta (v - S^T k))^T;      o = S^T q       (beta = sigmoid(z_b))
    ChannelDelta  the same with one decay per key channel, S <- diag(a) S

q, k and v pass a convolution over the last few tokens, channel by channel, and silu.  A request's
state slot holds every head's ``S`` and the convolution's last inputs in fp32, so that a prompt may
be cut anywhere.  The projections and the rows the convolution reads are in the engine's type;
the pre-activations of steps, decays and gates of the recurrence are products with fp32 sums
stored in fp32, and everything between them and the memory's read-out is fp32 in every mode.
"""

from __future__ import annotations

import torch

from kvforge_amd.kernels import ops
from kvforge_amd.parts.base import LayerState, Mixer, StateSpec, WeightSpec, add_product
from kvforge_amd.registry import register_mixer


def _padded_rows(w: torch.Tensor) -> torch.Tensor:
    """``w`` with zero rows up to a multiple of 16, which every product kernel takes."""
    pad = -w.shape[0] % 16
    return torch.cat([w, w.new_zeros(pad, w.shape[1])], dim=0).contiguous() if pad else w.contiguous()


def _one_type(mats: list[torch.Tensor]) -> list[torch.Tensor]:
    return mats if len({m.dtype for m in mats}) == 1 else [m.float() for m in mats]


class ConvMemory(Mixer):
    """What the two mixers share: two projections (``w_rows`` in the engine's type, ``w_gates`` stored
    in fp32), convolution, memory, output projection.  A subclass fills in the weights
    (``load``), where the channels and q, k, v lie (``conv_col``, ``channels``, ``q_off``, ``k_off``, ``v_off``),
    the gates' columns (``a_off``, ``b_off``) and what becomes of the read-out (``finish``)."""

    replayable = True
    shares_slot = True
    cache_spec = None

    b_off: int | None = None     # column of the delta rule's gates, ``None`` for plain writes
    unit = 0                     # how many of the first channels are q and k heads made unit vectors
    q_scale = 1.0
    chunk_from = ops.SSM_CHUNK_FROM   # runs of at least so many tokens go chunk by chunk

    def _sizes(self, prefix: str, hidden: int, heads: int, key_heads: int, key_dim: int, value_dim: int, taps: int,
               channels: int, norm_eps: float) -> None:
        self.prefix, self.hidden = prefix, int(hidden)
        self.H, self.G, self.dk, self.dv = int(heads), int(key_heads), int(key_dim), int(value_dim)
        self.taps, self.channels, self.norm_eps = int(taps), int(channels), float(norm_eps)
        if min(self.H, self.G, self.dk, self.dv) <= 0 or self.H % self.G or self.dk > 256:
            raise ValueError(f"state-space kernels take key heads of up to 256 elements that divide the heads, got "
                             f"{heads} heads over {key_heads}, {key_dim} x {value_dim}")
        if not 1 <= self.taps <= ops.SSM_MAX_TAPS:
            raise ValueError(f"convolutions of 1 to {ops.SSM_MAX_TAPS} taps, got {taps}")
        self.state_off = self.H * self.dk * self.dv
        self.state_spec = StateSpec((ops.ssm_state_floats(self.H, self.dk, self.dv, self.channels, self.taps),),
                                    torch.float32)
        self.w_rows = self.w_gates = self.w_o = self.conv_w = self.conv_b = None
        self.neg_a = self.dt_bias = self.skip = self.norm_w = None

    def _take_gates(self, tensors: dict[str, torch.Tensor]) -> None:
        t = lambda key: tensors[self._name(self.names[key])].float()  # noqa: E731
        self.neg_a = (-torch.exp(t("A_log"))).contiguous()
        self.dt_bias = t("dt_bias").contiguous()
        self.norm_w = t("norm").contiguous()
        self.w_o = tensors[self._name(self.names["o"])]

    def seal(self) -> None:
        self.w_rows, self.w_gates, self.w_o = (ops.streamed(ops.plain_of(w)) for w in (self.w_rows, self.w_gates, self.w_o))

    def kernel_modules(self, dtype: torch.dtype) -> set[str]:
        return {"ssm", "elementwise", "gemm_generic"} | ({"gemm_bf16"} if dtype == torch.bfloat16 else set())

    def _matrices(self) -> list:
        return [w for w in (self.w_rows, self.w_gates, self.w_o) if w is not None]

    def _small(self) -> list[torch.Tensor]:
        return [x for x in (self.conv_w, self.conv_b, self.neg_a, self.dt_bias, self.skip, self.norm_w) if x is not None]

    def num_bytes(self) -> int:
        return sum(x.numel() * x.element_size() for x in (*map(ops.plain_of, self._matrices()), *self._small()))

    def held_tensors(self) -> list[torch.Tensor]:
        return [c for w in self._matrices() for c in ops.copies_of(w)] + self._small()

    def _long_runs(self, step) -> dict | None:
        """Chunk and run tables of this step's long runs (made once per step, shared by the layers
        whose chunks are equally long) and scratch from the step's workspace.  ``None`` when no run
        is that long."""
        key = ("ssm.long_runs", ops.ssm_chunk_len(self.dk), self.chunk_from)
        plan = step.scratch.get(key)
        if plan is None:
            chunks, runs = ops.ssm_plan(step.q_lens, self.dk, self.chunk_from)
            plan = (step.upload_ints(chunks).view(-1, 4), step.upload_ints(runs).view(-1, 3)) if chunks else ()
            step.scratch[key] = plan
        if not plan:
            return None
        out = {"chunks": plan[0], "runs": plan[1]}
        for name, (shape, dtype) in self._chunk_scratch(step.n_tokens, plan[0].shape[0]).items():
            out[name] = step.ws.buf("ssm_" + name, shape, dtype)
        return out

    def _chunk_scratch(self, n_tokens: int, n_chunks: int) -> dict[str, tuple]:
        return ops.ssm_scratch(n_tokens, n_chunks, self.H, self.dk, self.dv, self.b_off is not None)

    def forward(self, x, step, layer: LayerState, residual) -> None:
        """``x``: the mixer's input rows in the step's activation type."""
        if layer.state is None:
            raise RuntimeError("a state-space mixer needs a state slot per request")
        n = x.shape[0]
        ws, act = step.ws, step.act_dtype
        step.settle()
        rows = ws.buf("ssm_rows", (n, self.w_rows.shape[0]), act)
        ops.gemm(x, self.w_rows, rows)
        gates = ws.buf("ssm_gates", (n, self.w_gates.shape[0]), torch.float32)
        ops.gemm(x, self.w_gates, gates)            # 32-bit sums, stored so
        mixed = ws.buf("ssm_mixed", (n, self.channels), torch.float32)
        ops.ssm_conv(rows, self.conv_col, self.conv_w, self.conv_b, step.cu_q, step.positions, step.slot_ids,
                     layer.state, self.state_off, mixed, step.n_seqs, max(step.q_lens), unit=self.unit,
                     key_dim=self.dk, q_scale=self.q_scale)
        raw = ws.buf("ssm_raw", (n, self.H * self.dv), torch.float32)
        gate_rows = self.scan(mixed, rows, gates, raw, step, layer)
        heads = ws.buf("ssm_heads", (n, self.H * self.dv), act)
        self.finish(raw, gate_rows, heads)
        add_product(step, heads, self.w_o, residual)

    def scan(self, mixed, rows, gates, raw, step, layer: LayerState) -> torch.Tensor:
        """``raw``: the memories' read-out (fp32), from the convolved rows ``mixed`` and what the two projections
        gave (``rows``, ``gates``).  Returns the rows that hold the output gate, for ``finish``."""
        # which kernels have work is known from the runs' lengths (all ones in a captured step of
        # single tokens, so a replay launches what the capture launched)
        ops.ssm_scan(mixed, self.q_off, self.k_off, self.v_off, gates, self.a_off, self.b_off, self.neg_a, self.dt_bias,
                     self.skip, step.cu_q, step.positions, step.slot_ids, layer.state, raw, step.n_seqs, self.H, self.G,
                     self.dk, self.dv, multi=self._long_runs(step),
                     short_runs=any(q < ops.SSM_CHUNK_FROM for q in step.q_lens))
        return rows

    def finish(self, raw: torch.Tensor, rows: torch.Tensor, heads: torch.Tensor) -> None:
        """``heads``: what the output projection reads, from the memories' read-out ``raw`` (fp32) and the rows that
        ``scan`` returned."""
        raise NotImplementedError


@register_mixer("mamba2")
class Mamba2(ConvMemory):
    """``key_heads``: groups that share B and C (what the memory is written under and read with);
    ``key_dim``: their size.  The input projection's rows are ``z | x | B | C | dt``.  The read-out is
    multiplied by ``silu(z)`` and then normalised in ``norm_parts`` equal parts of the row.  ``names``:
    checkpoint names under the prefix, by ``in conv conv_b dt_bias A_log D norm o``."""

    NAMES = {"in": "in", "conv": "conv", "conv_b": "conv.b", "dt_bias": "dt_bias", "A_log": "A_log", "D": "D",
             "norm": "norm", "o": "o"}

    def __init__(self, prefix: str, hidden: int, heads: int, key_heads: int, key_dim: int, value_dim: int, taps: int,
                 norm_parts: int, norm_eps: float, names: dict[str, str] | None = None) -> None:
        self.inner, gn = int(heads) * int(value_dim), int(key_heads) * int(key_dim)
        self._sizes(prefix, hidden, heads, key_heads, key_dim, value_dim, taps, self.inner + 2 * gn, norm_eps)
        self.norm_parts = int(norm_parts)
        if self.norm_parts <= 0 or self.inner % self.norm_parts:
            raise ValueError(f"rows of {self.inner} do not fall into {norm_parts} equal parts")
        self.conv_col = self.inner                      # behind z
        self.v_off, self.k_off, self.q_off = 0, self.inner, self.inner + gn
        self.a_off = 0
        self.names = dict(self.NAMES, **(names or {}))

    def weight_specs(self) -> dict[str, WeightSpec]:
        h, H, C = self.hidden, self.H, self.channels
        n = lambda key: self._name(self.names[key])  # noqa: E731
        return {n("in"): WeightSpec((self.inner + C + H, h)), n("conv"): WeightSpec((C, self.taps), std=0.3),
                n("conv_b"): WeightSpec((C,), std=0.1), n("dt_bias"): WeightSpec((H,), std=1.0),
                n("A_log"): WeightSpec((H,), std=0.5), n("D"): WeightSpec((H,), init="norm", std=0.3),
                n("norm"): WeightSpec((self.inner,), init="norm", std=0.1), n("o"): WeightSpec((h, self.inner))}

    def load(self, tensors: dict[str, torch.Tensor]) -> None:
        t = lambda key: tensors[self._name(self.names[key])]  # noqa: E731
        split = self.inner + self.channels
        self.w_rows, self.w_gates = _padded_rows(t("in")[:split]), _padded_rows(t("in")[split:])
        self.conv_w, self.conv_b = t("conv").float().contiguous(), t("conv_b").float().contiguous()
        self.skip = t("D").float().contiguous()
        self._take_gates(tensors)

    def finish(self, raw, rows, heads) -> None:
        ops.ssm_gate_norm(raw, rows[:, :self.inner], self.norm_w, self.norm_eps, self.norm_parts, heads)


@register_mixer("gated_delta")
class GatedDelta(ConvMemory):
    """``key_heads`` query/key heads of ``key_dim`` elements, made unit vectors behind the convolution
    (q also times ``key_dim^(-1/2)``).  Every memory's read-out is divided by its root mean square,
    multiplied by a weight ``[value_dim]`` that the heads share and by ``silu(W_g x)``.  ``names``:
    checkpoint names under the prefix, by ``q k v g b a A_log dt_bias norm o`` and ``conv`` (a format
    with ``{of}``, the name of the projection it follows)."""

    NAMES = {"q": "q", "k": "k", "v": "v", "g": "g", "b": "b", "a": "a", "A_log": "A_log", "dt_bias": "dt_bias",
             "norm": "norm", "o": "o", "conv": "{of}.conv"}

    def __init__(self, prefix: str, hidden: int, heads: int, key_heads: int, key_dim: int, value_dim: int, taps: int,
                 norm_eps: float, names: dict[str, str] | None = None) -> None:
        Q = int(key_heads) * int(key_dim)
        self._sizes(prefix, hidden, heads, key_heads, key_dim, value_dim, taps, 2 * Q + int(heads) * int(value_dim),
                    norm_eps)
        self.conv_col, self.q_off, self.k_off, self.v_off = 0, 0, Q, 2 * Q
        self.unit, self.q_scale = 2 * Q, float(key_dim) ** -0.5
        self.a_off, self.b_off = 0, self.H
        self.names = dict(self.NAMES, **(names or {}))

    def _conv(self, key: str) -> str:
        return self._name(self.names["conv"].format(of=self.names[key]))

    def weight_specs(self) -> dict[str, WeightSpec]:
        h, H, Q, V = self.hidden, self.H, self.G * self.dk, self.H * self.dv
        n = lambda key: self._name(self.names[key])  # noqa: E731
        out = {n("o"): WeightSpec((h, V)), n("g"): WeightSpec((V, h)), n("b"): WeightSpec((H, h)),
               n("a"): WeightSpec((H, h)), n("A_log"): WeightSpec((H,), std=0.5), n("dt_bias"): WeightSpec((H,), std=1.0),
               n("norm"): WeightSpec((self.dv,), init="norm", std=0.1)}
        for key, rows in (("q", Q), ("k", Q), ("v", V)):
            out[n(key)] = WeightSpec((rows, h))
            out[self._conv(key)] = WeightSpec((rows, self.taps), std=0.3)
        return out

    def load(self, tensors: dict[str, torch.Tensor]) -> None:
        t = lambda key: tensors[self._name(self.names[key])]  # noqa: E731
        # one product for q, k, v and the output gate: their heads side by side in that order
        self.w_rows = _padded_rows(torch.cat(_one_type([t(k) for k in ("q", "k", "v", "g")]), dim=0))
        self.w_gates = _padded_rows(torch.cat(_one_type([t("a"), t("b")]), dim=0))
        self.conv_w = torch.cat([tensors[self._conv(k)].float() for k in ("q", "k", "v")], dim=0).contiguous()
        self._take_gates(tensors)

    def kernel_modules(self, dtype: torch.dtype) -> set[str]:
        return super().kernel_modules(dtype) | {"linmem"}

    def finish(self, raw, rows, heads) -> None:
        V = self.H * self.dv
        ops.linmem_out(raw, rows[:, self.channels:self.channels + V], self.norm_w, self.norm_eps, heads, self.H, self.dv)


@register_mixer("channel_delta")
class ChannelDelta(GatedDelta):
    """The gated delta rule with a decay per head and key channel and gates of low rank.  Channel ``i`` of
    head ``h`` decays by ``exp(-exp(A_log[h]) softplus((W_a2 W_a1 x)[h, i] + dt_bias[h, i]))``.  Every memory's read-out
    is divided by its root mean square, multiplied by a weight ``[value_dim]`` that the heads share and by
    ``sigmoid(W_g2 W_g1 x)``, element by element.  ``a_rank``, ``g_rank``: the ranks (``None``: the checkpoint's).
    ``names``: checkpoint names under the prefix, by ``q k v b a1 a2 g1 g2 A_log dt_bias norm o`` and ``conv``.

    One product holds q, k, v and the two low-rank rows, a second (over ``[W_a1 x | W_g1 x]``, the two second
    matrices as diagonal blocks) the pre-activations of decays and output gate, with fp32 sums stored in fp32."""

    NAMES = {"q": "q", "k": "k", "v": "v", "b": "b", "a1": "a1", "a2": "a2", "g1": "g1", "g2": "g2", "A_log": "A_log",
             "dt_bias": "dt_bias", "norm": "norm", "o": "o", "conv": "{of}.conv"}

    def __init__(self, prefix: str, hidden: int, heads: int, key_heads: int, key_dim: int, value_dim: int, taps: int,
                 norm_eps: float, names: dict[str, str] | None = None, a_rank: int | None = None,
                 g_rank: int | None = None) -> None:
        super().__init__(prefix, hidden, heads, key_heads, key_dim, value_dim, taps, norm_eps, names)
        self.a_rank, self.g_rank = a_rank, g_rank
        self.b_off = 0
        self.w_low2 = None
        self.low = self.low2 = None      # columns of the low-rank rows in the first product, width of the second's input

    def weight_specs(self) -> dict[str, WeightSpec]:
        h, H, Q, V, K = self.hidden, self.H, self.G * self.dk, self.H * self.dv, self.H * self.dk
        n = lambda key: self._name(self.names[key])  # noqa: E731
        out = {n("o"): WeightSpec((h, V)), n("b"): WeightSpec((H, h)), n("A_log"): WeightSpec((H,), std=0.5),
               n("dt_bias"): WeightSpec((K,), std=1.0), n("norm"): WeightSpec((self.dv,), init="norm", std=0.1),
               n("a1"): WeightSpec((self.a_rank, h)), n("a2"): WeightSpec((K, self.a_rank)),
               n("g1"): WeightSpec((self.g_rank, h)), n("g2"): WeightSpec((V, self.g_rank))}
        for key, rows in (("q", Q), ("k", Q), ("v", V)):
            out[n(key)] = WeightSpec((rows, h))
            out[self._conv(key)] = WeightSpec((rows, self.taps), std=0.3)
        return out

    def load(self, tensors: dict[str, torch.Tensor]) -> None:
        t = lambda key: tensors[self._name(self.names[key])]  # noqa: E731
        a1, a2, g1, g2 = _one_type([t(k) for k in ("a1", "a2", "g1", "g2")])
        ra, rg = int(a1.shape[0]), int(g1.shape[0])
        for first, second, rank, want in (("a1", a2, ra, self.a_rank), ("g1", g2, rg, self.g_rank)):
            if second.shape[1] != rank or rank <= 0 or (want is not None and rank != want):
                raise ValueError(f"{self._name(self.names[first])} and the matrix behind it do not agree on their rank")
        pa, pg = -(-ra // 16) * 16, -(-rg // 16) * 16     # ranks as every product kernel takes them
        rows = _one_type([t(k) for k in ("q", "k", "v")] + [a1, g1])
        lead = rows[0].new_zeros(-self.channels % 16, self.hidden)      # the low-rank rows start on 16 bytes
        self.low = self.channels + lead.shape[0]
        self.low2 = pa + pg
        pad = lambda w, n: torch.cat([w, w.new_zeros(n - w.shape[0], w.shape[1])], dim=0)  # noqa: E731
        self.w_rows = torch.cat([*rows[:3], lead, pad(rows[3], pa), pad(rows[4], pg)], dim=0).contiguous()
        K, V = self.H * self.dk, self.H * self.dv
        second = a2.new_zeros(-(-(K + V) // 16) * 16, pa + pg)
        second[:K, :ra], second[K:K + V, pa:pa + rg] = a2, g2
        self.w_low2 = second
        self.w_gates = _padded_rows(t("b"))
        self.conv_w = torch.cat([tensors[self._conv(k)].float() for k in ("q", "k", "v")], dim=0).contiguous()
        self._take_gates(tensors)

    def seal(self) -> None:
        super().seal()
        self.w_low2 = ops.streamed(ops.plain_of(self.w_low2))

    def kernel_modules(self, dtype: torch.dtype) -> set[str]:
        return super().kernel_modules(dtype) | {"chdelta"}

    def _matrices(self) -> list:
        return super()._matrices() + ([self.w_low2] if self.w_low2 is not None else [])

    chunk_from = ops.CHDELTA_CHUNK_FROM

    def _chunk_scratch(self, n_tokens: int, n_chunks: int) -> dict[str, tuple]:
        return ops.chdelta_scratch(n_tokens, n_chunks, self.H, self.dk, self.dv)

    def scan(self, mixed, rows, gates, raw, step, layer: LayerState) -> torch.Tensor:
        n = rows.shape[0]
        low = step.ws.buf("chdelta_gates", (n, self.w_low2.shape[0]), torch.float32)
        ops.gemm(rows[:, self.low:self.low + self.low2], self.w_low2, low)     # 32-bit sums, stored so
        ops.chdelta_scan(mixed, self.q_off, self.k_off, self.v_off, low, 0, gates, self.b_off, self.neg_a, self.dt_bias,
                         step.cu_q, step.positions, step.slot_ids, layer.state, raw, step.n_seqs, self.H, self.G,
                         self.dk, self.dv, multi=self._long_runs(step),
                         short_runs=any(q < ops.CHDELTA_CHUNK_FROM for q in step.q_lens))
        return low[:, self.H * self.dk:self.H * (self.dk + self.dv)]

    def finish(self, raw, rows, heads) -> None:
        ops.linmem_out(raw, rows, self.norm_w, self.norm_eps, heads, self.H, self.dv, sigmoid=True)
