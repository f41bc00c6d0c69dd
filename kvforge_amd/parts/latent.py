"""Latent attention: keys and values of all heads are read out of one small latent vector per
token, which (with one rotated key part that the heads share) is all the cache holds.

For a token with input ``x``: ``q = W_q x`` (or ``q = W_uq norm(W_dq x)``, queries read out of a latent of their
own) holds per head ``dim`` plain and ``rot_dim`` rotated
elements; ``W_dkv x`` holds the latent ``c`` (``kv_rank`` elements, RMS-normed with a weight) and
the shared key part ``k_r`` (``rot_dim`` elements, rotated like the queries' part).  Head ``h``
scores a key as ``(q_h . W_uk_h c + q_r_h . k_r) * scale`` and its value is ``W_uv_h c``.

Because ``q_h . (W_uk_h c) = (W_uk_h^T q_h) . c``, the read-outs never touch the keys: the
queries are taken through ``W_uk_h^T`` once (``ops.head_product``), attention runs with ONE
key/value head over pages of ``[k_r | c]`` (the built-in paged kernels, window and sink
included), and the weighted sums of ``c`` are read out per head by ``W_uv_h`` before the output
projection.  A page row is ``rot_dim + kv_rank`` elements (rounded up to the kernels' step of
16) whatever the number of heads; rows of more than 256 elements (up to 640) take the fp32 attention
kernels in either mode.
"""

from __future__ import annotations

import torch

from kvforge_amd.kernels import ops
from kvforge_amd.parts.attention import PagedAttention
from kvforge_amd.parts.base import CacheSpec, LayerState, WeightSpec, add_product, attention_pages
from kvforge_amd.parts.positions import RotaryPositions
from kvforge_amd.registry import register_mixer


@register_mixer("latent_attention")
class LatentAttention(PagedAttention):
    """``names``: checkpoint names under the prefix, by ``q dkv dkv_norm uk uv o`` (and ``dq dq_norm uq g``).
    ``q_rank``: the queries go through a latent of so many elements, RMS-normed with a weight: ``W_dq``,
    its norm and ``W_uq`` take the place of ``W_q``.  ``gated``: the heads' outputs are multiplied by
    ``sigmoid(W_g x)`` element by element where the values are read out (instead of ``head_gate``).
    ``out_scale``: a constant on the heads' outputs, applied there as well.  ``own_kv=False``:
    the mixer has no ``dkv`` and uses the latents and rotated key parts that another call's pages
    hold (of equal ``kv_rank``, ``rot_dim`` and rotation).  ``head_gate``: checkpoint name of a matrix
    ``[heads, hidden]``; head ``h``'s output is multiplied by ``sigmoid(W_g x)_h`` where the values are
    read out.  ``rotary``:
    the rotation of the ``rot_dim`` parts (its width must be ``rot_dim`` at most); where it turns halves against
    each other, the rows of queries and key part are permuted once so that its pairs are neighbours.  ``window``,
    ``sink``, ``scale``: as in ``PagedAttention``, whose launch planning and kernels this
    mixer uses with one kv head of ``rot_dim + kv_rank`` elements."""

    LATENT_NAMES = {"q": "q", "dkv": "dkv", "dkv_norm": "dkv.norm", "uk": "uk", "uv": "uv", "o": "o", "dq": "dq",
                    "dq_norm": "dq.norm", "uq": "uq", "g": "g"}

    replayable = True
    settles_residual = False

    def __init__(self, prefix: str, hidden: int, num_heads: int, head_dim: int, rot_dim: int,
                 value_dim: int, kv_rank: int, rotary: RotaryPositions | None, scale: float,
                 norm_eps: float, window: int | None = None, sink: str | None = None,
                 names: dict[str, str] | None = None, head_gate: str | None = None, own_kv: bool = True,
                 q_rank: int | None = None, gated: bool = False, out_scale: float = 1.0) -> None:
        self.prefix, self.hidden, self.H, self.KV = prefix, int(hidden), int(num_heads), 1
        self.dim, self.rot, self.dv_out, self.rank = int(head_dim), int(rot_dim), int(value_dim), int(kv_rank)
        if min(self.H, self.dv_out, self.rank) <= 0 or self.dim < 0 or self.rot < 0 or self.dim + self.rot <= 0:
            raise ValueError(f"latent attention: sizes must be positive, got heads {num_heads}, "
                             f"{head_dim} + {rot_dim}, values {value_dim}, rank {kv_rank}")
        self.d = -(-(self.rot + self.rank) // 16) * 16
        if self.d > ops.ATTENTION_MAX_HEAD:
            raise ValueError(f"attention kernels take heads up to {ops.ATTENTION_MAX_HEAD} elements; rot_dim + "
                             f"kv_rank is {self.rot + self.rank}")
        self.dk = self.dv = self.d
        self.rotary = rotary
        if rotary is not None and rotary.rot_dim > self.rot:
            raise ValueError("latent attention rotates pairs within its rot_dim part")
        self.q_rank = int(q_rank) if q_rank is not None else None
        if self.q_rank is not None and self.q_rank <= 0:
            raise ValueError(f"q_rank must be positive, got {q_rank}")
        if gated and head_gate is not None:
            raise ValueError("latent attention has a gate per element or one per head, not both")
        self.elem_gate, self.out_scale = bool(gated), float(out_scale)
        self.scale, self.norm_eps_c = float(scale), float(norm_eps)
        if not self.scale > 0.0:
            raise ValueError(f"scale must be positive, got {scale}")
        self.window, self.chunk = int(window) if window else None, None
        self.keep_first = 0
        self.names = dict(self.LATENT_NAMES, **(names or {}))
        self.sink, self.head_gate = sink, head_gate
        self.gated, self.own_kv, self.qk_norm = False, bool(own_kv), None
        self.score_slopes = self.slopes = self.sinks = None
        self.score_cap = self.q_temp = None
        self.conv = self.dist = self.conv_w = self.row_norm = None
        self.cache_spec = CacheSpec(attention_pages(1, self.d), self.window, 0)
        self.w_in = self.w_uq = self.w_uk_t = self.w_uv = self.w_o = self.c_norm_w = self.cq_norm_w = None

    def weight_specs(self) -> dict[str, WeightSpec]:
        h, H = self.hidden, self.H
        n = lambda key: self._name(self.names[key])  # noqa: E731
        q_rows = H * (self.dim + self.rot)
        if self.q_rank is None:
            out = {n("q"): WeightSpec((q_rows, h))}
        else:
            out = {n("dq"): WeightSpec((self.q_rank, h)), n("dq_norm"): WeightSpec((self.q_rank,), init="norm", std=0.1),
                   n("uq"): WeightSpec((q_rows, self.q_rank))}
        if self.elem_gate:
            out[n("g")] = WeightSpec((H * self.dv_out, h))
        out.update({n("uk"): WeightSpec((H * self.dim, self.rank)),
               n("uv"): WeightSpec((H * self.dv_out, self.rank)),
               n("o"): WeightSpec((h, H * self.dv_out))})
        if self.own_kv:
            out[n("dkv")] = WeightSpec((self.rank + self.rot, h))
            out[n("dkv_norm")] = WeightSpec((self.rank,), init="norm", std=0.1)
        if self.head_gate is not None:
            out[self._name(self.head_gate)] = WeightSpec((H, h))
        if self.sink is not None:
            out[self._name(self.sink)] = WeightSpec((H,), std=1.0)
        return out

    def load(self, tensors: dict[str, torch.Tensor]) -> None:
        t = lambda key: tensors[self._name(self.names[key])]  # noqa: E731
        # rows of the rotated parts in the kernels' order (neighbouring pairs)
        perm = self.pair_permutation()

        def turned(w: torch.Tensor, heads: int, before: int) -> torch.Tensor:
            w = w.view(heads, before + self.rot, -1)
            return torch.cat([w[:, :before], w[:, before:][:, perm.to(w.device)]], dim=1).reshape(
                heads * (before + self.rot), -1)
        q = turned(t("q" if self.q_rank is None else "uq"), self.H, self.dim)
        if self.q_rank is not None:
            self.w_uq, q = q.contiguous(), t("dq")
            self.cq_norm_w = t("dq_norm").float().contiguous()
        mats = [q] + ([turned(t("dkv"), 1, self.rank)] if self.own_kv else [])
        # one product for the queries, the latent, the shared key part and the heads' gates (their
        # rows padded with zero rows, so that the product's rows start on 16 bytes)
        self.down_col = int(q.shape[0])
        self.gate_col = sum(int(m.shape[0]) for m in mats)
        if self.elem_gate:
            # (zero rows ahead of the gate's, so that its rows start on 16 bytes)
            lead = -self.gate_col % 8
            self.gate_col += lead
            g = t("g")
            mats += [g.new_zeros(lead, self.hidden), g, g.new_zeros(-(self.gate_col + g.shape[0]) % 16, self.hidden)]
        if self.head_gate is not None:
            g = tensors[self._name(self.head_gate)]
            mats += [g, g.new_zeros(-(self.gate_col + self.H) % 16, self.hidden)]
        if len({m.dtype for m in mats}) > 1:
            mats = [m.float() for m in mats]
        self.w_in = torch.cat(mats, dim=0).contiguous()
        # the queries go through the keys' read-out transposed: [H, rank, dim]
        self.w_uk_t = t("uk").view(self.H, self.dim, self.rank).transpose(1, 2).contiguous()
        self.w_uv = t("uv").view(self.H, self.dv_out, self.rank).contiguous()
        self.w_o = t("o")
        if self.own_kv:
            self.c_norm_w = t("dkv_norm").float().contiguous()
        if self.sink is not None:
            self.sinks = tensors[self._name(self.sink)].float().contiguous()

    def pair_permutation(self) -> torch.Tensor:
        """``perm[new] = old`` within a rotated part: a rotation of halves has its pairs moved next to each other."""
        perm = torch.arange(self.rot)
        if self.rotary is not None and not self.rotary.interleaved:
            half = self.rotary.rot_dim // 2
            for i in range(half):
                perm[2 * i], perm[2 * i + 1] = i, i + half
        return perm

    def absorb_norm(self, norm) -> bool:
        return False

    def seal(self) -> None:
        if self.w_uq is not None:
            self.w_uq = ops.streamed(ops.plain_of(self.w_uq))
        self.w_in, self.w_o = ops.streamed(ops.plain_of(self.w_in)), ops.streamed(ops.plain_of(self.w_o))

    def kernel_modules(self, dtype: torch.dtype) -> set[str]:
        return super().kernel_modules(dtype) | {"latent"}

    def _small(self) -> list[torch.Tensor]:
        return [x for x in (self.w_uk_t, self.w_uv, self.c_norm_w, self.cq_norm_w, self.sinks) if x is not None]

    def num_bytes(self) -> int:
        return sum(x.numel() * x.element_size()
                   for x in (*map(ops.plain_of, (self.w_in, self.w_uq, self.w_o)), *self._small()) if x is not None)

    def held_tensors(self) -> list[torch.Tensor]:
        return ops.copies_of(self.w_in) + ops.copies_of(self.w_uq) + ops.copies_of(self.w_o) + self._small()

    def forward(self, x, step, layer: LayerState, residual) -> None:
        """``x``: normalised activations."""
        n = x.shape[0]
        H, d, dim, rot, rank = self.H, self.d, self.dim, self.rot, self.rank
        ws, act = step.ws, step.act_dtype
        table = step.block_tables[layer.group]
        cos, sin = (self.rotary.cos, self.rotary.sin) if self.rotary is not None else (None, None)
        step.settle()
        proj = ws.buf("latent_proj", (n, self.w_in.shape[0]), act)
        ops.gemm(x, self.w_in, proj)
        qkv = ws.buf("latent_qkv", (n, (H + (2 if self.own_kv else 0)) * d), act)
        q, down = proj[:, :H * (dim + rot)], proj[:, self.down_col:]
        if self.q_rank is not None:
            cq = ws.buf("latent_cq", (n, self.q_rank), act)
            ops.latent_norm(proj[:, :self.q_rank], self.cq_norm_w, self.norm_eps_c, cq)
            q = ws.buf("latent_q", (n, H * (dim + rot)), act)
            ops.gemm(cq, self.w_uq, q)
        ops.latent_split(q, qkv, self.c_norm_w, self.norm_eps_c, H, dim, rot, rank, d, down=down)
        if dim:
            # q_h -> W_uk_h^T q_h, next to the head's rotated part
            ops.head_product(q, dim + rot, self.w_uk_t, qkv[:, rot:H * d], d)
        ops.rope_kvwrite(qkv, step.positions, step.seq_of_token, cos, sin, table, layer.k_pages,
                         layer.v_pages, H, 1, d, write_kv=layer.owns_cache and self.own_kv)
        out = ws.buf("attn_out", (n, H * d), act)
        bs = layer.k_pages.shape[2]
        work, rows_per_item = self._prefill_work(step, act, bs)
        window = self.window or 0
        if work is not None:
            ops.attn_prefill(qkv, layer.k_pages, layer.v_pages, table, step.cu_q, step.ctx_lens, work,
                             out, H, 1, d, self.scale, window, None, rows_per_item, sinks=self.sinks)
        if step.n_decode:
            splits = self._decode_cuts(step, ops.attention_on_matrix_cores(act, bs, d))
            workspace = None
            if splits > 1:
                workspace = (ws.buf("decode_part_acc", (step.n_decode * H * splits * d,), torch.float32),
                             ws.buf("decode_part_ml", (step.n_decode * H * splits * 2,), torch.float32))
            ops.attn_decode(qkv, layer.k_pages, layer.v_pages, table, step.decode_seq_ids, step.n_decode,
                            step.cu_q, step.ctx_lens, out, H, 1, d, self.scale, window, splits, workspace,
                            token_is_seq=step.decode_seq_ids is None and work is None, sinks=self.sinks)
        # the heads' weighted sums of the latent, read out by W_uv_h
        heads = ws.buf("latent_heads", (n, H * self.dv_out), act)
        gate = None
        if self.elem_gate:
            gate = proj[:, self.gate_col:self.gate_col + H * self.dv_out]
        elif self.head_gate is not None:
            gate = proj[:, self.gate_col:self.gate_col + H]
        ops.head_product(out[:, rot:], d, self.w_uv, heads, self.dv_out, gate=gate, gate_outputs=self.elem_gate,
                         scale=self.out_scale)
        add_product(step, heads, self.w_o, residual)
