"""``Balalorn``: how a Balalorn configuration becomes a list of parts.

A decoder in which every layer is described by itself in ``config.json``.  A layer is *post-norm*:
the sublayers read the residual stream as it is, and what they give joins it through a norm,
``x += N1(mixer(x))`` and, where the layer has a feed-forward, ``x += N2(ff(x))``, RMS norms with
plain weights.  The mixer is one of three.  *Mamba-2*: a matrix memory per head with one decay
per head and token behind a short convolution of its inputs, gated and then normalised in parts.
*Gated delta rule*: such a memory whose writes first take out what the memory already answers to
the key, over query/key heads that several memories share.  *Latent attention* with one sigmoid
gate per head, over one latent and one rotated key part per token; a layer may use an earlier
layer's (it then writes no cache of its own).  The feed-forward is dense and gated by silu, or a
layer of experts chosen by sigmoid scores that are multiplied into the experts' inputs.
Checkpoint names: ``embed``, ``l<i>.norm1``, ``l<i>.norm2``,
``l<i>.mix.{in,conv,conv.b,dt_bias,A_log,D,norm,o}`` (mamba2),
``l<i>.mix.{q,q.conv,k,k.conv,v,v.conv,b,a,A_log,dt_bias,g,norm,o}`` (delta),
``l<i>.mix.{q,dkv,dkv.norm,uk,uv,g,o}`` (latent attention), ``l<i>.mlp.{gate,up,down}`` (dense),
``l<i>.mlp.router``, ``l<i>.mlp.e<j>.{gate,up,down}`` (experts), ``final.norm``, ``head``.
"""

from __future__ import annotations

from kvforge_amd.config.balalorn import BalalornConfig
from kvforge_amd.config.rudorax import RotaryConfig
from kvforge_amd.parts.base import LayerCall, ModelSpec
from kvforge_amd.parts.embedding import LMHead, TokenEmbedding
from kvforge_amd.registry import (BLOCKS, FEED_FORWARDS, MIXERS, NORMS, POSITIONS, part_class,
                                  register_architecture)

FF_NAMES = {"gate": "gate", "up": "up", "down": "down"}


def build_balalorn(cfg: BalalornConfig) -> ModelSpec:
    norm_cls = part_class(NORMS, "rmsnorm_named", "norm")
    mamba_cls = part_class(MIXERS, "mamba2", "mixer")
    delta_cls = part_class(MIXERS, "gated_delta", "mixer")
    latent_cls = part_class(MIXERS, "latent_attention", "mixer")
    dense_cls = part_class(FEED_FORWARDS, "gated", "feed-forward")
    moe_cls = part_class(FEED_FORWARDS, "moe", "feed-forward")
    block_cls = part_class(BLOCKS, "post_norm", "block")
    rotary_cls = part_class(POSITIONS, "rotary", "position encoding")
    w, eps = cfg.width, cfg.norm_eps
    rotaries: dict[RotaryConfig, object] = {}    # layers with equal rotations share the tables

    def rotary_of(rot: RotaryConfig | None):
        if rot is None:
            return None
        if rot not in rotaries:
            rotaries[rot] = rotary_cls(rot.dims, rot.base, None, interleaved=True, rounded_once=True)
        return rotaries[rot]

    blocks, schedule = [], []
    for i, layer in enumerate(cfg.layers):
        p, m = f"l{i}", layer.mixer
        source = None
        if layer.type == "mamba2":
            mixer = mamba_cls(f"{p}.mix", w, m.heads, m.groups, m.state, m.vdim, m.conv, m.norm_groups, eps)
        elif layer.type == "delta":
            mixer = delta_cls(f"{p}.mix", w, m.heads, m.kv_heads, m.dim, m.vdim, m.conv, eps)
        else:
            source = m.kv_from
            mixer = latent_cls(f"{p}.mix", w, m.heads, m.dim, m.rot_dim, m.vdim, m.kv_rank, rotary_of(m.rot),
                               m.scale, eps, head_gate="g", own_kv=source is None)
        ffn = ffn_norm = None
        if layer.mlp is not None:
            f = layer.mlp
            if f.kind == "dense":
                ffn = dense_cls(f"{p}.mlp", w, f.ff, "silu", names=FF_NAMES)
            else:
                ffn = moe_cls(f"{p}.mlp", w, f.ff, f.experts, f.top, scores="sigmoid", renormalize=False,
                              correct=False, weigh_input=True)
            ffn_norm = norm_cls(f"{p}.norm2", w, eps)
        blocks.append(block_cls(mixer, norm_cls(f"{p}.norm1", w, eps), ffn, ffn_norm))
        # every layer runs once, so a layer's call has the layer's index
        schedule.append(LayerCall(i, cache_of=source))
    return ModelSpec(config=cfg, embedding=TokenEmbedding("", cfg.vocab_size, w, tensor="embed"),
                     blocks=blocks, final_norm=norm_cls("final.norm", w, eps),
                     head=LMHead("", cfg.vocab_size, w, tensor="head"), positions=list(rotaries.values()),
                     schedule=schedule)


register_architecture(BalalornConfig.NAME, BalalornConfig, build_balalorn)
