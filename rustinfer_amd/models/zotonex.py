"""Zotonex: a decoder whose layers are listed in config.json, pre-norm, ``x <- x + mixer(norm1(x));
x <- x + ff(norm2(x))``.  The mixer makes each head from the difference of two softmax maps over one set of
values, with normed queries and keys, no rotation, inside chunks of positions (a layer may read the keys and
values of an earlier one, through a chunk size of its own); the feed-forward is a mixture of clipped gated experts
on weighted inputs with a gated shared expert, or absent.  Embedded rows and logits are scaled; the head has
its own matrix.

Checkpoint names: ``embed``, ``l<i>.norm1|norm2``, ``l<i>.mix.*``, ``l<i>.mlp.*``, ``final.norm``, ``head``.
"""
from __future__ import annotations

from ..config.model_config import DifferenceAttentionSpec, ZotonexConfig
from ..config.registry import register_architecture
from ..parts import Embedding, LMHead, MoEFeedForward, PreNormBlock, RMSNorm, WindowAttention
from .decoder import DecoderModel, LayerCall

BLOCK_NAMES = {"mixer_norm": "norm1", "mixer": "mix", "ffn_norm": "norm2", "ffn": "mlp"}


def build_zotonex(cfg: ZotonexConfig) -> DecoderModel:
    width, eps = cfg.hidden_size, cfg.norm_eps
    layers, schedule = [], []
    for i, layer in enumerate(cfg.layers):
        m, f = layer.mixer, layer.mlp
        if not isinstance(m, DifferenceAttentionSpec):
            raise TypeError(f"layer {i}: unknown mixer {m!r}")
        mixer = WindowAttention(width, m.heads, m.kv_heads, m.dim, m.vdim, m.scale, qk_norm_eps=eps, own_kv=m.kv_from is None,
                                chunk=m.chunk, difference=m.diff, difference_eps=eps)
        ffn = ffn_norm = None
        if f is not None:
            ffn = MoEFeedForward(width, f.ff, f.experts, f.top, score="sigmoid", weigh_input=True, limit=f.limit,
                                 shared_size=f.shared_ff, shared_gate=f.shared_ff > 0, shared_limit=f.shared_limit)
            ffn_norm = RMSNorm(width, eps, weight_name="")
        layers.append(PreNormBlock(width, RMSNorm(width, eps, weight_name=""), mixer, ffn_norm, ffn, names=BLOCK_NAMES))
        reads = i if m.kv_from is None else m.kv_from       # the cache this layer's call uses
        schedule.append(LayerCall(i, cache=reads, write=reads == i))
    embed = Embedding(cfg.vocab_size, width, weight_name="", scale=cfg.embedding_scale)
    head = LMHead(cfg.vocab_size, width, weight_name="", logit_scale=cfg.logit_scale)
    return DecoderModel(cfg, embed, layers, RMSNorm(width, eps, weight_name=""), head, schedule=schedule,
                        names={"embed": "embed", "layer": "l{i}", "final_norm": "final.norm", "lm_head": "head"})


register_architecture("Zotonex", ZotonexConfig, build_zotonex)
