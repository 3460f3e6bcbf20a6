"""Sibodra: a decoder whose layers are listed in config.json, pre-norm (layer norms without a bias) on a residual of
several rows a token: every sub-layer reads a learned weighted sum of the rows and the rows are mixed by a learned matrix
when its result joins them (hyper-connections).  The mixer is soft-capped attention with normed and rotated queries and
keys, one added to the softmax's denominator and a gate a head, or attention through latents of queries and of keys and
values with a gate a feature; the feed-forward is a gated one, or a mixture of experts without gates weighed by the softmax
over the chosen logits, beside a shared one.  The head has a matrix of its own and its logits are soft-capped.

Checkpoint names: ``embed``, ``l<i>.norm1|norm2``, ``l<i>.hc1|hc2.in|out|mix``, ``l<i>.mix.*``, ``l<i>.mlp.*``, ``final.norm``, ``head``.
"""
from __future__ import annotations

import torch

from ..config.model_config import CappedAttentionSpec, QueryLatentAttentionSpec, SibodraConfig
from ..config.registry import register_architecture
from ..parts import (Embedding, HyperConnectedBlock, LMHead, LatentAttention, LayerNorm, MoEFeedForward, RotaryEmbedding,
                     StreamsNorm, SwiGLUMLP, WindowAttention)
from .decoder import DecoderModel


def build_sibodra(cfg: SibodraConfig) -> DecoderModel:
    width, eps, streams = cfg.hidden_size, cfg.norm_eps, cfg.streams
    rotations = {}

    def rotation(size, m):
        key = (size, m.rot_base, m.rot_dims, m.rot_scaling)
        if key not in rotations:
            rotations[key] = RotaryEmbedding(size, m.rot_base, scaling=m.rot_scaling, rot_dim=m.rot_dims)
        return rotations[key]

    norm = lambda: LayerNorm(width, eps, weight_name="", bias_name=None)
    layers = []
    for i, layer in enumerate(cfg.layers):
        m, f = layer.mixer, layer.mlp
        if isinstance(m, CappedAttentionSpec):
            mixer = WindowAttention(width, m.heads, m.kv_heads, m.dim, m.vdim, m.scale, qk_norm_eps=eps, pos_enc=rotation(m.dim, m),
                                    sink_score=0.0, softcap=m.softcap, head_gate=True)
        elif isinstance(m, QueryLatentAttentionSpec):
            mixer = LatentAttention(width, m.heads, m.dim, m.rot_dim, m.vdim, m.kv_rank, m.scale, eps, pos_enc=rotation(m.rot_dim, m),
                                    interleaved=False, q_rank=m.q_rank, output_gate=True)
        else:
            raise TypeError(f"layer {i}: unknown mixer {m!r}")
        ffn = None
        if f is not None and f.kind == "dense":
            ffn = SwiGLUMLP(width, f.ff, names={"gate": "gate", "up": "up", "down": "down"}, delta_dtype=torch.float32)
        elif f is not None:
            ffn = MoEFeedForward(width, f.ff, f.experts, f.top, score="chosen_softmax", router_bias=True, gated=False, shared_size=f.shared_ff)
        layers.append(HyperConnectedBlock(width, streams, norm(), mixer, norm() if ffn is not None else None, ffn))
    embed = Embedding(cfg.vocab_size, width, weight_name="")
    head = LMHead(cfg.vocab_size, width, softcap=cfg.logit_softcap or 0.0, weight_name="")
    return DecoderModel(cfg, embed, layers, StreamsNorm(norm(), streams), head, position_encodings=list(rotations.values()),
                        names={"embed": "embed", "layer": "l{i}", "final_norm": "final.norm", "lm_head": "head"})


register_architecture("Sibodra", SibodraConfig, build_sibodra)
