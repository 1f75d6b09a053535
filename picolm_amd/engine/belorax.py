"""The Belorax decoder as a list of parts, and its entry in the architecture registry.

A scaled embedding; layers whose sublayers read the residual rows themselves and pass a norm (weights
stored around nought) and a common factor before they join them; the mixer is retention (a matrix state
per head with a fixed decay, queries and keys turned by the position), softmax attention without
positions (a norm per query and key head, queries that grow with the position, some layers reading the
keys and values that an earlier layer cached), or attention over cached latents with a rotated key part
(YaRN-scaled); a dense gated feed-forward, routed experts weighed by their softmax scores as they are,
or none; a head of its own."""
from __future__ import annotations

from ..config import register_architecture
from ..config.belorax import BeloraxConfig
from ..parts import LMHead, RMSNorm, TokenEmbedding
from ..parts.block import OutputNormBlock
from ..parts.feedforward import RoutedExperts, SwiGLU
from ..parts.latent_attention import RotatedLatentAttention
from ..parts.position import RotaryEmbedding
from ..parts.recurrent import LinearAttention
from ..parts.sink_attention import SinkAttention
from ..weights import TensorSpec
from .begopel import _UnusedTensors
from .model import DecoderModel, LayerCall


def _mixer(prefix: str, layer, D: int, eps: float, rotation):
    m = layer.mixer
    if layer.kind == "retention":
        return LinearAttention(prefix, D, m.heads, m.dim, m.vdim, eps, decay=m.decay, k_scale=m.dim ** -0.5, norm_weight=False,
                               position=rotation(m.rot, "half"))
    if layer.kind == "attention":
        return SinkAttention(prefix, D, m.heads, m.kv_heads, m.dim, m.vdim, m.scale, eps, sink=False, gate=False, q_temp=m.q_temp,
                             reads_keys=m.kv_from is not None)
    return RotatedLatentAttention(prefix, D, m.heads, m.dim, m.rot_dim, m.vdim, m.kv_rank, m.scale, eps, rotation(m.rot, "pairwise"), gate=False)


def _feed_forward(prefix: str, mlp, D: int):
    if mlp.kind == "dense":
        return SwiGLU(prefix, D, mlp.ff, names=("gate", "up", "down"))
    return RoutedExperts(prefix, D, mlp.experts, mlp.top, mlp.ff, scoring="softmax_kept", bias_name=None)


def build_belorax(cfg: BeloraxConfig) -> DecoderModel:
    D, eps = cfg.width, cfg.norm_eps
    tables = {}                          # one set of tables for the layers that turn alike

    def rotation(rot, style: str):
        if rot is None:
            return None
        return tables.setdefault((rot, style), RotaryEmbedding(rot.dims, rot.base, rot.scaling, style=style))
    norm = lambda name: RMSNorm(name, D, eps, weight_offset=1.0)
    blocks, order, unused = [], [], []
    for i, layer in enumerate(cfg.layers):
        p = f"l{i}."
        ffn = _feed_forward(p + "mlp.", layer.mlp, D) if layer.mlp is not None else None
        if ffn is None:
            unused.append(TensorSpec(p + "norm2", (D,), optional=True, init=None))
        blocks.append(OutputNormBlock(_mixer(p + "mix.", layer, D, eps, rotation), norm(p + "norm1"), ffn, norm(p + "norm2") if ffn else None,
                                      cfg.residual_mult))
        order.append(LayerCall(i, reads_cache_of=layer.mixer.kv_from))
    emb = TokenEmbedding("embed", cfg.vocab, D, scale=cfg.embedding_scale)
    model = DecoderModel(cfg, emb, blocks, norm("final.norm"), LMHead("head", cfg.vocab, D, emb, tied=False), order)
    model.extra_parts = [_UnusedTensors(unused)]
    return model


register_architecture("Belorax", BeloraxConfig.from_dict, build_belorax, replace=True)
