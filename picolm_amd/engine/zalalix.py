"""The Zalalix decoder as a list of parts, and its entry in the architecture registry.

A scaled embedding; layers with an RMS norm ahead of each sublayer and one behind it, whose mixer is
lightning attention (a matrix state per head with a fixed decay, silu on queries, keys and values, one
norm over all heads behind a sigmoid gate), retention (the same state without the silu, every head of
unit RMS behind a silu gate), or two branches summed with a factor each: softmax attention over a window
and the first tokens (biases, a norm over all heads of q and of k, a partly turned head, capped scores,
one more in the softmax's denominator, a gate a head) and gated linear attention (a decay of the token's
own per key channel); a gated feed-forward or none; a head of its own."""
from __future__ import annotations

from ..config import register_architecture
from ..config.zalalix import ZalalixConfig
from ..parts import LMHead, RMSNorm, TokenEmbedding
from ..parts.block import SandwichBlock
from ..parts.feedforward import SwiGLU
from ..parts.parallel import ScaledParallelMixer
from ..parts.position import RotaryEmbedding
from ..parts.recurrent import LinearAttention
from ..parts.sink_attention import SinkAttention
from .model import DecoderModel


def _mixer(prefix: str, layer, D: int, eps: float, rotations: dict):
    m = layer.mixer
    if layer.kind == "lightning":
        return LinearAttention(prefix, D, m.heads, m.dim, m.vdim, eps, decay=m.decay, silu_qkv=True, norm="all", gate="sigmoid")
    if layer.kind == "retention":
        return LinearAttention(prefix, D, m.heads, m.dim, m.vdim, eps, decay=m.decay, k_scale=m.dim ** -0.5, norm_weight=False)
    l, r = m.left, m.right
    position = None
    if l.rot is not None:
        position = rotations.setdefault(l.rot, RotaryEmbedding(l.rot.dims, l.rot.base, l.rot.scaling, style="pairwise"))
    left = SinkAttention(prefix + "left.", D, l.heads, l.kv_heads, l.dim, l.vdim, l.scale, eps, sink=False, fixed_sink=0.0, proj_bias=True,
                         position=position, norm_all=True, softcap=l.softcap, window=l.window, keep_first=l.keep_first, gate_per_head=True,
                         out_bias=True)
    right = LinearAttention(prefix + "right.", D, r.heads, r.dim, r.vdim, eps, tau=r.tau, rank=r.rank, q_scale=r.dim ** -0.5)
    return ScaledParallelMixer(left, right, m.left_scale, m.right_scale, D)


def build_zalalix(cfg: ZalalixConfig) -> DecoderModel:
    D, eps = cfg.width, cfg.norm_eps
    rotations = {}                       # one set of tables for the layers that turn alike
    blocks = []
    for i, layer in enumerate(cfg.layers):
        p = f"l{i}."
        norm = lambda name: RMSNorm(p + name, D, eps)
        ffn = SwiGLU(p + "mlp.", D, layer.ff, names=("gate", "up", "down")) if layer.ff is not None else None
        blocks.append(SandwichBlock(norm("norm1"), _mixer(p + "mix.", layer, D, eps, rotations), norm("norm1b"),
                                    norm("norm2") if ffn else None, ffn, norm("norm2b") if ffn else None))
    emb = TokenEmbedding("embed", cfg.vocab, D, scale=cfg.embedding_scale)
    return DecoderModel(cfg, emb, blocks, RMSNorm("final.norm", D, eps), LMHead("head", cfg.vocab, D, emb, tied=False))


register_architecture("Zalalix", ZalalixConfig.from_dict, build_zalalix, replace=True)
