"""Rigodra: a decoder of softmax attention layers, grouped-query or latent, with feed-forwards without a gate and a layer
norm of the whole sum behind each branch, assembled from config.json layer by layer.

* embedding rows behind a layer norm (parts/embedding.py); the head is the embedding table;
* every layer x = norm1(alpha x + mixer(x)), then x = norm2(alpha x + ff(x)) where it has a feed-forward; the norms are layer
  norms with weight and bias (parts/block.py:SumNormBlock);
* 'attention' layers: per-head norms of queries and keys with shared weights, rotation on split halves of a head's leading
  elements, a sliding window that keeps the sequence's first tokens in sight, values mixed with those of the first
  layer that says so, one gate number per head (parts/attention.py);
* 'latent_attention' layers: attention over one latent row per token, queries through a latent of their own, rotation on
  split halves, a sliding window (parts/latent_attention.py);
* feed-forwards: dense, down(gelu(up h)), or routed, down(relu(up h)^2): picks are the largest of softmax + correction over
  experts and identity experts together, among the groups with the largest single values, weighted by the softmax
  values as they are; an identity expert returns the input; plus a shared expert;
* a last layer norm, then the head.

Tensor names: ``embed``, ``embed.norm``, ``l<i>.norm1|norm2`` (+ ``.b``), ``l<i>.mix.{q,k,v,q.norm,k.norm,vmix,g,o}``,
``l<i>.mix.{dq,dq.norm,uq,dkv,dkv.norm,uk,uv,o}``, ``l<i>.mlp.{up,down}``,
``l<i>.mlp.{router,correction,e<j>.{up,down},shared.{up,down}}``, ``final.norm`` (+ ``.b``).
"""
from __future__ import annotations

from ..cache.spec import WINDOW_NONE, WINDOW_SLIDING
from ..config.rigodra import RigodraConfig, UngatedMlpConfig
from ..parts.attention import Attention
from ..parts.block import SumNormBlock
from ..parts.embedding import NormedEmbedding
from ..parts.feedforward import DenseMLP, MoESwiGLU
from ..parts.latent_attention import LatentAttention
from ..parts.model import DecoderModel
from ..parts.norm import LayerNorm
from ..parts.position import Rotary
from ..registry import register_architecture

BLOCK_NAMES = {"norm1": "norm1", "mixer": "mix.", "norm2": "norm2", "ffn": "mlp."}
ATTENTION_NAMES = {"q": "q", "k": "k", "v": "v", "o": "o", "q_norm": "q.norm", "k_norm": "k.norm", "g": "g", "v_mix": "vmix"}
MOE_NAMES = {"router": "router", "correction": "correction", "up": "e{e}.up", "down": "e{e}.down", "shared": "shared.",
             "shared_up": "up", "shared_down": "down"}
DENSE_ACTIVATION, EXPERT_ACTIVATION = "gelu", "relu2"
GROUP_TOP = 1                  # a group of experts ranks by its largest choice score


def _feed_forward(width: int, f: UngatedMlpConfig):
    if f.kind == "dense":
        return DenseMLP(width, f.ff, DENSE_ACTIVATION, names={"up": "up", "down": "down"})
    return MoESwiGLU(width, f.experts, f.top, f.ff, shared_intermediate=f.shared_ff or None, gate="softmax", renormalise=False,
                     score_on_input=False, activation=EXPERT_ACTIVATION, correction=True, n_groups=f.groups, keep_groups=f.keep,
                     names=MOE_NAMES, gated=False, identity=f.identity, group_top=GROUP_TOP)


def build_rigodra(cfg: RigodraConfig) -> DecoderModel:
    cfg.validate()
    W, eps = cfg.width, cfg.norm_eps
    blocks, values_shared = [], False
    for layer in cfg.layers:
        m = layer.mixer
        window = dict(window_kind=WINDOW_SLIDING if m.window else WINDOW_NONE, window=m.window or 0)
        rotary = None
        if m.rot is not None:
            rotary = Rotary(m.dim if layer.type == "attention" else m.rot_dim, m.rot.base, None, "half", m.rot.dims)
        if layer.type == "attention":
            mix = None
            if m.v_mix:
                mix, values_shared = "mixed" if values_shared else "source", True
            mixer = Attention(W, m.heads, m.kv_heads, m.dim, rotary=rotary, qk_norm_eps=eps, scale=m.scale, v_head_dim=m.vdim,
                              qk_norm_weights="head", names=ATTENTION_NAMES, head_gate=True, keep_first=m.keep_first, value_mix=mix,
                              **window)
        else:
            mixer = LatentAttention(W, m.heads, m.dim, m.rot_dim, m.vdim, m.kv_rank, rotary, eps, m.scale, sink=False, gate=False,
                                    q_rank=m.q_rank, **window)
        ffn = _feed_forward(W, layer.mlp) if layer.mlp is not None else None
        blocks.append(SumNormBlock(LayerNorm(W, eps, name=""), mixer, LayerNorm(W, eps, name="") if ffn else None, ffn, cfg.alpha,
                                   names=BLOCK_NAMES))
    return DecoderModel(cfg.vocab_size, W, blocks, LayerNorm(W, eps, name=""), tie_embeddings=True, config=cfg, layer_prefix="l",
                        embed_name="embed", norm_prefix="final.norm", embedding=NormedEmbedding(LayerNorm(W, eps, name="embed.norm")))


register_architecture("Rigodra", RigodraConfig, build_rigodra)
