"""Pagonex: a decoder whose layers hold the gated delta rule or latent attention, each followed by a routed
clamped feed-forward, with layer norms on the branches' outputs and short convolutions in front of them,
assembled from config.json layer by layer.

* embedding rows plus a row of a second table chosen by the previous and the current token (parts/embedding.py);
* every layer x += norm1(mixer(c1(x))), then x += norm2(ff(c2(x))) where it has a feed-forward; the norms are layer norms
  with weight and bias, c(x) = x + conv(x) with a causal convolution over time per channel (parts/conv.py);
* 'channel_delta' layers: the gated delta rule with a decay per key channel (parts/delta_rule.py);
* 'latent_attention' layers: attention over one latent row per token (parts/latent_attention.py), queries through a
  latent of their own, YaRN frequencies on the rotated part, a sliding window; a layer with ``kv_from`` keeps no
  latent and reads the rows of the layer it names, which are kept for the widest window among their readers;
* feed-forwards: experts g = min(gate h, limit), u = clamp(up h, -limit, limit), down(g sigmoid(1.702 g) (u + 1)); the picks are the
  largest of a softmax over all experts, weighted by their share of the picked scores times ``router.scale``
  (dividing softmax values by the sum of the picked ones is the softmax over the picked logits, which is what
  the router computes); plus a shared expert with a width and a limit of its own;
* final layer norm, head, logits times ``logit_scale``.

Tensor names: ``embed``, ``bigram``, ``l<i>.canon1|canon2``, ``l<i>.norm1|norm2`` (+ ``.b``), ``l<i>.mix.{q,k,v}`` (+ ``.conv``),
``l<i>.mix.{b,A_log,norm,a1,a2,dt_bias,g1,g2,o}``, ``l<i>.mix.{dq,dq.norm,uq,dkv,dkv.norm,uk,uv,o}``,
``l<i>.mlp.{router,e<j>.{gate,up,down},shared.{gate,up,down}}``, ``final.norm`` (+ ``.b``), ``head``.
"""
from __future__ import annotations

from typing import Dict, Tuple

from ..cache.spec import WINDOW_NONE, WINDOW_SLIDING
from ..config.pagonex import DEFAULT_RANK, PagonexConfig
from ..parts.block import ConvPostNormBlock
from ..parts.conv import ResidualConv
from ..parts.delta_rule import GatedDeltaRule
from ..parts.embedding import BigramEmbedding
from ..parts.feedforward import MoESwiGLU
from ..parts.latent_attention import LatentAttention
from ..parts.model import DecoderModel, Run
from ..parts.norm import LayerNorm
from ..parts.position import Rotary, YarnRotary, YarnScaling
from ..registry import register_architecture

BLOCK_NAMES = {"conv1": "canon1", "mixer": "mix.", "norm1": "norm1", "conv2": "canon2", "ffn": "mlp.", "norm2": "norm2"}
MOE_NAMES = {"router": "router", "gate": "e{e}.gate", "up": "e{e}.up", "down": "e{e}.down", "shared": "shared.", "shared_gate": "gate",
             "shared_up": "up", "shared_down": "down"}
ACTIVATION = "swish_clamp"


def _windows_kept(cfg: PagonexConfig) -> Dict[int, Tuple[int, int]]:
    """Per layer that keeps latent rows: the (kind, window) they are kept for, the widest among its readers."""
    seen: Dict[int, list] = {}
    for i, layer in enumerate(cfg.layers):
        if layer.type == "latent_attention":
            seen.setdefault(i if layer.mixer.kv_from is None else layer.mixer.kv_from, []).append(layer.mixer.window)
    return {i: (WINDOW_NONE, 0) if None in ws else (WINDOW_SLIDING, max(ws)) for i, ws in seen.items()}


def build_pagonex(cfg: PagonexConfig) -> DecoderModel:
    cfg.validate()
    W, eps = cfg.width, cfg.norm_eps
    kept = _windows_kept(cfg)
    blocks, schedule = [], []
    for i, layer in enumerate(cfg.layers):
        m, f = layer.mixer, layer.mlp
        run = Run(i, i)
        if layer.type == "channel_delta":
            mixer = GatedDeltaRule(W, m.heads, m.kv_heads, m.dim, m.vdim, m.conv, m.decay_rank or DEFAULT_RANK,
                                   m.gate_rank or DEFAULT_RANK, eps)
        else:
            rotary = None
            if m.rot is not None and m.rot.scaling is not None:
                rotary = YarnRotary(m.rot_dim, m.rot.base, YarnScaling(**m.rot.scaling_dict()), "interleaved", m.rot.dims)
            elif m.rot is not None:
                rotary = Rotary(m.rot_dim, m.rot.base, None, "interleaved", m.rot.dims)
            owner = i if m.kv_from is None else m.kv_from
            mixer = LatentAttention(W, m.heads, m.dim, m.rot_dim, m.vdim, m.kv_rank, rotary, eps, m.scale, sink=False, gate=False,
                                    own_latent=m.kv_from is None, window_kind=WINDOW_SLIDING if m.window else WINDOW_NONE,
                                    window=m.window or 0, q_rank=m.q_rank, kept=kept[owner])
            if m.kv_from is not None:
                run = Run(i, i, kv_from=m.kv_from)
        ffn = None
        if f is not None:
            ffn = MoESwiGLU(W, f.experts, f.top, f.ff, shared_intermediate=f.shared_ff or None, gate="softmax_picked", renormalise=False,
                            score_on_input=False, activation=ACTIVATION, names=MOE_NAMES, limit=f.limit,
                            shared_limit=f.shared_limit or None, weight_scale=f.scale)
        blocks.append(ConvPostNormBlock(ResidualConv(W, cfg.canon_taps), mixer, LayerNorm(W, eps, name=""),
                                        ResidualConv(W, cfg.canon_taps) if ffn else None, ffn, LayerNorm(W, eps, name="") if ffn else None,
                                        names=BLOCK_NAMES))
        schedule.append(run)
    b = cfg.bigram
    return DecoderModel(cfg.vocab_size, W, blocks, LayerNorm(W, eps, name=""), schedule=schedule, tie_embeddings=False, config=cfg,
                        layer_prefix="l", embed_name="embed", norm_prefix="final.norm", head_name="head", logit_scale=cfg.logit_scale,
                        embedding=None if b is None else BigramEmbedding(W, b.buckets, b.mul_prev, b.mul_cur))


register_architecture("Pagonex", PagonexConfig, build_pagonex)
