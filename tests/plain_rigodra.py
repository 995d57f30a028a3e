"""A plain, slow Rigodra decoder: whole sequences, no cache, one function a mechanism.

The yardstick of the Rigodra tests.  It shares no code with the package: ``config.json`` as a raw
dict, weights as a ``{name: tensor}`` dict, dense tensor arithmetic on the CPU (float64 unless
told otherwise), every key and value of a sequence recomputed from its first token.

Notation: T tokens, W the model width, H query heads, G key/value heads, d the width of a key head (or
of the unrotated part of one), r the width of a rotated part, e the width of a value head.
"""
from __future__ import annotations

import json
import math
import os
from typing import Callable, Dict, List, Optional, Sequence

import torch


def _same(x: torch.Tensor) -> torch.Tensor:
    return x


def store_bf16(x: torch.Tensor) -> torch.Tensor:
    """x rounded to bfloat16 and widened again: what a tensor kept in 16 bits loses.  Handed to the
    functions below as ``store``, it is applied where a 16-bit engine may keep a tensor (the inputs and
    outputs of matrix products, of activations and of the attention), and nowhere in what the design
    computes in 32 bits (scores and softmax, rotations, norms, the router, the residual sum)."""
    return x.to(torch.bfloat16).to(x.dtype)


def read_config(model_dir: str) -> dict:
    with open(os.path.join(model_dir, "config.json")) as f:
        return json.load(f)


def load_weights(model_dir: str, dtype=torch.float64) -> Dict[str, torch.Tensor]:
    """Every tensor of model.safetensors, floats widened to `dtype` (own reader: 8 bytes of
    length, a JSON header, raw data)."""
    with open(os.path.join(model_dir, "model.safetensors"), "rb") as f:
        n = int.from_bytes(f.read(8), "little")
        header = json.loads(f.read(n))
        base = 8 + n
        out = {}
        kinds = {"BF16": torch.bfloat16, "F32": torch.float32, "F16": torch.float16, "I32": torch.int32, "I64": torch.int64}
        for name, e in header.items():
            if name == "__metadata__":
                continue
            a, b = e["data_offsets"]
            f.seek(base + a)
            t = torch.frombuffer(bytearray(f.read(b - a)), dtype=kinds[e["dtype"]]).reshape(e["shape"])
            out[name] = t.to(dtype) if t.dtype.is_floating_point else t.to(torch.int64)
    return out


# ----------------------------------------------------------------------------
# the small pieces
# ----------------------------------------------------------------------------
def rms_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt(x.pow(2).mean(dim=-1, keepdim=True) + eps) * w


def layer_norm(x: torch.Tensor, w: torch.Tensor, b: torch.Tensor, eps: float) -> torch.Tensor:
    """(x - mean) / sqrt(mean squared deviation + eps) * w + b along the last axis."""
    c = x - x.mean(dim=-1, keepdim=True)
    return c / torch.sqrt(c.pow(2).mean(dim=-1, keepdim=True) + eps) * w + b


def gelu(z: torch.Tensor) -> torch.Tensor:
    """z times the standard normal distribution function."""
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def relu2(z: torch.Tensor) -> torch.Tensor:
    return torch.clamp(z, min=0.0).pow(2)


def rotation(positions: torch.Tensor, base: float, dims: int, dtype) -> tuple:
    """(cos, sin), each [T, dims / 2], of the pairs of a rotated part at `positions`."""
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=dtype)
    a = positions.to(dtype)[:, None] * f[None, :]
    return torch.cos(a), torch.sin(a)


def rotate_halves(x: torch.Tensor, cos: torch.Tensor, sin: torch.Tensor) -> torch.Tensor:
    """x [T, heads, n]: with k pairs in cos and sin, elements i and i + k turn together (i < k); the rest pass."""
    k = cos.shape[1]
    u, v = x[..., :k], x[..., k:2 * k]
    c, s = cos[:, None, :], sin[:, None, :]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * k:]], dim=-1)


def turned(x: torch.Tensor, rot: Optional[dict]) -> torch.Tensor:
    if not rot:
        return x
    return rotate_halves(x, *rotation(torch.arange(x.shape[0]), rot["base"], rot["dims"], x.dtype))


def visible(T: int, mask: Optional[dict]) -> torch.Tensor:
    """[T, T] bool: key j is seen from i when j <= i and, with a mask, i - j < size or j < keep_first."""
    i = torch.arange(T)[:, None]
    j = torch.arange(T)[None, :]
    ok = j <= i
    if not mask:
        return ok
    return ok & ((i - j < mask["size"]) | (j < mask.get("keep_first", 0)))


# ----------------------------------------------------------------------------
# mixers
# ----------------------------------------------------------------------------
def mixed_values(v: torch.Tensor, v_first: Optional[torch.Tensor], lam) -> torch.Tensor:
    return v if v_first is None else (1.0 - lam) * v + lam * v_first


def attention(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict, eps: float, v_first: Optional[torch.Tensor],
              store: Callable = _same) -> tuple:
    """(output [T, W], this layer's values as projected [T, G, e])."""
    T = h.shape[0]
    H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_norm(store(h @ w[p + "q"].T).reshape(T, H, d), w[p + "q.norm"], eps)
    k = rms_norm(store(h @ w[p + "k"].T).reshape(T, G, d), w[p + "k.norm"], eps)
    q, k = store(turned(q, m.get("rot"))), store(turned(k, m.get("rot")))
    own = store(h @ w[p + "v"].T).reshape(T, G, e)
    v = store(mixed_values(own, v_first, w[p + "vmix"] if v_first is not None else None))
    gate = torch.sigmoid(store(h @ w[p + "g"].T))
    mask = visible(T, m.get("mask"))
    heads = []
    for i in range(H):
        g = i // (H // G)
        s = (q[:, i] @ k[:, g].T) * m["scale"]
        a = torch.softmax(s.masked_fill(~mask, float("-inf")), dim=-1)
        heads.append(store((a @ v[:, g]) * gate[:, i, None]))
    return store(torch.cat(heads, dim=-1) @ w[p + "o"].T), own


def latent_attention(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict, eps: float, store: Callable = _same) -> torch.Tensor:
    """Keys and values expanded per head from the latent of every token."""
    T = h.shape[0]
    H, d, r, e, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    y = store(h @ w[p + "dkv"].T)
    c = store(rms_norm(y[:, :R], w[p + "dkv.norm"], eps))
    k_rot = store(turned(y[:, R:].reshape(T, 1, r), m.get("rot")))
    cq = store(rms_norm(store(h @ w[p + "dq"].T), w[p + "dq.norm"], eps))
    q = store(cq @ w[p + "uq"].T).reshape(T, H, d + r)
    q_rot = store(turned(q[..., d:], m.get("rot")))
    uk, uv = w[p + "uk"].reshape(H, d, R), w[p + "uv"].reshape(H, e, R)
    mask = visible(T, m.get("mask"))
    heads = []
    for i in range(H):
        s = (store(q[:, i, :d] @ uk[i]) @ c.T + q_rot[:, i] @ k_rot[:, 0].T) * m["scale"]
        a = torch.softmax(s.masked_fill(~mask, float("-inf")), dim=-1)
        heads.append(store(store(a @ c) @ uv[i].T))
    return store(torch.cat(heads, dim=-1) @ w[p + "o"].T)


# ----------------------------------------------------------------------------
# feed-forward
# ----------------------------------------------------------------------------
def two_layers(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, act: Callable, store: Callable = _same) -> torch.Tensor:
    return store(store(act(store(h @ w[p + "up"].T))) @ w[p + "down"].T)


def route(h: torch.Tensor, router: torch.Tensor, correction: torch.Tensor, top: int, groups: Optional[dict]):
    """(ids, weights) [T, top]: softmax over every output; the largest corrected values are chosen, among the best
    groups of neighbours alone (a group ranks by its largest corrected value); the weights are uncorrected."""
    s = torch.softmax(h @ router.T, dim=-1)
    choice = s + correction
    if groups:
        T, E = choice.shape
        per = E // groups["count"]
        best = torch.topk(choice.reshape(T, groups["count"], per).max(dim=-1).values, groups["keep"], dim=-1).indices
        open_ = torch.zeros(T, groups["count"], dtype=torch.bool).scatter(1, best, True).repeat_interleave(per, dim=1)
        choice = choice.masked_fill(~open_, float("-inf"))
    ids = torch.topk(choice, top, dim=-1).indices
    return ids, s.gather(1, ids)


def experts(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, f: dict, x: torch.Tensor, store: Callable = _same,
            picks=None) -> torch.Tensor:
    """`x`: what an identity expert returns (the layer's input before any rounding).  `picks`: (ids, weights) to use
    instead of the router's own (16-bit comparisons: a close call falls either way)."""
    r = f["router"]
    ids, wts = route(h, w[p + "router"], w[p + "correction"], r["top"], r.get("groups")) if picks is None else picks
    y = torch.zeros_like(h)
    for j in range(r["experts"] + r.get("identity", 0)):
        for i in range(r["top"]):
            rows = (ids[:, i] == j).nonzero(as_tuple=True)[0]
            if rows.numel():
                out = two_layers(h[rows], w, f"{p}e{j}.", relu2, store) if j < r["experts"] else x[rows]
                y[rows] += wts[rows, i, None] * out
    if f.get("shared"):
        y = y + two_layers(h, w, p + "shared.", relu2, store)
    return y


# ----------------------------------------------------------------------------
# the model
# ----------------------------------------------------------------------------
def forward(cfg: dict, w: Dict[str, torch.Tensor], tokens: Sequence[int], layer_outputs: Optional[list] = None,
            store: Callable = _same, router_picks: Optional[list] = None) -> torch.Tensor:
    """Logits [T, vocab] of the whole sequence."""
    eps, alpha = cfg["norm"]["eps"], cfg["postln_alpha"]
    x = layer_norm(w["embed"][torch.tensor(list(tokens))], w["embed.norm"], w["embed.norm.b"], eps)
    v_first = None
    routed = 0
    for i, layer in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", layer["mixer"], layer.get("mlp")
        h = store(x)
        if layer["type"] == "attention":
            y, own = attention(h, w, p + "mix.", m, eps, v_first if m.get("v_mix") else None, store)
            if m.get("v_mix") and v_first is None:
                v_first = own
        else:
            y = latent_attention(h, w, p + "mix.", m, eps, store)
        x = layer_norm(alpha * x + y, w[p + "norm1"], w[p + "norm1.b"], eps)
        if f:
            h = store(x)
            if f["kind"] == "dense":
                y = two_layers(h, w, p + "mlp.", gelu, store)
            else:
                y = experts(h, w, p + "mlp.", f, x, store, None if router_picks is None else router_picks[routed])
                routed += 1
            x = layer_norm(alpha * x + y, w[p + "norm2"], w[p + "norm2.b"], eps)
        if layer_outputs is not None:
            layer_outputs.append(x.clone())
    n = store(layer_norm(x, w["final.norm"], w["final.norm.b"], eps))
    return n @ w["embed"].T


def generate(cfg: dict, w: Dict[str, torch.Tensor], prompt: Sequence[int], n: int) -> List[int]:
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(forward(cfg, w, toks)[-1].argmax()))
    return toks[len(prompt):]
