"""A plain, slow Pagonex decoder: whole sequences, no cache, one function a mechanism.

The yardstick of the Pagonex tests.  It shares no code with the package: ``config.json`` as a raw
dict, weights as a ``{name: tensor}`` dict, dense tensor arithmetic on the CPU (float64 unless
told otherwise), every key and every state of a sequence recomputed from its first token.

Notation: T tokens, W the model width, H heads, G key heads, d the width of a key head (or of the
unrotated part of one), r the width of a rotated part, e the width of a value head, n the taps of a
convolution.
"""
from __future__ import annotations

import json
import math
import os
from typing import Callable, Dict, List, Optional, Sequence

import torch

SWISH_SLOPE = 1.702       # an expert's gate is g * sigmoid(SWISH_SLOPE * g)
UNIT_FLOOR = 1e-6         # added to a sum of squares before its root is divided by
SHARE_FLOOR = 1e-20       # added to the picked scores' sum
YARN_SLOPE = 0.1


def _same(x: torch.Tensor) -> torch.Tensor:
    return x


def store_bf16(x: torch.Tensor) -> torch.Tensor:
    """x rounded to bfloat16 and widened again: what a tensor kept in 16 bits loses.  Handed to the
    functions below as ``store``, it is applied where a 16-bit engine may keep a tensor (the inputs and
    outputs of matrix products, of short convolutions, of activations and of the attention), and nowhere
    in what the design computes in 32 bits (scores and softmax, rotations, everything inside the
    recurrence, norms' statistics, the router, the residual sum)."""
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


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def softplus(z: torch.Tensor) -> torch.Tensor:
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def unit_vector(x: torch.Tensor) -> torch.Tensor:
    return x / torch.sqrt(x.pow(2).sum(dim=-1, keepdim=True) + UNIT_FLOOR)


def causal_conv(u: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """u [T, C], w [C, n]: y_t = sum_j w[:, j] * u_(t - n + 1 + j), zeros before the first row."""
    T, n = u.shape[0], w.shape[1]
    padded = torch.cat([torch.zeros(n - 1, u.shape[1], dtype=u.dtype), u], dim=0)
    y = torch.zeros_like(u)
    for j in range(n):
        y = y + padded[j:j + T] * w[:, j][None, :]
    return y


def bigram_rows(tokens: Sequence[int], mul_prev: int, mul_cur: int, buckets: int) -> List[int]:
    """Per token the row of the bigram table: (previous * mul_prev + current * mul_cur) mod buckets; the
    first token takes the row behind the last bucket."""
    return [buckets if i == 0 else (tokens[i - 1] * mul_prev + t * mul_cur) % buckets for i, t in enumerate(tokens)]


def rotation(positions: torch.Tensor, base: float, dims: int, scaling: Optional[dict], dtype) -> tuple:
    """(cos, sin), each [T, dims / 2], of the pairs of a rotated part at `positions`."""
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    magnitude = 1.0
    if scaling is not None:
        factor, original = scaling["factor"], scaling["original"]

        def place(turns):
            return dims * math.log(original / (2 * math.pi * turns)) / (2 * math.log(base))
        lo, hi = max(math.floor(place(scaling["fast"])), 0), min(math.ceil(place(scaling["slow"])), dims - 1)
        ramp = [min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0) for i in range(dims // 2)]
        f = [x / factor * s + x * (1.0 - s) for x, s in zip(f, ramp)]
        magnitude = YARN_SLOPE * math.log(factor) + 1.0
    a = positions.to(dtype)[:, None] * torch.tensor(f, dtype=dtype)[None, :]
    return torch.cos(a) * magnitude, torch.sin(a) * magnitude


def rotate_pairs(x: torch.Tensor, cos: torch.Tensor, sin: torch.Tensor) -> torch.Tensor:
    """x [T, heads, r]: elements 2i and 2i + 1 turn together for every pair cos and sin hold; the rest pass."""
    k = 2 * cos.shape[1]
    u, v = x[..., 0:k:2], x[..., 1:k:2]
    c, s = cos[:, None, :], sin[:, None, :]
    turned = torch.stack([u * c - v * s, v * c + u * s], dim=-1).flatten(-2)
    return torch.cat([turned, x[..., k:]], dim=-1)


def visible(T: int, window: Optional[int]) -> torch.Tensor:
    """[T, T] bool: key j is seen from i when j <= i and, with a window, i - j < window."""
    i = torch.arange(T)[:, None]
    j = torch.arange(T)[None, :]
    ok = j <= i
    return ok & (i - j < window) if window else ok


# ----------------------------------------------------------------------------
# mixers
# ----------------------------------------------------------------------------
def delta_rule(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, g: torch.Tensor, beta: torch.Tensor,
               S: Optional[torch.Tensor] = None):
    """The gated delta rule on q, k, g [T, H, d], v [T, H, e], beta [T, H] from state S [H, d, e] (zeros): per token and
    head S <- g S (rows), u = beta (v - S^T k), S <- S + k u^T, o = S^T q.  Returns o [T, H, e] and the last S."""
    T, H, d = q.shape
    if S is None:
        S = torch.zeros(H, d, v.shape[2], dtype=q.dtype)
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for t in range(T):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out, S


def channel_delta(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict, eps: float, store: Callable = _same) -> torch.Tensor:
    T = h.shape[0]
    H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]

    def stream(name, heads, width):
        return store(silu(causal_conv(store(h @ w[p + name].T), w[p + name + ".conv"]))).reshape(T, heads, width)
    q = unit_vector(stream("q", G, d)) * d ** -0.5
    k = unit_vector(stream("k", G, d))
    v = stream("v", H, e)
    q, k = q.repeat_interleave(H // G, dim=1), k.repeat_interleave(H // G, dim=1)
    beta = torch.sigmoid(h @ w[p + "b"].T)
    z = ((h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "dt_bias"]).reshape(T, H, d)
    g = torch.exp(-torch.exp(w[p + "A_log"])[None, :, None] * softplus(z))
    o, _ = delta_rule(q, k, v, g, beta)
    gate = torch.sigmoid(store(store(h @ w[p + "g1"].T) @ w[p + "g2"].T)).reshape(T, H, e)
    y = store(rms_norm(o, w[p + "norm"], eps) * gate).reshape(T, H * e)
    return store(y @ w[p + "o"].T)


def latent_rows(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict, eps: float, store: Callable = _same):
    """What a latent layer keeps of every token: the normed latent [T, kv_rank] and the rotated key part [T, 1, r]."""
    T, R = h.shape[0], m["kv_rank"]
    y = store(h @ w[p + "dkv"].T)
    rot = m.get("rot")
    k_rot = y[:, R:].reshape(T, 1, m["rot_dim"])
    if rot:
        cos, sin = rotation(torch.arange(T), rot["base"], rot["dims"], rot.get("scaling"), h.dtype)
        k_rot = rotate_pairs(k_rot, cos, sin)
    return store(rms_norm(y[:, :R], w[p + "dkv.norm"], eps)), store(k_rot)


def latent_attention(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict, eps: float, kept: tuple,
                     store: Callable = _same) -> torch.Tensor:
    """Keys and values expanded per head from the kept rows (this layer's own, or those of the layer it shares)."""
    T = h.shape[0]
    H, d, r, e = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    c, k_rot = kept
    cq = store(rms_norm(store(h @ w[p + "dq"].T), w[p + "dq.norm"], eps))
    q = store(cq @ w[p + "uq"].T).reshape(T, H, d + r)
    q_rot = q[..., d:]
    rot = m.get("rot")
    if rot:
        cos, sin = rotation(torch.arange(T), rot["base"], rot["dims"], rot.get("scaling"), h.dtype)
        q_rot = rotate_pairs(q_rot, cos, sin)
    q_rot = store(q_rot)
    uk, uv = w[p + "uk"].reshape(H, d, -1), w[p + "uv"].reshape(H, e, -1)
    mask = visible(T, m["mask"]["size"] if m.get("mask") else None)
    heads = []
    for i in range(H):
        s = (store(q[:, i, :d] @ uk[i]) @ c.T + q_rot[:, i] @ k_rot[:, 0].T) * m["scale"]
        a = torch.softmax(s.masked_fill(~mask, float("-inf")), dim=-1)
        heads.append(store(store(a @ c) @ uv[i].T))
    return store(torch.cat(heads, dim=-1) @ w[p + "o"].T)


# ----------------------------------------------------------------------------
# feed-forward
# ----------------------------------------------------------------------------
def clamped_unit(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, limit: float, store: Callable = _same) -> torch.Tensor:
    g = torch.clamp(store(h @ w[p + "gate"].T), max=limit)
    u = torch.clamp(store(h @ w[p + "up"].T), min=-limit, max=limit)
    return store(store(g * torch.sigmoid(SWISH_SLOPE * g) * (u + 1.0)) @ w[p + "down"].T)


def route(h: torch.Tensor, router: torch.Tensor, top: int, scale: float):
    """(ids, weights) [T, top]: the largest of the softmax over all experts, divided by their sum, times scale."""
    s = torch.softmax(h @ router.T, dim=-1)
    val, ids = torch.topk(s, top, dim=-1)
    return ids, val / (val.sum(-1, keepdim=True) + SHARE_FLOOR) * scale


def experts(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, f: dict, store: Callable = _same, picks=None) -> torch.Tensor:
    """`picks`: (ids, weights) to use instead of the router's own (16-bit comparisons: a close call falls either way)."""
    r, ex = f["router"], f["expert"]
    ids, wts = route(h, w[p + "router"], r["top"], r["scale"]) if picks is None else picks
    y = torch.zeros_like(h)
    for j in range(r["experts"]):
        for i in range(r["top"]):
            rows = (ids[:, i] == j).nonzero(as_tuple=True)[0]
            if rows.numel():
                y[rows] += wts[rows, i, None] * clamped_unit(h[rows], w, f"{p}e{j}.", ex["limit"], store)
    if f.get("shared"):
        y = y + clamped_unit(h, w, p + "shared.", f["shared"]["limit"], store)
    return y


# ----------------------------------------------------------------------------
# the model
# ----------------------------------------------------------------------------
def forward(cfg: dict, w: Dict[str, torch.Tensor], tokens: Sequence[int], layer_outputs: Optional[list] = None,
            store: Callable = _same, router_picks: Optional[list] = None) -> torch.Tensor:
    """Logits [T, vocab] of the whole sequence."""
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.tensor(list(tokens))]
    big = (cfg.get("embedding") or {}).get("bigram")
    if big:
        x = x + w["bigram"][torch.tensor(bigram_rows(list(tokens), big["mul_prev"], big["mul_cur"], big["buckets"]))]
    kept: Dict[int, tuple] = {}
    routed = 0
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]

        def read(which):
            return store(x + causal_conv(x, w[p + which])) if p + which in w else store(x)
        h = read("canon1")
        if layer["type"] == "channel_delta":
            y = channel_delta(h, w, p + "mix.", m, eps, store)
        else:
            src = m.get("kv_from")
            if src is None:
                kept[i] = latent_rows(h, w, p + "mix.", m, eps, store)
            y = latent_attention(h, w, p + "mix.", m, eps, kept[i if src is None else src], store)
        x = x + layer_norm(y, w[p + "norm1"], w[p + "norm1.b"], eps)
        if layer.get("mlp"):
            y = experts(read("canon2"), w, p + "mlp.", layer["mlp"], store, None if router_picks is None else router_picks[routed])
            routed += 1
            x = x + layer_norm(y, w[p + "norm2"], w[p + "norm2.b"], eps)
        if layer_outputs is not None:
            layer_outputs.append(x.clone())
    n = store(layer_norm(x, w["final.norm"], w["final.norm.b"], eps))
    return (n @ w["head"].T) * cfg.get("logit_scale", 1.0)


def generate(cfg: dict, w: Dict[str, torch.Tensor], prompt: Sequence[int], n: int) -> List[int]:
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(forward(cfg, w, toks)[-1].argmax()))
    return toks[len(prompt):]
