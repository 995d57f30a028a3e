"""The gated delta rule with a decay per key channel: a matrix-valued state that corrects what it holds."""
from __future__ import annotations

from typing import Dict, List, Optional, Tuple

import numpy as np
import torch

from .. import ops
from ..cache.spec import MixedSpec, StateSpec
from ..ops.profile import section
from .base import INIT_NORM_WEIGHT, HostStep, LayerCache, ParamSpec, Part, StepContext, StepPlanner, TensorSource
from .matrix_memory import _fuse


class DeltaChunks(StepPlanner):
    """The work lists of the chunked form, made once a step for all layers that run the delta rule: none in steps
    of single tokens."""

    key = "delta rule"

    def plan(self, host: HostStep) -> Tuple[List[np.ndarray], dict]:
        if not host.lens or max(host.lens) <= 1:
            empty = np.zeros(0, dtype=np.int32)
            return [empty, empty], dict(n=0)
        chunks, ents = ops.delta_chunks_of(host.lens, host.cu_tokens)
        return [chunks.reshape(-1), ents.reshape(-1)], dict(n=chunks.shape[0])

    def attach(self, ctx: StepContext, views: List[torch.Tensor], facts: dict) -> None:
        ctx.extras[self.key] = (views[0], views[1]) if facts["n"] else None


_CHUNKS = DeltaChunks()


class GatedDeltaRule(Part):
    """Linear attention whose state corrects itself.  With h the input: q = W_q h and k = W_k h (``kv_heads`` x dk), v = W_v h
    (heads x dv), each behind a causal convolution of ``conv_taps`` taps per channel and SiLU; q and k become unit vectors per
    head, x / sqrt(sum x^2 + 1e-6), q times dk^(-1/2) besides; head i reads key head i // (heads / kv_heads).  beta =
    sigmoid(W_b h), one per head; a decay per head and key channel g = exp(-exp(A_log) softplus(W_a2 (W_a1 h) + dt_bias)).
    Per head S <- g S (rows), u = beta (v - S^T k), S <- S + k u^T, o = S^T q; o is RMS-normed over dv with weights shared by the
    heads, multiplied by sigmoid(W_g2 (W_g1 h)), and the heads side by side go through W_o.

    Kept per request, in its state slot: S (``ops.delta_state_shape``) and a ring of the convolution's last inputs (float).
    The middles a1 and g1 and the beta logits are one product with a float result; from there on, and from the
    convolution on, everything up to the head norm is float.  Steps of single tokens run as one kernel from the projections
    to the gated heads; others in chunks of 16 tokens as matrix products (csrc/delta_rule.hip)."""

    NAMES = {"q": "q", "k": "k", "v": "v", "q_conv": "q.conv", "k_conv": "k.conv", "v_conv": "v.conv", "b": "b", "A_log": "A_log", "a1": "a1",
             "a2": "a2", "dt_bias": "dt_bias", "g1": "g1", "g2": "g2", "norm": "norm", "o": "o"}

    def __init__(self, hidden: int, num_heads: int, kv_heads: int, key_dim: int, value_dim: int, conv_taps: int, decay_rank: int,
                 gate_rank: int, norm_eps: float, names: Optional[Dict[str, str]] = None):
        if min(num_heads, kv_heads, key_dim, value_dim, decay_rank, gate_rank) < 1 or num_heads % kv_heads:
            raise ValueError("heads, kv_heads, key_dim, value_dim and the ranks must be positive, kv_heads divide heads")
        if key_dim > ops.DELTA_MAX_KEY_DIM or value_dim > ops.DELTA_MAX_VALUE_DIM:
            raise ValueError(f"heads of {key_dim} x {value_dim} are not taken: at most {ops.DELTA_MAX_KEY_DIM} x {ops.DELTA_MAX_VALUE_DIM}")
        if not 1 <= conv_taps <= ops.DELTA_MAX_TAPS:
            raise ValueError(f"a convolution of {conv_taps} taps is not taken: 1 to {ops.DELTA_MAX_TAPS}")
        self.hidden, self.nh, self.nkv, self.dk, self.dv = int(hidden), int(num_heads), int(kv_heads), int(key_dim), int(value_dim)
        self.taps, self.a_rank, self.g_rank, self.eps = int(conv_taps), int(decay_rank), int(gate_rank), float(norm_eps)
        self.channels = 2 * self.nkv * self.dk + self.nh * self.dv
        self.names = {**self.NAMES, **(names or {})}
        self.graph_safe = True         # entries and their state slots are read from the step's device arrays
        self.w_in = None               # [q | k | v] rows
        self.w_mid = None              # [a1 | g1 | b] rows: a product of its own, with a float result
        self.w_a2: Optional[torch.Tensor] = None      # [heads * dk, a_rank]
        self.w_g2: Optional[torch.Tensor] = None      # [heads * dv, g_rank]
        self.w_conv: Optional[torch.Tensor] = None    # float32 [channels, taps]
        self.dt_bias: Optional[torch.Tensor] = None
        self.a_log: Optional[torch.Tensor] = None
        self.w_norm: Optional[torch.Tensor] = None    # float32 [dv]
        self.w_norm_heads: Optional[torch.Tensor] = None      # the same, once per head
        self.w_o = None

    def step_planners(self):
        return (_CHUNKS,)

    def cache_spec(self):
        state = StateSpec(ops.delta_state_shape(self.nh, self.dk, self.dv), torch.float32)
        if self.taps == 1:
            return state
        return MixedSpec(None, (state, StateSpec((self.taps, self.channels), torch.float32)))

    def param_specs(self, prefix: str) -> Dict[str, ParamSpec]:
        n, qk, vv = self.names, self.nkv * self.dk, self.nh * self.dv
        return {
            prefix + n["q"]: ParamSpec((qk, self.hidden)),
            prefix + n["k"]: ParamSpec((qk, self.hidden)),
            prefix + n["v"]: ParamSpec((vv, self.hidden)),
            prefix + n["q_conv"]: ParamSpec((qk, self.taps)),
            prefix + n["k_conv"]: ParamSpec((qk, self.taps)),
            prefix + n["v_conv"]: ParamSpec((vv, self.taps)),
            prefix + n["b"]: ParamSpec((self.nh, self.hidden)),
            prefix + n["A_log"]: ParamSpec((self.nh,)),
            prefix + n["a1"]: ParamSpec((self.a_rank, self.hidden)),
            prefix + n["a2"]: ParamSpec((self.nh * self.dk, self.a_rank)),
            prefix + n["dt_bias"]: ParamSpec((self.nh * self.dk,)),
            prefix + n["g1"]: ParamSpec((self.g_rank, self.hidden)),
            prefix + n["g2"]: ParamSpec((vv, self.g_rank)),
            prefix + n["norm"]: ParamSpec((self.dv,), INIT_NORM_WEIGHT),
            prefix + n["o"]: ParamSpec((self.hidden, vv)),
        }

    def load(self, prefix: str, source: TensorSource) -> None:
        n = self.names
        get = lambda k: source.get(prefix + n[k])
        self.w_in = ops.pack_weight(_fuse([get(k) for k in ("q", "k", "v")], self.hidden))
        self.w_mid = ops.pack_weight(_fuse([get(k) for k in ("a1", "g1", "b")], self.hidden))
        self.w_a2, self.w_g2 = get("a2").contiguous(), get("g2").contiguous()
        if self.w_a2.dtype != self.w_g2.dtype:
            self.w_a2, self.w_g2 = self.w_a2.float(), self.w_g2.float()
        self.w_conv = torch.cat([get(k).float() for k in ("q_conv", "k_conv", "v_conv")]).contiguous()
        self.dt_bias, self.a_log, self.w_norm = (get(k).float().contiguous() for k in ("dt_bias", "A_log", "norm"))
        self.w_norm_heads = self.w_norm.repeat(self.nh).contiguous()
        self.w_o = ops.pack_weight(get("o"))

    def forward(self, x: torch.Tensor, ctx: StepContext, cache: LayerCache) -> torch.Tensor:
        T = x.shape[0]
        nk, vv = self.nh * self.dk, self.nh * self.dv
        width = 2 if ctx.act_dtype == torch.bfloat16 else 4
        n_mid = self.a_rank + self.g_rank + self.nh
        with section("q|k|v", nbytes=width * self.channels * (self.hidden + T) + width * T * self.hidden, flops=2.0 * T * self.hidden * self.channels):
            proj = ops.linear(x, self.w_in, ctx.act_dtype)
        with section("a1|g1|b", nbytes=width * n_mid * self.hidden + width * T * self.hidden + 4 * T * n_mid, flops=2.0 * T * self.hidden * n_mid):
            mid = ops.linear(x, self.w_mid, torch.float32)
        with section("decays + gate", nbytes=width * (nk * self.a_rank + vv * self.g_rank) + T * (4 * n_mid + 4 * nk + width * vv),
                     flops=2.0 * T * (nk * self.a_rank + vv * self.g_rank)):
            log_decay, gate = ops.lowrank(mid, (0, self.w_a2, self.dt_bias, self.a_log), (self.a_rank, self.w_g2))
            if gate.dtype != ctx.act_dtype:
                gate = ops.cast(gate, ctx.act_dtype)
        state, ring = cache.states[0], cache.states[1] if self.taps > 1 else None
        args = (proj, 0, self.w_conv, ring, log_decay, mid, self.a_rank + self.g_rank, state, ctx, self.nh, self.nkv, self.dk, self.dv)
        moved = lambda: 8 * ctx.n_entries * nk * self.dv + T * (width * (self.channels + 2 * vv) + 4 * nk)
        lists = ctx.extras.get(_CHUNKS.key)
        if lists is None:
            with section("recurrence", nbytes=moved, flops=8.0 * T * nk * self.dv):
                y = ops.delta_step(*args, self.w_norm, self.eps, gate)
        else:
            with section("recurrence", nbytes=moved, flops=8.0 * T * nk * self.dv):
                o = ops.delta_chunks(*args, lists)
            with section("head norm + gate", nbytes=T * vv * (4 + 2 * width)):
                y = ops.group_norm_gate(o, self.w_norm_heads, self.eps, self.nh, ctx.act_dtype, gate, 0, ops.GATE_SIGMOID_ACT)
        with section("o", nbytes=width * self.hidden * (vv + T) + width * T * vv, flops=2.0 * T * self.hidden * vv):
            return ops.linear(y, self.w_o, ctx.act_dtype)
