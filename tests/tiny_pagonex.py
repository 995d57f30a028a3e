"""Small Pagonex configurations for the tests: every size differs between them and between layers, and
what one has the other lacks (masks, rotation and its scaling, shared rows, feed-forwards, shared experts, the
bigram table, convolutions of more than one tap)."""
import copy


def _delta(heads, kv_heads, dim, vdim, conv, decay_rank, gate_rank):
    return {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv,
                                               "decay_rank": decay_rank, "gate_rank": gate_rank}}


def _latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, rot=None, window=None, kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale}
    if rot:
        m["rot"] = {"base": rot[0], "dims": rot[1]}
        if len(rot) > 2:
            m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), rot[2:]))
    if window:
        m["mask"] = {"size": window}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m}


def _moe(experts, top, ff, limit, scale, shared=None):
    m = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top, "scale": scale}}
    if shared:
        m["shared"] = {"ff": shared[0], "limit": shared[1]}
    return m


def _layer(mixer, mlp):
    return {**mixer, "mlp": mlp}


# odd sizes: heads and latents no matrix-core kernel takes, several heads over one key head, a rotated part that turns
# only in part, rows shared by layers with a wider window and with none, one pick and three, a layer without a
# feed-forward, windows that are no multiple of a page
ODD = {
    "architecture": "Pagonex", "vocab": 103, "width": 76, "norm": {"eps": 1e-5}, "canon": {"taps": 3}, "logit_scale": 0.6,
    "embedding": {"bigram": {"buckets": 59, "mul_prev": 13, "mul_cur": 5}},
    "layers": [
        _layer(_latent(3, 10, 6, 14, 20, 24, 0.25, rot=(500.0, 4, 3.0, 64, 8.0, 1.0), window=29), _moe(5, 3, 24, 0.9, 2.5, shared=(20, 1.4))),
        _layer(_delta(6, 2, 20, 12, 2, 6, 10), _moe(4, 1, 18, 1.2, 0.7)),
        _layer(_latent(5, 8, 6, 9, 14, 24, 0.3, rot=(500.0, 4, 3.0, 64, 8.0, 1.0), window=41, kv_from=0), None),
        _layer(_delta(4, 4, 9, 30, 5, 7, 5), _moe(3, 2, 10, 2.0, 1.0, shared=(10, 2.0))),
        _layer(_latent(2, 12, 8, 16, 10, 18, 0.2), _moe(6, 4, 12, 0.6, 1.3)),
        _layer(_latent(4, 6, 8, 5, 9, 18, 0.35, window=17, kv_from=4), _moe(3, 3, 14, 1.1, 1.9, shared=(26, 0.8))),
    ],
}

# sizes the matrix-core kernels take (latents in sixteens, widths that are multiples of 128), a shared expert of the
# experts' own width and limit (it rides with the routed ones), and one of another width
EVEN = {
    "architecture": "Pagonex", "vocab": 192, "width": 128, "norm": {"eps": 1e-6}, "canon": {"taps": 4}, "logit_scale": 1.0,
    "embedding": {"bigram": {"buckets": 211, "mul_prev": 100003, "mul_cur": 65537}},
    "layers": [
        _layer(_delta(4, 2, 32, 48, 4, 16, 24), _moe(8, 2, 128, 1.5, 1.7, shared=(128, 1.5))),
        _layer(_latent(4, 32, 16, 32, 64, 80, 0.14, rot=(20000.0, 16, 8.0, 256, 32.0, 1.0), window=48), _moe(6, 2, 128, 1.0, 1.0, shared=(256, 3.0))),
        _layer(_latent(8, 16, 16, 24, 48, 80, 0.18, rot=(20000.0, 16, 8.0, 256, 32.0, 1.0), window=100, kv_from=1), _moe(4, 4, 128, 0.7, 2.2)),
        _layer(_delta(2, 1, 64, 64, 3, 32, 8), _moe(6, 3, 256, 2.0, 0.5)),
    ],
}

# key channels beyond 64 and 128, one tap everywhere (nothing kept for convolutions), no bigram table, no rotation
WIDE = {
    "architecture": "Pagonex", "vocab": 61, "width": 96, "norm": {"eps": 1e-5}, "canon": {"taps": 1}, "logit_scale": 3.0,
    "layers": [
        _layer(_delta(2, 1, 136, 40, 1, 12, 20), _moe(2, 1, 16, 0.8, 1.4, shared=(24, 0.6))),
        _layer(_latent(2, 16, 4, 16, 32, 32, 0.25, window=16), None),
        _layer(_delta(1, 1, 72, 33, 8, 5, 3), _moe(3, 3, 32, 1.3, 0.9)),
        _layer(_latent(3, 8, 8, 20, 16, 32, 0.3, rot=(30.0, 8)), _moe(4, 2, 24, 1.0, 1.0)),
    ],
}

# delta layers alone: no pages at all; eight taps in front of the branches
SOLO = {
    "architecture": "Pagonex", "vocab": 50, "width": 64, "norm": {"eps": 1e-6}, "canon": {"taps": 8}, "logit_scale": 0.8,
    "embedding": {"bigram": {"buckets": 7, "mul_prev": 3, "mul_cur": 2}},
    "layers": [
        _layer(_delta(2, 2, 16, 16, 4, 8, 8), _moe(4, 2, 16, 1.0, 1.1)),
        _layer(_delta(3, 3, 40, 17, 3, 4, 6), None),
    ],
}

CONFIGS = {"odd": ODD, "even": EVEN, "wide": WIDE, "solo": SOLO}
SEEDS = {"odd": 61, "even": 62, "wide": 63, "solo": 64}
# convolutions that mix their taps, decays from almost none to strong, biases and norms that show, branches as large
# as the sum they are added to
STD_BY_SUFFIX = {".conv": 0.6, "canon1": 0.4, "canon2": 0.4, ".A_log": 2.0, ".dt_bias": 1.0, "norm1.b": 0.3, "norm2.b": 0.3,
                 "final.norm.b": 0.3, "bigram": 0.3, ".b": 0.3, ".g2": 0.3, ".a2": 0.3}


def config(name):
    return copy.deepcopy(CONFIGS[name])
