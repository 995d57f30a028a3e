"""Small Rigodra configurations for the tests: every size differs between them and between layers, and what one has the
other lacks (masks, kept first tokens, rotation, value mixing, feed-forwards, groups, identity experts, shared experts)."""
import copy


def _rot(rot):
    return {"base": rot[0], "dims": rot[1]}


def _attn(heads, kv_heads, dim, vdim, scale, rot=None, window=None, keep=0, v_mix=False):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if rot:
        m["rot"] = _rot(rot)
    if window:
        m["mask"] = {"size": window, **({"keep_first": keep} if keep else {})}
    if v_mix:
        m["v_mix"] = True
    return {"type": "attention", "mixer": m}


def _latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, rot=None, window=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale}
    if rot:
        m["rot"] = _rot(rot)
    if window:
        m["mask"] = {"size": window}
    return {"type": "latent_attention", "mixer": m}


def _dense(ff):
    return {"kind": "dense", "ff": ff}


def _moe(experts, top, ff, groups=None, identity=0, shared=0):
    r = {"experts": experts, "top": top}
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    if identity:
        r["identity"] = identity
    m = {"kind": "moe", "expert": {"ff": ff}, "router": r}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def _layer(mixer, mlp):
    return {**mixer, "mlp": mlp}


# odd sizes: heads and latents no matrix-core kernel takes, rotated parts that turn only in part, windows that are no
# multiple of a page, kept tokens that end inside a page and beyond one, a mixing layer between two that do not mix,
# identity experts that are half of a group and a whole one, one pick and four, a layer without a feed-forward
ODD = {
    "architecture": "Rigodra", "vocab": 107, "width": 68, "norm": {"eps": 1e-5}, "postln_alpha": 1.4,
    "layers": [
        _layer(_attn(6, 2, 10, 14, 0.31, rot=(300.0, 6), window=29, keep=3, v_mix=True), _moe(4, 2, 20, groups=(3, 2), identity=2, shared=22)),
        _layer(_latent(3, 10, 6, 13, 21, 24, 0.25, rot=(500.0, 6), window=31), _dense(50)),
        _layer(_attn(2, 2, 16, 16, 0.25, rot=(300.0, 16), window=45), _moe(5, 4, 12)),
        _layer(_attn(4, 2, 22, 14, 0.2, rot=(90.0, 8), window=40, keep=21, v_mix=True), _moe(6, 3, 18, groups=(3, 2), identity=3, shared=18)),
        _layer(_attn(3, 1, 8, 20, 0.4), None),
        _layer(_latent(2, 12, 8, 9, 10, 18, 0.3), _moe(3, 1, 16, identity=1)),
        _layer(_attn(2, 2, 12, 14, 0.3, window=17, keep=40, v_mix=True), _dense(30)),
    ],
}

# sizes the matrix-core kernels take (keys and values of different widths, latents in sixteens, widths that are multiples
# of 128), a shared expert of the experts' own width (it rides with the routed ones), and one of another width
EVEN = {
    "architecture": "Rigodra", "vocab": 200, "width": 128, "norm": {"eps": 1e-6}, "postln_alpha": 0.8,
    "layers": [
        _layer(_attn(8, 2, 64, 32, 0.13, rot=(20000.0, 32), window=48, keep=5, v_mix=True), _moe(6, 2, 128, groups=(4, 2), identity=2, shared=128)),
        _layer(_latent(8, 16, 16, 24, 64, 80, 0.18, rot=(20000.0, 16), window=50), _dense(256)),
        _layer(_attn(4, 2, 96, 32, 0.1, rot=(1000.0, 64), window=100, keep=1, v_mix=True), _moe(7, 3, 128, groups=(2, 1), identity=1, shared=256)),
        _layer(_attn(2, 1, 32, 32, 0.2, rot=(500.0, 32)), _moe(4, 2, 256)),
    ],
}

# latents alone, one with no window and no rotation; every pick of every token possible
LATENTS = {
    "architecture": "Rigodra", "vocab": 61, "width": 96, "norm": {"eps": 1e-5}, "postln_alpha": 1.0,
    "layers": [
        _layer(_latent(2, 16, 4, 16, 32, 32, 0.25, rot=(30.0, 4), window=16), None),
        _layer(_latent(3, 8, 8, 20, 16, 48, 0.3), _moe(2, 3, 24, identity=1, shared=40)),
    ],
}

# one query head, one group, no kept tokens; the mixing layers stand side by side, then one at the end
SOLO = {
    "architecture": "Rigodra", "vocab": 50, "width": 64, "norm": {"eps": 1e-6}, "postln_alpha": 3.0,
    "layers": [
        _layer(_attn(1, 1, 32, 64, 0.2, rot=(100.0, 32), window=1, keep=2, v_mix=True), _dense(64)),
        _layer(_attn(2, 1, 64, 64, 0.15, rot=(100.0, 2), window=33, keep=16, v_mix=True), None),
        _layer(_attn(4, 1, 30, 64, 0.2, v_mix=True), _moe(1, 1, 16)),
    ],
}

CONFIGS = {"odd": ODD, "even": EVEN, "latents": LATENTS, "solo": SOLO}
SEEDS = {"odd": 71, "even": 72, "latents": 73, "solo": 74}
# projections that make the scores sharp, biases and norms that show, branches as large as the sum they are added to,
# corrections that move picks
STD_BY_SUFFIX = {"norm1.b": 0.3, "norm2.b": 0.3, "final.norm.b": 0.3, "embed.norm.b": 0.3, ".vmix": 0.6, ".correction": 0.3, ".router": 0.3,
                 ".mix.g": 0.3, ".up": 0.25, ".down": 0.25, ".mix.o": 0.2}


def config(name):
    return copy.deepcopy(CONFIGS[name])
