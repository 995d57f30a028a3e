"""Rigodra without a GPU: the configuration reader, the tensors the model asks for, the memory each layer gets and what a
window that keeps first tokens holds of it, and the plain implementation's own consistency (what the GPU tests lean on)."""
import math

import pytest
import torch

import plain_rigodra as P
from tiny_rigodra import CONFIGS, config

from sharpinference_amd import load_config, ops
from sharpinference_amd.cache.manager import CacheError, CacheManager, pages_to_hold, pool_sizes
from sharpinference_amd.cache.spec import WINDOW_NONE, WINDOW_SLIDING, KVSpec
from sharpinference_amd.config.base import ConfigError
from sharpinference_amd.config.rigodra import RigodraConfig
from sharpinference_amd.parts.attention import Attention
from sharpinference_amd.parts.feedforward import MoESwiGLU
from sharpinference_amd.parts.latent_attention import LatentAttention
from sharpinference_amd.parts.position import Rotary
from sharpinference_amd.registry import build_model, registered_architectures


def test_the_design_is_registered_and_its_configuration_round_trips():
    assert "Rigodra" in registered_architectures()
    for name in CONFIGS:
        cfg = load_config(config(name))
        assert isinstance(cfg, RigodraConfig)
        assert cfg.to_dict() == config(name)
        assert load_config(cfg.to_dict()) == cfg


def test_what_the_file_leaves_out_is_off():
    cfg = load_config(config("odd"))
    bare = cfg.layers[4].mixer
    assert bare.window is None and bare.rot is None and bare.keep_first == 0 and not bare.v_mix
    assert cfg.layers[4].mlp is None and cfg.layers[2].mlp.identity == 0 and cfg.layers[2].mlp.shared_ff == 0
    assert (cfg.layers[2].mlp.groups, cfg.layers[2].mlp.keep) == (1, 1) and cfg.layers[2].mixer.keep_first == 0
    d = config("odd")
    m = d["layers"][2]["mixer"]
    m.pop("kv_heads"), m.pop("vdim"), m.pop("scale"), m["rot"].pop("dims")
    m["mask"]["keep_first"] = 0
    got = load_config(d).layers[2].mixer
    assert (got.kv_heads, got.vdim, got.scale, got.rot.dims, got.keep_first) == (2, 16, pytest.approx(0.25), 16, 0)


@pytest.mark.parametrize("path, value, what", [
    (("layers", 0, "mixer", "sink"), 1.0, "sink"),
    (("layers", 0, "mixer", "rot", "kind"), "half", "kind"),
    (("layers", 0, "mixer", "rot", "scaling"), {"factor": 2.0}, "factor"),
    (("layers", 0, "mixer", "mask", "kind"), "chunk", "kind"),
    (("layers", 1, "mixer", "mask", "keep_first"), 2, "keep_first"),
    (("layers", 1, "mixer", "rot", "scaling"), {"factor": 2.0}, "scaling"),
    (("layers", 1, "mixer", "kv_from"), 0, "kv_from"),
    (("layers", 1, "mlp", "limit"), 2.0, "limit"),
    (("layers", 0, "mlp", "router", "scale"), 2.0, "scale"),
    (("layers", 0, "mlp", "router", "groups", "top"), 2, "top"),
    (("layers", 0, "mlp", "expert", "limit"), 2.0, "limit"),
    (("layers", 0, "mlp", "shared", "count"), 2, "count"),
    (("norm", "kind"), "rms", "kind"),
    (("logit_scale",), 2.0, "logit_scale"),
])
def test_a_key_the_reader_does_not_know_is_refused_by_name(path, value, what):
    d = config("odd")
    at = d
    for k in path[:-1]:
        at = at[k]
    at[path[-1]] = value
    with pytest.raises(ConfigError, match=what):
        load_config(d)


@pytest.mark.parametrize("change, what", [
    (lambda d: d["layers"][0]["mixer"].update(kv_heads=4), "kv_heads"),
    (lambda d: d["layers"][0]["mixer"].update(v_mix=1), "v_mix"),
    (lambda d: d["layers"][3]["mixer"].update(vdim=15), "whose values it mixes in"),
    (lambda d: d["layers"][0]["mixer"]["rot"].update(dims=12), "dims"),
    (lambda d: d["layers"][0]["mixer"]["mask"].update(size=0), "size"),
    (lambda d: d["layers"][0]["mixer"]["mask"].update(keep_first=-1), "keep_first"),
    (lambda d: d["layers"][1]["mixer"].update(q_rank=0), "q_rank"),
    (lambda d: d["layers"][1]["mixer"]["rot"].update(dims=7), "dims"),
    (lambda d: d["layers"][0]["mlp"]["router"].update(top=5), "top"),
    (lambda d: d["layers"][0]["mlp"]["router"].update(identity=1), "groups"),
    (lambda d: d["layers"][0]["mlp"]["router"]["groups"].update(keep=4), "groups"),
    (lambda d: d["layers"][0]["mlp"]["expert"].update(ff=0), "ff"),
    (lambda d: d["layers"][0].update(type="mamba2"), "mamba2"),
    (lambda d: d["layers"][1]["mlp"].update(kind="gated"), "kind"),
    (lambda d: d.pop("postln_alpha"), "postln_alpha"),
    (lambda d: d.update(vocab=0), "vocab"),
])
def test_sizes_that_contradict_each_other_are_refused(change, what):
    d = config("odd")
    change(d)
    with pytest.raises(ConfigError, match=what):
        load_config(d)


def _expected_tensors(d):
    W = d["width"]
    out = {"embed": (d["vocab"], W)}
    for n in ("embed.norm", "final.norm"):
        out.update({n: (W,), n + ".b": (W,)})
    for i, layer in enumerate(d["layers"]):
        p, m, f = f"l{i}.", layer["mixer"], layer["mlp"]
        for n in ("1", "2") if f else ("1",):
            out.update({p + "norm" + n: (W,), p + "norm" + n + ".b": (W,)})
        x, H = p + "mix.", m["heads"]
        if layer["type"] == "attention":
            G, dk, dv = m["kv_heads"], m["dim"], m["vdim"]
            out.update({x + "q": (H * dk, W), x + "k": (G * dk, W), x + "v": (G * dv, W), x + "o": (W, H * dv), x + "g": (H, W),
                        x + "q.norm": (dk,), x + "k.norm": (dk,)})
            if m.get("v_mix"):
                out[x + "vmix"] = ()
        else:
            R = m["kv_rank"]
            out.update({x + "dq": (m["q_rank"], W), x + "dq.norm": (m["q_rank"],), x + "uq": (H * (m["dim"] + m["rot_dim"]), m["q_rank"]),
                        x + "dkv": (R + m["rot_dim"], W), x + "dkv.norm": (R,), x + "uk": (H * m["dim"], R), x + "uv": (H * m["vdim"], R),
                        x + "o": (W, H * m["vdim"])})
        if f and f["kind"] == "dense":
            out.update({p + "mlp.up": (f["ff"], W), p + "mlp.down": (W, f["ff"])})
        elif f:
            E, I, ff = f["router"]["experts"], f["router"].get("identity", 0), f["expert"]["ff"]
            out.update({p + "mlp.router": (E + I, W), p + "mlp.correction": (E + I,)})
            names = [(f"e{e}", ff) for e in range(E)] + ([("shared", f["shared"]["ff"])] if f.get("shared") else [])
            for n, width in names:
                out.update({f"{p}mlp.{n}.up": (width, W), f"{p}mlp.{n}.down": (W, width)})
    return out


@pytest.mark.parametrize("name", list(CONFIGS))
def test_the_model_asks_for_the_designs_tensors_by_name_and_shape(name):
    specs = build_model(load_config(config(name))).param_specs()
    assert {n: tuple(s.shape) for n, s in specs.items()} == _expected_tensors(config(name))


def test_the_memory_every_layer_gets():
    specs = build_model(load_config(config("odd"))).cache_specs()
    assert specs[0] == KVSpec(2, 10, WINDOW_SLIDING, 29, 14, keep_first=3)
    assert specs[1] == KVSpec(1, 30, WINDOW_SLIDING, 31, 24, values_in_keys=True)
    assert specs[2] == KVSpec(2, 16, WINDOW_SLIDING, 45) and specs[4] == KVSpec(1, 8, WINDOW_NONE, 0, 20)
    assert specs[6] == KVSpec(2, 12, WINDOW_SLIDING, 17, 14, keep_first=40) and specs[7] is None
    # layers whose pages live and die together share a table; the same window with and without kept tokens does not
    keys = [s.group_key() for s in specs if s is not None]
    assert len(set(keys)) == 6 and keys[4] == keys[5]
    assert KVSpec(1, 2, WINDOW_SLIDING, 8).group_key() != KVSpec(1, 2, WINDOW_SLIDING, 8, keep_first=1).group_key()


def test_keys_seen_and_pages_held_behind_a_window_that_keeps_first_tokens():
    s = KVSpec(1, 4, WINDOW_SLIDING, 10, keep_first=5)
    mask = P.visible(64, {"size": 10, "keep_first": 5})
    assert [s.keys_seen(p) for p in range(64)] == [int(mask[p].sum()) for p in range(64)]
    assert [KVSpec(1, 4, WINDOW_SLIDING, 10, keep_first=k).kept_blocks(16) for k in (0, 1, 16, 17, 40)] == [0, 1, 1, 2, 3]
    assert pages_to_hold(s, 16, 4096, 1) == pages_to_hold(KVSpec(1, 4, WINDOW_SLIDING, 10), 16, 4096, 1) + 1
    assert pages_to_hold(s, 16, 20, 1) == 2


@pytest.mark.parametrize("keep, window", [(1, 20), (16, 20), (17, 33), (40, 17), (5, 1)])
@pytest.mark.parametrize("cut", [1, 7, 32])
def test_pages_of_kept_tokens_stay_with_the_request_and_the_others_go_back(keep, window, cut):
    spec = KVSpec(1, 4, WINDOW_SLIDING, window, keep_first=keep)
    held = pages_to_hold(spec, 16, 400, cut)
    cache = CacheManager([spec], 16, {spec.group_key(): 2 * held}, 2, torch.float32, "cpu", allocate=False)
    assert cache.can_admit(400, cut)
    for r in ("a", "b"):
        cache.add_request(r, reserve_tokens=400, max_step_tokens=cut)
    at = 0
    while at < 400:
        n = min(cut, 400 - at)
        for r in ("a", "b"):
            assert cache.append(r, n), f"{held} pages a request do not reach at {at}"
            tbl = cache.block_table(r, 0)
            for p in range(at, at + n):                   # every key that a query of this step sees has a page
                for key in [k for k in range(p + 1) if p - k < window or k < keep]:
                    assert tbl[key // 16] >= 0
            cache.commit(r)
        at += n
        cache.check_invariants()
    tbl = cache.block_table("a", 0)
    kept, first = (keep + 15) // 16, (400 - window + 1) // 16
    assert all(p >= 0 for p in tbl[:kept]) and all(p == -1 for p in tbl[kept:max(kept, first)]) and all(p >= 0 for p in tbl[first:])
    for r in ("a", "b"):
        cache.free_request(r)
    assert cache.groups[0].pool.num_free == 2 * held
    cache.check_invariants()


def test_a_step_that_is_rolled_back_keeps_the_first_pages():
    spec = KVSpec(1, 4, WINDOW_SLIDING, 16, keep_first=4)
    cache = CacheManager([spec], 16, 8, 1, torch.float32, "cpu", allocate=False)
    cache.add_request("a")
    for n in (40, 40):
        assert cache.append("a", n)
        cache.commit("a")
    before = list(cache.block_table("a", 0))
    assert before[0] >= 0 and before[1] == before[2] == -1
    assert cache.append("a", 30)
    cache.rollback("a")
    assert cache.block_table("a", 0) == before and cache.length("a") == 80
    cache.check_invariants()
    with pytest.raises(CacheError):
        cache.add_request("a")


def test_pools_count_the_kept_pages():
    specs = build_model(load_config(config("odd"))).cache_specs()
    sizes = pool_sizes(specs, 16, 3, 1024, 8)
    assert sizes[("kv", WINDOW_SLIDING, 17, 40)] == 3 * (2 + 1 + 3) and sizes[("kv", WINDOW_SLIDING, 45)] == 3 * (4 + 1)
    assert sizes[("kv", WINDOW_NONE, 0)] == 3 * 64


def test_the_runs_of_a_decoded_token_fit_the_bound():
    """A token walks the 16-key blocks of its kept keys and of its window; the launch is sized by `decode_runs`."""
    for keep in (0, 1, 16, 17, 300):
        for window in (1, 2, 15, 16, 17, 72, 255, 256, 257, 1000):
            for p in list(range(0, 700)) + [4095, 4096, 9000]:
                start = max(0, p - window + 1)
                kept = (keep + 15) // 16
                blocks = p // 16 + 1 if p // 16 < kept else kept + p // 16 - max(start // 16, kept) + 1
                assert (blocks + 15) // 16 <= ops.decode_runs(p + 1, ops.WINDOW_SLIDING, window, keep), (keep, window, p)
    assert ops.decode_runs(100000, ops.WINDOW_SLIDING, 72, 4) == 1
    assert ops.decode_runs(700, ops.WINDOW_NONE, 0) == ops.decode_max_splits(700)


def test_parts_refuse_what_they_do_not_compute():
    kw = dict(qk_norm_eps=1e-5, qk_norm_weights="head")
    with pytest.raises(ValueError, match="keep_first"):
        Attention(64, 2, 2, 16, keep_first=3, **kw)
    with pytest.raises(ValueError, match="value_mix"):
        Attention(64, 2, 2, 16, value_mix="last", **kw)
    with pytest.raises(ValueError, match="shared values"):
        Attention(64, 2, 2, 16, value_mix="mixed", values_from_keys=True, **kw)
    with pytest.raises(ValueError, match="excludes"):
        Attention(64, 2, 2, 16, head_gate=True, gate=True)
    moe = dict(gate="softmax", score_on_input=False, gated=False, activation="relu2")
    with pytest.raises(ValueError, match="groups"):
        MoESwiGLU(64, 5, 2, 16, n_groups=3, keep_groups=1, identity=2, **moe)
    with pytest.raises(ValueError, match="activation"):
        MoESwiGLU(64, 4, 2, 16, **{**moe, "activation": "swish_clamp"})
    with pytest.raises(ValueError, match="inputs"):
        MoESwiGLU(64, 4, 2, 16, identity=1, **{**moe, "score_on_input": True})
    MoESwiGLU(64, 5, 2, 16, n_groups=3, keep_groups=1, identity=1, **moe)


def test_rows_of_split_halves_are_loaded_as_neighbours():
    """Rotating neighbours behind the reordered projection gives the reordered rotation of split halves, so scores stay."""
    H, dn, dr, R, r = 2, 3, 8, 5, 6
    part = LatentAttention(16, H, dn, dr, 4, R, Rotary(dr, 50.0, None, "half", r), 1e-5, 0.3, sink=False, gate=False, q_rank=7)
    order = part._pair_order()
    assert order.tolist() == [0, 3, 1, 4, 2, 5, 6, 7]
    gen = torch.Generator().manual_seed(1)
    w, x = torch.randn(H * (dn + dr), 7, generator=gen, dtype=torch.float64), torch.randn(9, 7, generator=gen, dtype=torch.float64)
    q, qp = (x @ w.T).view(9, H, dn + dr), (x @ part._query_rows(w).T).view(9, H, dn + dr)
    assert torch.equal(q[..., :dn], qp[..., :dn])
    cos, sin = P.rotation(torch.arange(9), 50.0, r, torch.float64)
    want = P.rotate_halves(q[..., dn:], cos, sin)
    u, v = qp[..., dn:dn + r:2], qp[..., dn + 1:dn + r:2]
    got = torch.cat([torch.stack([u * cos[:, None] - v * sin[:, None], v * cos[:, None] + u * sin[:, None]], -1).flatten(-2), qp[..., dn + r:]], -1)
    assert torch.allclose(got, want[..., order])
    wl = torch.randn(R + dr, 7, generator=gen)
    assert torch.equal(part._latent_rows(wl)[:R], wl[:R]) and torch.equal(part._latent_rows(wl)[R:], wl[R:][order])
    plain = LatentAttention(16, H, dn, dr, 4, R, Rotary(dr, 50.0, None, "interleaved", r), 1e-5, 0.3, sink=False, gate=False, q_rank=7)
    assert plain._pair_order() is None and plain._query_rows(w) is w


# ---------------------------------------------------------------------------
# the plain implementation's own identities
# ---------------------------------------------------------------------------
def test_the_small_pieces():
    x = torch.tensor([[1.0, 2.0, 6.0]], dtype=torch.float64)
    want = (x - 3.0) / math.sqrt((4 + 1 + 9) / 3 + 0.5) * 2.0 + 1.0
    assert torch.allclose(P.layer_norm(x, torch.full((3,), 2.0), torch.ones(3), 0.5), want)
    assert P.visible(9, {"size": 3, "keep_first": 2})[6].tolist() == [True, True, False, False, True, True, True, False, False]
    assert P.visible(9, {"size": 3})[6].tolist() == [False] * 4 + [True] * 3 + [False] * 2
    assert P.visible(9, {"size": 1, "keep_first": 4})[1].tolist() == [True, True] + [False] * 7
    z = torch.tensor([-3.0, -1.0, 0.0, 0.5, 2.0], dtype=torch.float64)
    assert torch.allclose(P.gelu(z), z * torch.distributions.Normal(0.0, 1.0).cdf(z).double(), atol=1e-6)
    assert P.relu2(z).tolist() == [0.0, 0.0, 0.0, 0.25, 4.0]
    x = torch.arange(10, dtype=torch.float64).reshape(1, 1, 10)
    c, s = torch.tensor([[0.0, 1.0, 0.0]], dtype=torch.float64), torch.tensor([[1.0, 0.0, 1.0]], dtype=torch.float64)
    assert P.rotate_halves(x, c, s)[0, 0].tolist() == [-3.0, 1.0, -5.0, 0.0, 4.0, 2.0, 6.0, 7.0, 8.0, 9.0]
    v, first = torch.tensor([2.0]), torch.tensor([6.0])
    assert float(P.mixed_values(v, first, 0.25)) == 3.0 and float(P.mixed_values(v, None, None)) == 2.0


def test_the_choice_of_experts():
    logits = torch.log(torch.tensor([[0.30, 0.05, 0.25, 0.20, 0.06, 0.14]], dtype=torch.float64))
    eye = torch.eye(6, dtype=torch.float64)
    none = torch.zeros(6, dtype=torch.float64)
    ids, wts = P.route(logits, eye, none, 2, None)
    assert ids.tolist() == [[0, 2]] and wts[0].tolist() == [pytest.approx(0.30), pytest.approx(0.25)]
    # groups rank by their single largest value: {0, 1} has the largest, although {2, 3} has the larger sum
    assert P.route(logits, eye, none, 2, {"count": 3, "keep": 1})[0].tolist() == [[0, 1]]
    # the correction moves the choice and the groups, not the weights; corrected values may all be negative
    corr = torch.tensor([-2.0, -2.0, -2.0, -2.0, -0.9, -1.9], dtype=torch.float64)
    ids, wts = P.route(logits, eye, corr, 2, {"count": 3, "keep": 1})
    assert ids.tolist() == [[4, 5]] and wts[0].tolist() == [pytest.approx(0.06), pytest.approx(0.14)]


def test_identity_experts_return_the_input():
    d = torch.float64
    W = 3
    w = {"p.router": torch.tensor([[0.0] * W, [1.0, 0, 0], [2.0, 0, 0]], dtype=d), "p.correction": torch.zeros(3, dtype=d),
         "p.e0.up": torch.eye(W, dtype=d), "p.e0.down": 2.0 * torch.eye(W, dtype=d)}
    h = torch.tensor([[1.0, -2.0, 3.0]], dtype=d)
    s = torch.softmax(torch.tensor([0.0, 1.0, 2.0], dtype=d), 0)
    f = {"router": {"experts": 1, "identity": 2, "top": 3}, "expert": {"ff": W}}
    want = (s[1] + s[2]) * h + s[0] * 2.0 * torch.tensor([[1.0, 0.0, 9.0]], dtype=d)
    assert torch.allclose(P.experts(h, w, "p.", f, h), want)
