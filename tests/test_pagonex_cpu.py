"""Pagonex without a GPU: the configuration reader, the tensors the model asks for, the memory each layer
gets, and the plain implementation's own consistency (what the GPU tests lean on)."""
import math

import pytest
import torch

import plain_pagonex as P
from tiny_pagonex import CONFIGS, config

from sharpinference_amd import load_config
from sharpinference_amd.cache.manager import CacheManager, pool_sizes
from sharpinference_amd.cache.spec import WINDOW_NONE, WINDOW_SLIDING, KVSpec, StateSpec, kv_of, states_of
from sharpinference_amd.config.base import ConfigError
from sharpinference_amd.config.pagonex import PagonexConfig
from sharpinference_amd.parts.model import DecoderModel, Run
from sharpinference_amd.parts.position import YarnRotary, YarnScaling
from sharpinference_amd.registry import build_model, registered_architectures


def test_the_design_is_registered_and_its_configuration_round_trips():
    assert "Pagonex" in registered_architectures()
    for name in CONFIGS:
        cfg = load_config(config(name))
        assert isinstance(cfg, PagonexConfig)
        assert cfg.to_dict() == config(name)
        assert load_config(cfg.to_dict()) == cfg


def test_what_the_file_leaves_out_is_off():
    cfg = load_config(config("odd"))
    bare = cfg.layers[4].mixer
    assert bare.window is None and bare.rot is None and bare.kv_from is None
    assert cfg.layers[2].mlp is None and cfg.layers[1].mlp.shared_ff == 0
    wide = load_config(config("wide"))
    assert wide.bigram is None and build_model(wide).embedding is None
    assert wide.layers[3].mixer.rot.scaling is None
    d = config("odd")
    d["layers"][1]["mixer"].pop("kv_heads"), d["layers"][1]["mixer"].pop("vdim"), d.pop("logit_scale")
    d["layers"][0]["mixer"].pop("scale"), d["layers"][1]["mlp"]["router"].pop("scale")
    cfg = load_config(d)
    assert (cfg.layers[1].mixer.kv_heads, cfg.layers[1].mixer.vdim, cfg.logit_scale) == (6, 20, 1.0)
    assert cfg.layers[0].mixer.scale == pytest.approx(0.25) and cfg.layers[1].mlp.scale == 1.0


@pytest.mark.parametrize("path, value, what", [
    (("layers", 0, "mixer", "sink"), 1.0, "sink"),
    (("layers", 0, "mixer", "rot", "kind"), "half", "kind"),
    (("layers", 0, "mixer", "rot", "scaling", "low"), 1.0, "low"),
    (("layers", 0, "mixer", "mask", "kind"), "chunk", "kind"),
    (("layers", 1, "mixer", "tau"), 2.0, "tau"),
    (("layers", 1, "mlp", "router", "groups"), 2, "groups"),
    (("layers", 0, "mlp", "shared", "count"), 2, "count"),
    (("embedding", "scale"), 2.0, "scale"),
    (("embedding", "bigram", "trigram"), 2, "trigram"),
    (("canon", "bias"), True, "bias"),
    (("norm", "kind"), "rms", "kind"),
    (("loop",), {"start": 0}, "loop"),
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
    (lambda d: d["layers"][1]["mixer"].update(kv_heads=4), "kv_heads"),
    (lambda d: d["layers"][1]["mixer"].update(conv=0), "conv"),
    (lambda d: d["layers"][0]["mixer"]["rot"].update(dims=8), "dims"),
    (lambda d: d["layers"][0]["mixer"]["rot"]["scaling"].update(factor=0.0), "scaling"),
    (lambda d: d["layers"][0]["mixer"]["mask"].update(size=0), "size"),
    (lambda d: d["layers"][2]["mixer"].update(kv_from=1), "kv_from"),
    (lambda d: d["layers"][2]["mixer"].update(kv_from=4), "kv_from"),
    (lambda d: d["layers"][5]["mixer"].update(kv_from=2), "latent of its own"),
    (lambda d: d["layers"][2]["mixer"].update(kv_rank=25), "kv_rank"),
    (lambda d: d["layers"][2]["mixer"]["rot"].update(base=501.0), "rot"),
    (lambda d: d["layers"][0]["mixer"].update(q_rank=0), "q_rank"),
    (lambda d: d["layers"][0]["mlp"]["router"].update(top=6), "top"),
    (lambda d: d["layers"][0]["mlp"]["expert"].update(limit=0.0), "limit"),
    (lambda d: d["layers"][0]["mlp"]["shared"].update(limit=0.0), "limit"),
    (lambda d: d["layers"][0].update(type="mamba2"), "mamba2"),
    (lambda d: d["layers"][0]["mlp"].update(kind="dense"), "kind"),
    (lambda d: d["embedding"]["bigram"].update(buckets=0), "buckets"),
    (lambda d: d["canon"].update(taps=0), "canon"),
    (lambda d: d.update(vocab=0), "vocab"),
])
def test_sizes_that_contradict_each_other_are_refused(change, what):
    d = config("odd")
    change(d)
    with pytest.raises(ConfigError, match=what):
        load_config(d)


def _expected_tensors(d):
    W = d["width"]
    out = {"embed": (d["vocab"], W), "head": (d["vocab"], W), "final.norm": (W,), "final.norm.b": (W,)}
    if d.get("embedding"):
        out["bigram"] = (d["embedding"]["bigram"]["buckets"] + 1, W)
    for i, layer in enumerate(d["layers"]):
        p, m, f = f"l{i}.", layer["mixer"], layer["mlp"]
        for n in ("1", "2") if f else ("1",):
            out.update({p + "norm" + n: (W,), p + "norm" + n + ".b": (W,), p + "canon" + n: (W, d["canon"]["taps"])})
        x = p + "mix."
        if layer["type"] == "channel_delta":
            H, qk, kk, vv = m["heads"], m["kv_heads"] * m["dim"], m["heads"] * m["dim"], m["heads"] * m["vdim"]
            out.update({x + "q": (qk, W), x + "k": (qk, W), x + "v": (vv, W), x + "o": (W, vv), x + "b": (H, W), x + "A_log": (H,),
                        x + "norm": (m["vdim"],), x + "dt_bias": (kk,), x + "a1": (m["decay_rank"], W), x + "a2": (kk, m["decay_rank"]),
                        x + "g1": (m["gate_rank"], W), x + "g2": (vv, m["gate_rank"])})
            out.update({x + n + ".conv": (c, m["conv"]) for n, c in (("q", qk), ("k", qk), ("v", vv))})
        else:
            H, R = m["heads"], m["kv_rank"]
            out.update({x + "dq": (m["q_rank"], W), x + "dq.norm": (m["q_rank"],), x + "uq": (H * (m["dim"] + m["rot_dim"]), m["q_rank"]),
                        x + "uk": (H * m["dim"], R), x + "uv": (H * m["vdim"], R), x + "o": (W, H * m["vdim"])})
            if m.get("kv_from") is None:
                out.update({x + "dkv": (R + m["rot_dim"], W), x + "dkv.norm": (R,)})
        if f:
            E, ff = f["router"]["experts"], f["expert"]["ff"]
            out[p + "mlp.router"] = (E, W)
            names = [(f"e{e}", ff) for e in range(E)] + ([("shared", f["shared"]["ff"])] if f.get("shared") else [])
            for n, width in names:
                out.update({f"{p}mlp.{n}.gate": (width, W), f"{p}mlp.{n}.up": (width, W), f"{p}mlp.{n}.down": (W, width)})
    return out


@pytest.mark.parametrize("name", list(CONFIGS))
def test_the_model_asks_for_the_designs_tensors_by_name_and_shape(name):
    specs = build_model(load_config(config(name))).param_specs()
    want = _expected_tensors(config(name))
    assert {n: tuple(s.shape) for n, s in specs.items()} == want


def test_the_narrow_middles_come_from_the_tensors_shapes():
    d = config("odd")
    want = _expected_tensors(d)
    for layer in d["layers"]:
        layer["mixer"].pop("decay_rank", None), layer["mixer"].pop("gate_rank", None)
    cfg = load_config(d).with_tensor_shapes({n: (s, torch.bfloat16) for n, s in want.items()})
    assert (cfg.layers[1].mixer.decay_rank, cfg.layers[1].mixer.gate_rank) == (6, 10)
    assert (cfg.layers[3].mixer.decay_rank, cfg.layers[3].mixer.gate_rank) == (7, 5)
    assert {n: tuple(s.shape) for n, s in build_model(cfg).param_specs().items()} == want


def test_the_memory_every_layer_gets():
    from sharpinference_amd import ops

    f32 = torch.float32
    specs = build_model(load_config(config("odd"))).cache_specs()
    ring = StateSpec((3, 76), f32)
    # layer 2 (window 41) reads layer 0's rows, which are therefore kept for its wider window
    assert kv_of(specs[0]) == KVSpec(1, 30, WINDOW_SLIDING, 41, 24, values_in_keys=True) and states_of(specs[0]) == (ring, ring)
    assert kv_of(specs[1]) is None
    assert states_of(specs[1]) == (StateSpec(ops.delta_state_shape(6, 20, 12), f32), StateSpec((2, 2 * 40 + 72), f32), ring, ring)
    assert kv_of(specs[2]) is None and states_of(specs[2]) == (ring,)          # no pages of its own, no feed-forward
    # layer 4 sees everything: its rows are kept for good although layer 5 looks back 17 tokens only
    assert kv_of(specs[4]) == KVSpec(1, 26, WINDOW_NONE, 0, 18, values_in_keys=True) and kv_of(specs[5]) is None
    assert specs[6] == StateSpec((2,), torch.int32)                              # the previous token
    wide = build_model(load_config(config("wide"))).cache_specs()
    assert wide[0] == StateSpec(ops.delta_state_shape(2, 136, 40), f32) and len(wide) == 4       # one tap: nothing to keep
    assert wide[3] == KVSpec(1, 40, WINDOW_NONE, 0, 32, values_in_keys=True)


def test_rows_behind_the_widest_readers_window_are_given_back_and_states_start_from_zero():
    specs = build_model(load_config(config("even"))).cache_specs()
    sizes = pool_sizes(specs, 16, 2, 512, 32)
    cache = CacheManager(specs, 16, sizes, 2, torch.float32, "cpu")
    assert len(cache.groups) == 1 and cache.groups[0].spec.window == 100 and cache.groups[0].slots == [1]
    rc = cache.add_request("a")
    for _ in range(10):
        assert cache.append("a", 32)
        cache.commit("a")
    tbl = cache.block_table("a", 0)
    assert tbl[(320 - 99) // 16] >= 0 and tbl[(320 - 99) // 16 - 1] == -1
    for per in cache.states:
        for t in per:
            t[rc.state_slot].fill_(3)
    cache.free_request("a")
    rb = cache.add_request("b")
    assert rb.state_slot == rc.state_slot and not any(t[rb.state_slot].any() for per in cache.states for t in per)
    cache.check_invariants()


def test_a_schedule_that_reads_rows_nobody_has_stored_or_of_another_shape_is_refused():
    model = build_model(load_config(config("odd")))
    make = lambda schedule: DecoderModel(103, 76, model.blocks, model.final_norm, schedule=schedule)
    make([Run(0, 0), Run(2, 1, kv_from=0)])
    with pytest.raises(ValueError, match="before any entry"):
        make([Run(2, 0, kv_from=1), Run(0, 1)])
    with pytest.raises(ValueError, match="shape differs"):
        make([Run(4, 0), Run(2, 1, kv_from=0)])


def test_yarn_frequencies_and_their_magnitude():
    for base, dims, sc in ((500.0, 4, (3.0, 64, 8.0, 1.0)), (20000.0, 16, (8.0, 256, 32.0, 1.0)), (1e6, 64, (40.0, 4096, 32.0, 1.0)),
                           (100.0, 8, (1.0, 32, 4.0, 1.0)), (10000.0, 32, (16.0, 2048, 1.0, 1.0))):
        scaling = dict(zip(("factor", "original", "fast", "slow"), sc))
        y = YarnRotary(dims, base, YarnScaling(**scaling), "interleaved", dims)
        cos, sin = P.rotation(torch.tensor([1]), base, dims, scaling, torch.float64)
        mag = 0.1 * math.log(sc[0]) + 1.0
        assert y.magnitude == pytest.approx(mag)
        assert torch.allclose(y.frequencies().double(), torch.atan2(sin[0], cos[0]), rtol=1e-6, atol=1e-9)
        assert torch.allclose(cos[0] ** 2 + sin[0] ** 2, torch.full((dims // 2,), mag * mag, dtype=torch.float64))


def test_the_work_lists_of_the_chunked_form():
    import numpy as np

    from sharpinference_amd import ops
    from sharpinference_amd.parts.base import HostStep
    from sharpinference_amd.parts.delta_rule import DeltaChunks

    lens = [1, 40, 16, 17]
    cu = np.concatenate([[0], np.cumsum(lens)]).astype(np.int32)
    chunks, ents = ops.delta_chunks_of(lens, cu)
    assert chunks[:, :3].tolist() == [[0, 0, 1], [1, 1, 16], [1, 17, 16], [1, 33, 8], [2, 41, 16], [3, 57, 16], [3, 73, 1]]
    assert ents.tolist() == [[0, 1], [1, 3], [4, 1], [5, 2]]
    arrays, facts = DeltaChunks().plan(HostStep(3, 3, [1, 1, 1], [5, 9, 0], np.arange(4, dtype=np.int32)))
    assert facts["n"] == 0 and all(a.size == 0 for a in arrays)


def test_runs_of_a_window():
    from sharpinference_amd import ops

    for run in (32, 128, 1024):
        for window in (1, 2, 31, 72, 129, 130, 1000):
            for p in list(range(0, 400)) + [4095, 4096, 5000]:
                first = max(0, p - window + 1)
                held = p // run - first // run + 1
                rows, blocks = ops.latent_runs(p + 1, window, run)
                assert held <= rows
                last = p + ops.LATENT_BLOCK_TOKENS - 1
                assert last // run - first // run + 1 <= ops.latent_runs(last + 1, window, run)[1]
    assert ops.latent_runs(1000, 0, 128) == (8, 8) and ops.latent_runs(100, 5000, 128) == (1, 1)


# ---------------------------------------------------------------------------
# the plain implementation's own identities
# ---------------------------------------------------------------------------
def test_the_delta_rule_reads_its_own_write_replaces_what_a_key_held_and_carries_its_state():
    d = torch.float64
    k = torch.tensor([[[1.0, 0.0]], [[1.0, 0.0]], [[0.0, 1.0]]], dtype=d)
    q = torch.tensor([[[1.0, 0.0]], [[1.0, 0.0]], [[1.0, 0.0]]], dtype=d)
    v = torch.tensor([[[3.0]], [[5.0]], [[7.0]]], dtype=d)
    g = torch.ones(3, 1, 2, dtype=d)
    o, S = P.delta_rule(q, k, v, g, torch.ones(3, 1, dtype=d))
    assert o[:, 0, 0].tolist() == [3.0, 5.0, 5.0] and S[0, :, 0].tolist() == [5.0, 7.0]
    g[1] = torch.tensor([0.5, 1.0], dtype=d)                     # decays act on the rows before the key reads them
    o, _ = P.delta_rule(q, k, v, g, torch.tensor([[1.0], [0.5], [0.0]], dtype=d))
    assert o[:, 0, 0].tolist() == [3.0, 1.5 + 0.5 * (5.0 - 1.5), 1.5 + 0.5 * (5.0 - 1.5)]
    gen = torch.Generator().manual_seed(3)
    r = lambda *s: torch.randn(*s, generator=gen, dtype=d)
    q, k, v, g, b = r(9, 2, 4), P.unit_vector(r(9, 2, 4)), r(9, 2, 3), torch.sigmoid(r(9, 2, 4)), torch.sigmoid(r(9, 2))
    whole, S = P.delta_rule(q, k, v, g, b)
    one, S1 = P.delta_rule(q[:4], k[:4], v[:4], g[:4], b[:4])
    two, S2 = P.delta_rule(q[4:], k[4:], v[4:], g[4:], b[4:], S1)
    assert torch.allclose(torch.cat([one, two]), whole) and torch.allclose(S, S2)


def test_the_chunked_form_of_the_recurrence_is_the_recurrence():
    """The algebra the chunk kernels rest on, in double: the triangular system, the two score matrices, the moved state."""
    gen = torch.Generator().manual_seed(4)
    r = lambda *s: torch.randn(*s, generator=gen, dtype=torch.float64)
    C, d, e = 16, 6, 5
    q, k, v = r(C, d), P.unit_vector(r(C, d)), r(C, e)
    l = -torch.exp(r(C, d))
    beta = torch.sigmoid(r(C))
    S0 = r(d, e)
    b = torch.cumsum(l, 0)
    L, A = torch.zeros(C, C, dtype=torch.float64), torch.zeros(C, C, dtype=torch.float64)
    for t in range(C):
        for s in range(t + 1):
            x = k[s] * torch.exp(b[t] - b[s])
            L[t, s] = (k[t] * x).sum() if s < t else 0.0
            A[t, s] = (q[t] * x).sum()
    M = torch.linalg.inv(torch.eye(C, dtype=torch.float64) + beta[:, None] * L) * beta[None, :]
    U = M @ v - M @ (torch.exp(b) * k) @ S0
    o = (torch.exp(b) * q) @ S0 + A @ U
    S = torch.exp(b[-1])[:, None] * S0 + (torch.exp(b[-1] - b) * k).T @ U
    want, Sw = P.delta_rule(q[:, None], k[:, None], v[:, None], torch.exp(l)[:, None], beta[:, None], S0[None])
    assert torch.allclose(o, want[:, 0]) and torch.allclose(S, Sw[0])


def test_scores_through_the_latent_are_scores_through_expanded_keys():
    gen = torch.Generator().manual_seed(5)
    r = lambda *s: torch.randn(*s, generator=gen, dtype=torch.float64)
    W, m = 12, {"heads": 2, "dim": 4, "rot_dim": 4, "vdim": 3, "q_rank": 5, "kv_rank": 6, "scale": 0.4, "mask": {"size": 3},
                "rot": {"base": 50.0, "dims": 4, "scaling": {"factor": 2.0, "original": 16, "fast": 4.0, "slow": 1.0}}}
    w = {"p.dq": r(5, W), "p.dq.norm": r(5), "p.uq": r(16, 5), "p.dkv": r(10, W), "p.dkv.norm": r(6), "p.uk": r(8, 6), "p.uv": r(6, 6), "p.o": r(W, 6)}
    h = r(7, W)
    kept = P.latent_rows(h, w, "p.", m, 1e-5)
    got = P.latent_attention(h, w, "p.", m, 1e-5, kept)
    c, kr = kept
    cos, sin = P.rotation(torch.arange(7), 50.0, 4, m["rot"]["scaling"], torch.float64)
    q = (P.rms_norm(h @ w["p.dq"].T, w["p.dq.norm"], 1e-5) @ w["p.uq"].T).reshape(7, 2, 8)
    qr = P.rotate_pairs(q[..., 4:], cos, sin)
    out = []
    for i in range(2):
        key, val = c @ w["p.uk"][4 * i:4 * i + 4].T, c @ w["p.uv"][3 * i:3 * i + 3].T
        s = (q[:, i, :4] @ key.T + qr[:, i] @ kr[:, 0].T) * 0.4
        out.append(torch.softmax(s.masked_fill(~P.visible(7, 3), float("-inf")), -1) @ val)
    assert torch.allclose(got, torch.cat(out, -1) @ w["p.o"].T)


def test_the_small_pieces():
    x = torch.tensor([[1.0, 2.0, 6.0]], dtype=torch.float64)
    want = (x - 3.0) / math.sqrt((4 + 1 + 9) / 3 + 0.5) * 2.0 + 1.0
    assert torch.allclose(P.layer_norm(x, torch.full((3,), 2.0), torch.ones(3), 0.5), want)
    assert P.bigram_rows([4, 9, 2], 23, 11, 50) == [50, (4 * 23 + 99) % 50, (9 * 23 + 22) % 50]
    assert P.visible(9, 3)[5].tolist() == [False] * 3 + [True] * 3 + [False] * 3
    u = torch.arange(8, dtype=torch.float64).reshape(4, 2) + 1.0
    y = P.causal_conv(u, torch.tensor([[0.0, 0.0, 1.0], [1.0, 0.0, 0.0]], dtype=torch.float64))
    assert torch.equal(y[:, 0], u[:, 0]) and y[:, 1].tolist() == [0.0, 0.0, 2.0, 4.0]
    assert float(P.unit_vector(torch.zeros(3)).abs().max()) == 0.0
    h, router = torch.tensor([[1.0, 0.0]], dtype=torch.float64), torch.tensor([[2.0, 0], [1.0, 0], [3.0, 0]], dtype=torch.float64)
    ids, wts = P.route(h, router, 2, 1.5)
    assert ids.tolist() == [[2, 0]] and float(wts.sum()) == pytest.approx(1.5)
    assert torch.allclose(wts[0] / 1.5, torch.softmax(torch.tensor([3.0, 2.0], dtype=torch.float64), 0))
    assert P.route(h, router, 1, 0.7)[1].tolist() == [[pytest.approx(0.7)]]
