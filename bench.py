#!/usr/bin/env python3
"""Serving benchmark on one MI355X: Llama 4 Scout-shaped layers, random bfloat16 weights.

    python bench.py [--gpus 1] [--steps K] [--warmup W] [--layers L] [--batch B]

A step is one decode step of a batch of B requests, each with a 2,048-token prompt already in
the cache.  Prints ONE JSON line: decoded tokens per second at the default batch, the prefill of
one 2,048-token prompt, the decode step's HBM roofline, and decode at batch 1 and 64 (with the
roofline fraction of each point), beside the peaks two measuring kernels of the library reach on
this GPU.  ``--profile`` adds, on stderr, milliseconds / bytes / GB/s per kernel class of one
prefill and one decode step, from event pairs.  ``--shape maverick8`` and ``--shape long16`` run
two other workloads instead (128 experts alternating with dense layers at batch 64; 32,768-token
prompts read in 4,096-token portions beside decoding requests) and print a JSON line of their own;
``--shape kuvonex`` runs Kuvonex layers (latent attention, routed experts in groups) at two sizes,
each beside Llama 4 layers of the same width, heads and experts, with the kernel-class tables of both;
``--shape pazatar`` does the same for Pazatar layers (attention that norms before it rotates, gated linear
attention beside it, dense feed-forwards) beside Llama 4 layers with dense feed-forwards;
``--shape nosedra`` runs Nosedra layers (attention with a learned sink beside a matrix memory with exponential
gates, state-space layers) beside Pazatar layers of the same sizes;
``--shape fovosun`` runs Fovosun layers (differential attention, retention, clamped routed experts, four
residual streams) beside Llama 4 layers of the same width, heads and experts;
``--shape pagonex`` runs Pagonex layers (the gated delta rule, latent attention behind a window, routed experts)
beside Kuvonex layers of the same width, heads and experts and Pazatar layers with the same recurrent heads;
``--shape rigodra`` runs Rigodra layers (attention that keeps the first tokens in its window beside latent attention, routed
experts without a gate with identity experts among them) beside Kuvonex and Llama 4 layers of the same width, heads and experts.
"""
from __future__ import annotations

import argparse
import json
import os
import random
import sys
import time

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

# published peaks of MI355X
PEAK_HBM_GBS = 8000.0
PEAK_DENSE_TFLOPS = {"bf16": 2500.0, "fp16": 2500.0, "fp8": 5000.0, "fp32": 157.3}

SCOUT = {
    "architectures": ["Llama4ForCausalLM"],
    "hidden_size": 5120, "num_hidden_layers": 48, "num_attention_heads": 40, "num_key_value_heads": 8,
    "head_dim": 128, "vocab_size": 202048,
    "intermediate_size": 8192, "intermediate_size_mlp": 16384,
    "num_local_experts": 16, "num_experts_per_tok": 1, "interleave_moe_layer_step": 1,
    "attention_chunk_size": 8192, "use_qk_norm": True, "attn_temperature_tuning": True,
    "floor_scale": 8192, "attn_scale": 0.1, "rms_norm_eps": 1e-5, "rope_theta": 500000.0,
    "rope_scaling": {"rope_type": "llama3", "factor": 16.0, "low_freq_factor": 1.0, "high_freq_factor": 4.0,
                     "original_max_position_embeddings": 8192},
    "tie_word_embeddings": False, "max_position_embeddings": 4096, "torch_dtype": "bfloat16",
}
FULL_LAYERS = 48
PROMPT_LEN = 2048
GEN_LEN = 256
CONTEXT = 4096


def log(msg: str) -> None:
    print(f"[bench] {msg}", file=sys.stderr, flush=True)


def build_engine(layers: int, max_batch: int, page_size: int, graphs: bool = True, gen_len: int = GEN_LEN,
                 prompt_len: int = PROMPT_LEN, overrides: dict = None, max_tokens_per_step: int = 8192, **engine_kw):
    from sharpinference_amd.engine import Engine

    cfg = dict(SCOUT)
    cfg.update(overrides or {})
    cfg["num_hidden_layers"] = layers
    cfg["no_rope_layers"] = [0 if (l + 1) % 4 == 0 else 1 for l in range(layers)]
    per_req = (prompt_len + gen_len + page_size - 1) // page_size * page_size + 2 * page_size   # (room for the run-ahead's own warm-up and the traced step)
    context = max(CONTEXT, per_req)
    cfg["max_position_embeddings"] = context
    t0 = time.time()
    eng = Engine(config=cfg, weight_seed=2, dtype="bfloat16", device="cuda:0", max_model_len=context,
                 max_num_seqs=max_batch, max_tokens_per_step=max_tokens_per_step, kv_tokens=max_batch * per_req,
                 page_size=page_size, decode_graphs=graphs, **engine_kw)
    log(f"engine with {layers} layers ready in {time.time() - t0:.1f}s")
    return eng


def layer_bytes(cfg) -> dict:
    """Bytes of the weights one decode step reads, by class (bfloat16)."""
    H, hd = cfg.hidden_size, cfg.head_dim
    q, kv = cfg.num_attention_heads * hd, cfg.num_key_value_heads * hd
    attn = 2 * ((q + 2 * kv) * H + H * q)
    expert = 2 * 3 * H * cfg.intermediate_size
    dense = 2 * 3 * H * cfg.intermediate_size_mlp
    router = 2 * cfg.num_local_experts * H
    norms = 2 * 2 * H
    head = 2 * cfg.vocab_size * H
    return {"attn": attn, "expert": expert, "dense": dense, "router": router, "norms": norms, "head": head,
            "kv_per_token": 2 * 2 * kv}


def decode_step_bytes(cfg, layers: int, batch: int, context: int, distinct: float) -> float:
    """Bytes one decode step has to read: every weight it uses once (the shared expert and
    `distinct` routed experts on a routed layer, the dense feed-forward on the others) and the
    cache of the live requests (what each layer's window lets the query at `context - 1` see)."""
    b = layer_bytes(cfg)
    total = b["head"]
    for l in range(layers):
        ffn = b["router"] + b["expert"] * (1 + distinct) if cfg.is_moe_layer(l) else b["dense"]
        total += b["attn"] + b["norms"] + ffn + batch * b["kv_per_token"] * visible_keys(cfg, l, context - 1)
    return total


def visible_keys(cfg, layer: int, position: int) -> int:
    """Keys the query at `position` sees in a layer: all before it, or those of its chunk."""
    if cfg.no_rope_layers[layer] == 0:
        return position + 1
    return position % cfg.attention_chunk_size + 1


def prefill_flops(cfg, T: int, layers: int) -> float:
    H, hd = cfg.hidden_size, cfg.head_dim
    q, kv = cfg.num_attention_heads * hd, cfg.num_key_value_heads * hd
    attn_lin = (q + 2 * kv) * H + H * q
    moe = cfg.num_local_experts * H + 2 * 3 * H * cfg.intermediate_size       # router, one routed expert, the shared one
    dense = 3 * H * cfg.intermediate_size_mlp
    lin = sum(attn_lin + (moe if cfg.is_moe_layer(l) else dense) for l in range(layers))
    C = cfg.attention_chunk_size
    whole, rest = divmod(T, C)
    pairs_chunked = whole * (C * (C + 1) / 2) + rest * (rest + 1) / 2       # (query, key) pairs, causal inside a chunk
    pairs = sum(T * (T + 1) / 2 if cfg.no_rope_layers[l] == 0 else pairs_chunked for l in range(layers))
    attn = 2 * 2 * cfg.num_attention_heads * hd * pairs                     # QK^T and PV
    return 2.0 * T * lin + attn + 2.0 * cfg.vocab_size * H                 # one row through the head


def prefill_bytes(cfg, layers: int, experts_used=None) -> float:
    """Weights a prompt of thousands of tokens has to read once: every expert of every routed layer
    (or `experts_used` of them a layer, where a prompt does not reach them all)."""
    b = layer_bytes(cfg)
    total = b["head"]
    used = cfg.num_local_experts if experts_used is None else experts_used
    for l in range(layers):
        total += b["attn"] + b["norms"] + (b["router"] + b["expert"] * (1 + used) if cfg.is_moe_layer(l) else b["dense"])
    return total


def run_prefill(eng, rid, prompt):
    import torch
    from sharpinference_amd.engine import StepEntry

    eng.add_request(rid)
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    logits = None
    for o in range(0, len(prompt), eng.max_tokens_per_step):     # a prompt longer than a step goes in portions
        part = prompt[o:o + eng.max_tokens_per_step]
        logits = eng.step([StepEntry(rid, part, (len(part) - 1,) if o + len(part) == len(prompt) else ())])
    torch.cuda.synchronize()
    return time.perf_counter() - t0, logits


def decode_run(eng, batch: int, steps: int, warmup: int, rng: random.Random, count_experts: bool = False,
               prompt_len: int = PROMPT_LEN):
    """Prefill `batch` prompts, then time `steps` decode steps.  Returns seconds, the mean
    number of distinct experts a step used per layer (if asked), the length the requests reached and
    the host's milliseconds per step."""
    import torch
    from sharpinference_amd import ops
    from sharpinference_amd.engine import StepEntry

    vocab = eng.config.vocab_size
    ids = [f"b{batch}_{i}" for i in range(batch)]
    last = []
    per_step = max(1, eng.max_tokens_per_step // prompt_len)
    for i in range(0, batch, per_step):
        group = ids[i:i + per_step]
        for r in group:
            eng.add_request(r)
        prompts = [[rng.randrange(vocab) for _ in range(prompt_len)] for _ in group]
        if prompt_len <= eng.max_tokens_per_step:
            lg = eng.step([StepEntry(r, p, (prompt_len - 1,)) for r, p in zip(group, prompts)])
        else:                                                # one prompt at a time, in portions of a step
            for o in range(0, prompt_len, eng.max_tokens_per_step):
                part = prompts[0][o:o + eng.max_tokens_per_step]
                lg = eng.step([StepEntry(group[0], part, (len(part) - 1,) if o + len(part) == prompt_len else ())])
        last += ops.argmax_rows(lg).cpu().tolist()
        log(f"  prefilled {min(i + per_step, batch)}/{batch}")

    host = [0.0]

    def one_step(tokens, trace=None):
        # greedy decoding as the engine serves it: the choice is made on the device behind the head.
        # The host's share of a step is what passes inside `step` (bookkeeping, the index arrays, the
        # launch); the wait for the chosen tokens after it is the GPU's.
        h0 = time.perf_counter()
        chosen = eng.step([StepEntry(r, (t,), (0,)) for r, t in zip(ids, tokens)], router_trace=trace, select="argmax")
        host[0] += time.perf_counter() - h0
        return chosen.cpu().tolist()

    def steps_on_end(tokens, n):
        # as the engine generates while every request decodes greedily: `decode_run_ahead` steps are
        # launched on end, each on what the one before chose, and their tokens read back together
        done = 0
        while done < n:
            chosen = eng.decode_steps([StepEntry(r, (t,), (0,)) for r, t in zip(ids, tokens)],
                                      min(eng.decode_run_ahead, n - done)).cpu().tolist()
            tokens = chosen[-1]
            done += len(chosen)
        return tokens

    for _ in range(warmup):
        last = one_step(last)
    if eng.decode_run_ahead > 1:
        last = steps_on_end(last, eng.decode_run_ahead)     # (the step's graph and buffers exist before the clock starts)
    host[0] = 0.0                            # two more, one by one, where the host's share of a step is measured
    for _ in range(2):
        last = one_step(last)
    host_ms = host[0] / 2 * 1e3
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    if eng.decode_run_ahead > 1:
        last = steps_on_end(last, steps)
    else:
        for _ in range(steps):
            last = one_step(last)
    torch.cuda.synchronize()
    dt = time.perf_counter() - t0
    distinct = None
    if count_experts:
        trace: list = []
        last = one_step(last, trace)
        distinct = sum(len(set(p.flatten().cpu().tolist())) for p, _, _ in trace) / max(1, len(trace))
    ctx = eng.cache.length(ids[0])
    for r in ids:
        eng.free_request(r)
    return dt, distinct, ctx, host_ms


def profile_report(eng, batch: int, prompt_len: int, rng: random.Random):
    """ms / bytes / GB/s / TFLOP/s per kernel class of one prefill and one decode step (stderr); returns the two tables."""
    from sharpinference_amd.engine import StepEntry
    from sharpinference_amd.ops.profile import Profiler, format_table

    vocab = eng.config.vocab_size
    ids = [f"prof{i}" for i in range(batch)]
    prof = Profiler()
    for n, r in enumerate(ids):
        eng.add_request(r)
        entry = [StepEntry(r, [rng.randrange(vocab) for _ in range(prompt_len)], (prompt_len - 1,))]
        if n == 0:
            eng.profiled_step(entry, prof)
        else:
            eng.step(entry)
    pre_table = prof.table()
    log("\n" + format_table(pre_table, f"prefill of one prompt of {prompt_len} tokens, by kernel class (event pairs):"))
    decode = [StepEntry(r, (rng.randrange(vocab),), (0,)) for r in ids]
    eng.step(decode, select="argmax")                       # warm
    prof = Profiler()
    decode = [StepEntry(r, (rng.randrange(vocab),), (0,)) for r in ids]
    eng.profiled_step(decode, prof, select="argmax", filler_ms=40.0)
    log("\n" + format_table(prof.table(), f"one decode step at batch {batch}, contexts of {prompt_len + 2} tokens, launched part by "
                                          "part behind filler work, by kernel class (event pairs):"))
    for r in ids:
        eng.free_request(r)
    return pre_table, prof.table()


def host_report(eng, prompt_len: int, rng: random.Random, batch: int = 64) -> dict:
    """What the host does in steps where nothing hides it (no steps launched on end, no choice on
    the device): a sampled batch (temperature alone; with top-k / top-p / min-p; with the window
    penalties) and a mixed step (one prompt-sized portion beside the others' decode tokens).
    Per case: milliseconds inside `Engine.step` (index arrays, launches), milliseconds of the
    sampler on an idle GPU (packing the rows' settings, two copies, the kernels, the read-back),
    and the wall time of a whole step.  stderr, and returned for the JSON line."""
    import torch
    from sharpinference_amd import SamplingParams
    from sharpinference_amd.engine import StepEntry
    from sharpinference_amd.sampling.sampler import penalty_window

    vocab = eng.config.vocab_size
    batch = min(batch, eng.max_num_seqs)
    ids = [f"host{i}" for i in range(batch)]
    history = {}
    per_step = max(1, eng.max_tokens_per_step // prompt_len)
    for i in range(0, batch, per_step):
        group = ids[i:i + per_step]
        entries = []
        for r in group:
            eng.add_request(r)
            history[r] = [rng.randrange(vocab) for _ in range(prompt_len)]
            entries.append(StepEntry(r, history[r], ()))
        eng.step(entries)
    cases = {
        "temperature": SamplingParams(temperature=0.8, top_k=0, top_p=1.0, min_p=0.0),
        "filters": SamplingParams(temperature=0.8, top_k=40, top_p=0.95, min_p=0.05),
        "penalties": SamplingParams(temperature=0.8, top_k=40, top_p=0.95, min_p=0.05, repetition_penalty=1.1,
                                    frequency_penalty=0.1, presence_penalty=0.1, penalty_last_n=64),
    }
    out = {}
    tokens = [rng.randrange(vocab) for _ in ids]
    for name, sp in cases.items():
        params = [SamplingParams(**{**sp.__dict__, "seed": 100 + i}) for i in range(batch)]
        t_step = t_sample = t_wall = 0.0
        n, warm = 6, 5       # (a wide batch's graph is captured when its shape has been met four times: within the warm-up)
        for it in range(n + warm):
            torch.cuda.synchronize()
            t0 = time.perf_counter()
            logits = eng.step([StepEntry(r, (t,), (0,)) for r, t in zip(ids, tokens)])
            t1 = time.perf_counter()
            hist = [penalty_window(p, history[r][:prompt_len], history[r][prompt_len:]) if p.edits_logits else ()
                    for p, r in zip(params, ids)]
            torch.cuda.synchronize()
            t2 = time.perf_counter()
            tokens = eng.sampler.sample(logits, params, [it] * batch, hist)
            t3 = time.perf_counter()
            for r, t in zip(ids, tokens):
                history[r].append(t)
            if it >= warm:
                t_step += t1 - t0
                t_sample += t3 - t2
                t_wall += t3 - t0
        out[name] = {"step_host_ms": t_step / n * 1e3, "sampler_ms": t_sample / n * 1e3, "step_ms": t_wall / n * 1e3}
        log(f"host, {batch} sampled rows ({name}): {out[name]['step_host_ms']:.2f} ms inside the step function, "
            f"{out[name]['sampler_ms']:.2f} ms in the sampler, of a step of {out[name]['step_ms']:.2f} ms")
    # a mixed step: one request leaves, a new prompt's portion comes in beside the others' decode tokens
    eng.free_request(ids[-1])
    portion = min(prompt_len, eng.max_tokens_per_step - (batch - 1))
    t_step = t_wall = 0.0
    n = 3
    for it in range(n + 1):
        rid = f"hostmix{it}"
        eng.add_request(rid)
        entries = [StepEntry(r, (t,), (0,)) for r, t in zip(ids[:-1], tokens[:-1])]
        entries.append(StepEntry(rid, [rng.randrange(vocab) for _ in range(portion)], (portion - 1,)))
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        picked = eng.step(entries, select="argmax")
        t1 = time.perf_counter()
        tokens = picked.cpu().tolist()[:batch - 1] + [0]
        t2 = time.perf_counter()
        eng.free_request(rid)
        if it >= 1:
            t_step += t1 - t0
            t_wall += t2 - t0
    out["mixed"] = {"step_host_ms": t_step / n * 1e3, "step_ms": t_wall / n * 1e3, "portion_tokens": portion,
                    "decode_tokens": batch - 1}
    log(f"host, mixed step ({portion} prompt tokens beside {batch - 1} decode tokens): {out['mixed']['step_host_ms']:.2f} ms "
        f"inside the step function (launches run ahead of the GPU), of a step of {out['mixed']['step_ms']:.2f} ms")
    for r in ids[:-1]:
        eng.free_request(r)
    return out


def run_maverick8(args) -> int:
    """Eight Maverick-shaped layers: dense feed-forward (16,384) alternating with 128 experts
    top-1 + shared, no rotary scaling, no QK norm; router weights drawn so that router logits are
    about N(0, 1) and the experts' load is uneven.  Batch 64 of 1,024-token prompts, 128 decode steps."""
    import torch
    from sharpinference_amd.engine import StepEntry

    layers, batch, P, steps, warm = 8, 64, 1024, args.steps if args.steps != GEN_LEN - 8 else 120, 8
    over = {"num_local_experts": 128, "interleave_moe_layer_step": 2, "rope_scaling": None, "use_qk_norm": False}
    eng = build_engine(layers, batch, args.page_size, gen_len=steps + warm + 2, prompt_len=P, overrides=over,
                       weight_std_by_suffix={"router.weight": 5120 ** -0.5})
    cfg = eng.config
    rng = random.Random(3)
    prompt = [rng.randrange(cfg.vocab_size) for _ in range(P)]
    run_prefill(eng, "warm", prompt)
    eng.free_request("warm")
    eng.add_request("load")
    trace: list = []
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    eng.step([StepEntry("load", prompt, (P - 1,))], router_trace=trace)
    torch.cuda.synchronize()
    pre_s = time.perf_counter() - t0
    eng.free_request("load")
    hist = torch.bincount(trace[0][0].flatten().long().cpu(), minlength=cfg.num_local_experts).tolist()
    log(f"prefill {P} tokens: {pre_s * 1e3:.1f} ms; tokens per expert in the first routed layer: min {min(hist)}, "
        f"median {sorted(hist)[len(hist) // 2]}, max {max(hist)}, unused {hist.count(0)} of {len(hist)}")
    dt, distinct, ctx, _ = decode_run(eng, batch, steps, warm, rng, count_experts=True, prompt_len=P)
    ms_step = dt / steps * 1e3
    step_bytes = decode_step_bytes(cfg, layers, batch, ctx, distinct)
    achieved = step_bytes / (ms_step * 1e-3) / 1e9
    log(f"decode b{batch}: {ms_step:.2f} ms/step, {batch * steps / dt:.1f} tok/s, {achieved:.0f} GB/s ({distinct:.1f} experts per routed layer)")
    out = {"metric": "decode tok/s at batch 64 (8 Maverick-shaped layers, 1,024-token prompts)", "value": batch * steps / dt,
           "unit": "tok/s", "n_gpus": 1, "steps": steps, "warmup": warm, "ms_per_step": ms_step, "higher_is_better": True,
           "scaling": "weak", "vs_baseline": None, "dtype": "bf16", "data": "synthetic",
           "config": {"model": "llama4-maverick-shaped-random", "global_batch": batch, "seq_len": eng.max_model_len,
                      "parallelism": "single-gpu", "layers": layers, "layers_of_full_model": 48, "hidden_size": cfg.hidden_size,
                      "heads": cfg.num_attention_heads, "kv_heads": cfg.num_key_value_heads, "head_dim": cfg.head_dim,
                      "experts": cfg.num_local_experts, "moe_every": cfg.interleave_moe_layer_step,
                      "expert_ffn": cfg.intermediate_size, "dense_ffn": cfg.intermediate_size_mlp, "vocab": cfg.vocab_size,
                      "prompt_len": P, "generated": steps + warm, "page_size": args.page_size},
           "prefill": {"value": P / pre_s, "tokens": P, "ms": pre_s * 1e3,
                       "frac": prefill_flops(cfg, P, layers) / pre_s / (PEAK_DENSE_TFLOPS["bf16"] * 1e12),
                       # with 8 tokens an expert the prompt is a stream of the weights it touches
                       "hbm_frac": prefill_bytes(cfg, layers, experts_used=len(hist) - hist.count(0)) / pre_s / 1e9 / PEAK_HBM_GBS},
           "roofline": {"bound": "hbm", "achieved": achieved, "peak": PEAK_HBM_GBS, "unit": "GB/s", "frac": achieved / PEAK_HBM_GBS},
           "expert_load": {"min": min(hist), "median": sorted(hist)[len(hist) // 2], "max": max(hist), "unused": hist.count(0),
                           "distinct_per_decode_step": distinct}}
    print(json.dumps(out), flush=True)
    return 0


def run_long16(args) -> int:
    """Sixteen Scout-shaped layers, 8 prompts of 32,768 tokens read in portions of 4,096 beside the
    decoded tokens of the requests that are already through (the scheduler mixes them), then
    decoding alone; 512 generated tokens a request.  Four chunk edges of 8,192 are crossed, the
    windowed layers give pages back behind them, and the query temperature works at long positions."""
    import torch
    from sharpinference_amd.engine import StepEntry
    from sharpinference_amd.engine.scheduler import Request, Scheduler
    from sharpinference_amd.sampling.params import SamplingParams

    layers, batch, P, portion = 16, 8, 32768, 4096
    gen = args.steps if args.steps != GEN_LEN - 8 else 512
    eng = build_engine(layers, batch, args.page_size, gen_len=gen + 8, prompt_len=P, max_tokens_per_step=portion + batch)
    cfg = eng.config
    rng = random.Random(4)
    sched = Scheduler(eng.cache, batch, portion + batch, eng.max_model_len)
    reqs = [Request(("long", i), [rng.randrange(cfg.vocab_size) for _ in range(P)],
                    SamplingParams(temperature=0.0, max_new_tokens=gen, stop_token_ids=())) for i in range(batch)]
    for r in reqs:
        sched.add(r)
    phases = {"mixed": [0.0, 0, 0, 0], "decode": [0.0, 0, 0, 0]}        # seconds, steps, prompt tokens, decoded tokens
    pools = {g.key: g.pool.num_pages for g in eng.cache.groups}
    distinct = None
    while sched.has_work():
        b = sched.schedule()
        if not b:
            break
        entries = [StepEntry(s.request.req_id, s.tokens, (len(s.tokens) - 1,) if s.samples else ()) for s in b]
        n_prompt = sum(len(s.tokens) for s in b if s.request.in_prefill)
        n_dec = sum(1 for s in b if not s.request.in_prefill)
        trace = [] if (not n_prompt and distinct is None) else None   # the first step of decoding alone says how many experts a step uses
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        picked = eng.step(entries, select="argmax", router_trace=trace)
        picked = picked.cpu().tolist() if picked is not None else []
        dt = time.perf_counter() - t0
        if trace:
            distinct = sum(len(set(p.flatten().cpu().tolist())) for p, _, _ in trace) / len(trace)
        it = iter(picked)
        sched.update(b, [next(it) if s.samples else None for s in b])
        ph = phases["mixed" if n_prompt else "decode"]
        ph[0] += dt; ph[1] += 1; ph[2] += n_prompt; ph[3] += n_dec
        if ph[1] % 64 == 0:
            log(f"  {ph[1]} {'mixed' if n_prompt else 'decode'} steps")
    mixed, dec = phases["mixed"], phases["decode"]
    assert all(r.finish_reason == "length" and len(r.output) == gen for r in reqs)
    ms_step = dec[0] / max(1, dec[1]) * 1e3
    ctx = P + gen
    # bytes of a decode step in the middle of the decoding phase
    from_trace = distinct if distinct is not None else 0.0
    step_bytes = decode_step_bytes(cfg, layers, dec[3] / max(1, dec[1]), ctx - gen // 2, from_trace)
    achieved = step_bytes / (ms_step * 1e-3) / 1e9
    log(f"mixed phase: {mixed[1]} steps, {mixed[2]} prompt tokens beside {mixed[3]} decoded tokens in {mixed[0]:.2f} s "
        f"({mixed[2] / mixed[0]:.0f} prompt tok/s); decode alone: {dec[1]} steps, {dec[3] / dec[0]:.1f} tok/s, {ms_step:.2f} ms/step")
    out = {"metric": "decode tok/s at batch 8 after 32,768-token prompts (16 Scout-shaped layers)", "value": dec[3] / dec[0],
           "unit": "tok/s", "n_gpus": 1, "steps": dec[1], "warmup": 0, "ms_per_step": ms_step, "higher_is_better": True,
           "scaling": "weak", "vs_baseline": None, "dtype": "bf16", "data": "synthetic",
           "config": {"model": "llama4-scout-shaped-random", "global_batch": batch, "seq_len": eng.max_model_len,
                      "parallelism": "single-gpu", "layers": layers, "layers_of_full_model": FULL_LAYERS,
                      "hidden_size": cfg.hidden_size, "heads": cfg.num_attention_heads, "kv_heads": cfg.num_key_value_heads,
                      "head_dim": cfg.head_dim, "experts": cfg.num_local_experts, "expert_ffn": cfg.intermediate_size,
                      "vocab": cfg.vocab_size, "attention_chunk": cfg.attention_chunk_size, "prompt_len": P,
                      "portion": portion, "generated": gen, "page_size": args.page_size},
           "prefill": {"value": mixed[2] / mixed[0], "tokens": mixed[2], "ms": mixed[0] * 1e3,
                       "frac": batch * prefill_flops(cfg, P, layers) / mixed[0] / (PEAK_DENSE_TFLOPS["bf16"] * 1e12),
                       "steps": mixed[1], "decoded_beside": mixed[3]},
           "roofline": {"bound": "hbm", "achieved": achieved, "peak": PEAK_HBM_GBS, "unit": "GB/s", "frac": achieved / PEAK_HBM_GBS,
                        "experts_per_step": from_trace},
           "pools": {f"window_{k[1]}_{k[2]}": v for k, v in pools.items()}}
    print(json.dumps(out), flush=True)
    return 0


# ---------------------------------------------------------------------------
# Kuvonex beside Llama 4 at equal sizes
# ---------------------------------------------------------------------------
# width, layers, heads, experts, picks, expert width, vocabulary; the latent layers take 128 + 64
# wide query heads over a latent of 512, the Llama 4 layers heads of 128 in groups of 8 over a key head
KUVONEX_SIZES = {
    "w2048": dict(width=2048, layers=4, heads=16, experts=64, top=6, ff=1408, groups=(8, 4), vocab=32000),
    "w4096": dict(width=4096, layers=2, heads=64, experts=32, top=4, ff=2048, groups=(4, 2), vocab=32000),
}


def kuvonex_config(z: dict) -> dict:
    mixer = {"heads": z["heads"], "dim": 128, "rot_dim": 64, "vdim": 128, "kv_rank": 512, "scale": 192 ** -0.5,
             "rot": {"base": 10000.0, "dims": 64}}
    mlp = {"kind": "moe", "expert": {"ff": z["ff"]},
           "router": {"experts": z["experts"], "top": z["top"], "groups": {"count": z["groups"][0], "keep": z["groups"][1]}}}
    layers = [{"type": "latent_attention", "mixer": dict(mixer), "mlp": mlp} for _ in range(z["layers"])]
    layers[-1]["mixer"]["kv_from"] = z["layers"] - 2          # the last layer attends over its neighbour's latents
    return {"architecture": "Kuvonex", "vocab": z["vocab"], "width": z["width"], "norm": {"eps": 1e-5},
            "embedding": {"scale": 1.0}, "layers": layers}


def llama4_config_like(z: dict) -> dict:
    cfg = dict(SCOUT)
    cfg.update({"hidden_size": z["width"], "num_hidden_layers": z["layers"], "num_attention_heads": z["heads"],
                "num_key_value_heads": max(1, z["heads"] // 8), "head_dim": 128, "vocab_size": z["vocab"],
                "intermediate_size": z["ff"], "intermediate_size_mlp": z["ff"], "num_local_experts": z["experts"],
                "num_experts_per_tok": z["top"], "interleave_moe_layer_step": 1, "rope_scaling": None,
                "no_rope_layers": [0 if (l + 1) % 4 == 0 else 1 for l in range(z["layers"])], "max_position_embeddings": CONTEXT})
    return cfg


def _beside(args, sizes: dict, pairs) -> tuple:
    """Prefill of one prompt and decode at batch 8 and 64 for every size and every (model, configuration
    maker) of `pairs`, with the per-kernel-class tables of one prefill and one decode step of each."""
    import torch
    from sharpinference_amd.engine import Engine

    P, steps, warm = args.prompt_len, min(args.steps, 48), 4
    per_req = (P + steps + warm + 16 + args.page_size - 1) // args.page_size * args.page_size + 2 * args.page_size
    rows = []
    for size, z in sizes.items():
        for model, make in pairs:
            cfg = make(z)
            t0 = time.time()
            eng = Engine(config=cfg, weight_seed=2, dtype="bfloat16", device="cuda:0", max_model_len=CONTEXT, max_num_seqs=64,
                         max_tokens_per_step=8192, kv_tokens=64 * per_req, page_size=args.page_size,
                         decode_graphs=not args.no_graphs)
            log(f"{model} {size}: engine ready in {time.time() - t0:.1f}s")
            rng = random.Random(5)
            prompt = [rng.randrange(z["vocab"]) for _ in range(P)]
            best = None
            for i in range(4):                                  # once to warm up, then three times timed
                dt, _ = run_prefill(eng, f"pre{i}", prompt)
                eng.free_request(f"pre{i}")
                best = dt if i and (best is None or dt < best) else best
            row = {"size": size, "model": model, "prefill_tok_s": P / best, "prefill_ms": best * 1e3}
            for batch in (8, 64):
                dt, _, ctx, host_ms = decode_run(eng, batch, steps, warm, rng, prompt_len=P)
                row[f"decode_b{batch}_tok_s"] = batch * steps / dt
                row[f"decode_b{batch}_ms_per_step"] = dt / steps * 1e3
            log(f"{model} {size}: prefill {row['prefill_ms']:.2f} ms ({row['prefill_tok_s']:.0f} tok/s), decode b8 "
                f"{row['decode_b8_ms_per_step']:.3f} ms/step, b64 {row['decode_b64_ms_per_step']:.3f} ms/step")
            pre, dec = profile_report(eng, 8, P, rng)
            row["prefill_classes"] = {k: {"ms": round(v["ms"], 4), "gbs": round(v["bytes"] / v["ms"] / 1e6, 1) if v["ms"] else 0,
                                          "tflops": round(v["flops"] / v["ms"] / 1e9, 2) if v["ms"] else 0} for k, v in pre.items()}
            row["decode_b8_classes"] = {k: {"ms": round(v["ms"], 4), "gbs": round(v["bytes"] / v["ms"] / 1e6, 1) if v["ms"] else 0}
                                        for k, v in dec.items()}
            rows.append(row)
            del eng
            torch.cuda.empty_cache()
    return rows, P, steps, warm


def run_kuvonex(args) -> int:
    """Prefill of one 2,048-token prompt and decode at batch 8 and 64 for the Kuvonex design at two
    sizes, each beside Llama 4 layers of the same width, heads, experts and expert width (random
    weights), with the per-kernel-class tables of one prefill and one decode step of both."""
    rows, P, steps, warm = _beside(args, KUVONEX_SIZES, (("kuvonex", kuvonex_config), ("llama4", llama4_config_like)))
    k0 = rows[0]
    out = {"metric": "decode tok/s at batch 8 (Kuvonex, width 2048, 4 layers, 2,048-token prompts)", "value": k0["decode_b8_tok_s"],
           "unit": "tok/s", "n_gpus": 1, "steps": steps, "warmup": warm, "ms_per_step": k0["decode_b8_ms_per_step"],
           "higher_is_better": True, "scaling": "weak", "vs_baseline": None, "dtype": "bf16", "data": "synthetic",
           "config": {"model": "kuvonex-random beside llama4-random at equal sizes", "global_batch": 8, "seq_len": CONTEXT,
                      "parallelism": "single-gpu", "prompt_len": P, "sizes": KUVONEX_SIZES},
           "rows": rows}
    print(json.dumps(out), flush=True)
    return 0


# ---------------------------------------------------------------------------
# Pazatar beside Llama 4 with dense feed-forwards at equal sizes
# ---------------------------------------------------------------------------
# width, layers (attention and parallel layers in turn), heads of 128 over kv heads, the gated linear mixer's heads of
# 128 key and 128 value channels, feed-forward width, vocabulary
PAZATAR_SIZES = {
    "w2048": dict(width=2048, layers=4, heads=16, kv_heads=4, ff=8192, vocab=32000, chunk=1024, decay_rank=64),
    "w4096": dict(width=4096, layers=2, heads=32, kv_heads=8, ff=14336, vocab=32000, chunk=1024, decay_rank=128),
}


def pazatar_config(z: dict) -> dict:
    attention = {"heads": z["heads"], "kv_heads": z["kv_heads"], "dim": 128, "vdim": 128, "scale": 128 ** -0.5,
                 "mask": {"size": z["chunk"]},
                 "rot": {"base": 10000.0, "dims": 128, "scaling": {"factor": 8.0, "original": 1024, "fast": 32.0, "slow": 1.0}}}
    left = {"heads": z["heads"], "kv_heads": z["kv_heads"], "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "conv": 4,
            "softcap": 50.0, "mask": {"size": z["chunk"] // 2},
            "rot": {"base": 20000.0, "dims": 64, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 2048}}}
    right = {"heads": z["heads"], "dim": 128, "vdim": 128, "tau": 16.0, "decay_rank": z["decay_rank"]}
    mlp = {"kind": "dense", "ff": z["ff"]}
    kinds = z.get("kinds") or ["attention" if i % 2 == 0 else "parallel" for i in range(z["layers"])]
    layers = [{"type": "attention", "mixer": attention, "mlp": mlp} if kind == "attention" else
              {"type": "parallel", "mixer": {"left": left, "right": right}, "mlp": mlp} for kind in kinds]
    return {"architecture": "Pazatar", "vocab": z["vocab"], "width": z["width"], "norm": {"eps": 1e-5}, "layers": layers,
            "loop": {"start": 0, "stop": z["layers"], "times": 1}}


def llama4_dense_like(z: dict) -> dict:
    """Llama 4 layers of the same width, heads and kv heads, every feed-forward dense (gated: three
    matrices of the width where the other design has two) and every layer chunked."""
    cfg = dict(SCOUT)
    cfg.update({"hidden_size": z["width"], "num_hidden_layers": z["layers"], "num_attention_heads": z["heads"],
                "num_key_value_heads": z["kv_heads"], "head_dim": 128, "vocab_size": z["vocab"],
                "intermediate_size": z["ff"], "intermediate_size_mlp": z["ff"], "num_local_experts": 1,
                "num_experts_per_tok": 1, "interleave_moe_layer_step": z["layers"] + 1, "rope_scaling": None,
                "attention_chunk_size": z["chunk"], "no_rope_layers": [1] * z["layers"], "max_position_embeddings": CONTEXT})
    return cfg


def run_pazatar(args) -> int:
    """Prefill of one 2,048-token prompt and decode at batch 8 and 64 for the Pazatar design at two
    sizes (attention layers and parallel layers in turn, random weights), each beside Llama 4
    layers of the same width and heads with dense feed-forwards, with the per-kernel-class tables
    of one prefill and one decode step of both."""
    rows, P, steps, warm = _beside(args, PAZATAR_SIZES, (("pazatar", pazatar_config), ("llama4", llama4_dense_like)))
    k0 = rows[0]
    out = {"metric": "decode tok/s at batch 8 (Pazatar, width 2048, 4 layers, 2,048-token prompts)", "value": k0["decode_b8_tok_s"],
           "unit": "tok/s", "n_gpus": 1, "steps": steps, "warmup": warm, "ms_per_step": k0["decode_b8_ms_per_step"],
           "higher_is_better": True, "scaling": "weak", "vs_baseline": None, "dtype": "bf16", "data": "synthetic",
           "config": {"model": "pazatar-random beside llama4-random (dense feed-forwards) at equal sizes", "global_batch": 8,
                      "seq_len": CONTEXT, "parallelism": "single-gpu", "prompt_len": P, "sizes": PAZATAR_SIZES},
           "rows": rows}
    print(json.dumps(out), flush=True)
    return 0


# ---------------------------------------------------------------------------
# Nosedra beside Pazatar at equal sizes
# ---------------------------------------------------------------------------
# width, layers (three parallel layers and a state-space layer in third place), attention heads of 128 over kv heads,
# the matrix memory's heads of 128 key and 128 value channels, the state space's heads of 64 values over a state of
# 128 in 8 groups (twice the width in all) behind four taps, feed-forward width, the token input's width, vocabulary
NOSEDRA_SIZES = {
    "w2048": dict(width=2048, layers=4, heads=16, kv_heads=4, ff=8192, vocab=32000, side=256, chunk=1024, decay_rank=64),
    "w4096": dict(width=4096, layers=4, heads=32, kv_heads=8, ff=14336, vocab=32000, side=256, chunk=1024, decay_rank=128),
}
NOSEDRA_KINDS = ["parallel", "parallel", "mamba2", "parallel"]


def nosedra_config(z: dict) -> dict:
    left = {"heads": z["heads"], "kv_heads": z["kv_heads"], "dim": 128, "vdim": 128, "scale": 128 ** -0.5,
            "rot": {"base": 1000000.0, "dims": 64, "scaling": {"factor": 4.0}}}
    right = {"heads": z["heads"], "dim": 128, "vdim": 128, "gate_cap": 10.0}
    space = {"heads": 2 * z["width"] // 64, "vdim": 64, "state": 128, "groups": 8, "conv": 4, "norm_groups": 8}
    mlp = {"kind": "dense", "ff": z["ff"]}
    layers = [{"type": "parallel", "mixer": {"left": left, "right": right, "left_scale": 1.0, "right_scale": 1.0}, "mlp": mlp}
              if kind == "parallel" else {"type": "mamba2", "mixer": space, "mlp": mlp} for kind in NOSEDRA_KINDS[:z["layers"]]]
    return {"architecture": "Nosedra", "vocab": z["vocab"], "width": z["width"], "norm": {"eps": 1e-5},
            "token_side": {"dim": z["side"]}, "logit_softcap": 50.0, "layers": layers}


def pazatar_like_nosedra(z: dict) -> dict:
    """Pazatar layers of the same width, heads and feed-forward width: a parallel layer (attention beside gated
    linear attention) where Nosedra has one, an attention layer where it has its state space."""
    return pazatar_config(dict(z, kinds=["parallel" if kind == "parallel" else "attention" for kind in NOSEDRA_KINDS[:z["layers"]]]))


def run_nosedra(args) -> int:
    """Prefill of one 2,048-token prompt and decode at batch 8 and 64 for the Nosedra design at two sizes
    (random weights), each beside Pazatar layers of the same width, heads and feed-forward width, with the
    per-kernel-class tables of one prefill and one decode step of both."""
    rows, P, steps, warm = _beside(args, NOSEDRA_SIZES, (("nosedra", nosedra_config), ("pazatar", pazatar_like_nosedra)))
    k0 = rows[0]
    out = {"metric": "decode tok/s at batch 8 (Nosedra, width 2048, 4 layers, 2,048-token prompts)", "value": k0["decode_b8_tok_s"],
           "unit": "tok/s", "n_gpus": 1, "steps": steps, "warmup": warm, "ms_per_step": k0["decode_b8_ms_per_step"],
           "higher_is_better": True, "scaling": "weak", "vs_baseline": None, "dtype": "bf16", "data": "synthetic",
           "config": {"model": "nosedra-random beside pazatar-random at equal sizes", "global_batch": 8, "seq_len": CONTEXT,
                      "parallelism": "single-gpu", "prompt_len": P, "sizes": NOSEDRA_SIZES},
           "rows": rows}
    print(json.dumps(out), flush=True)
    return 0


# ---------------------------------------------------------------------------
# Fovosun beside Llama 4 at equal sizes
# ---------------------------------------------------------------------------
# width, layers (differential attention with a window, behind a convolution, retention, with a window again), heads
# (two score maps of 64 over values of 128, where Llama 4 has heads of 128) in groups of 8 over a key head, retention
# heads of 128 key and 128 value channels, routed experts, picks, expert width (and a shared expert of that width with
# a limit of its own), four residual streams, vocabulary
FOVOSUN_SIZES = {
    "w2048": dict(width=2048, layers=4, heads=16, experts=64, top=6, ff=1408, vocab=32000, window=1024),
    "w4096": dict(width=4096, layers=4, heads=32, experts=32, top=4, ff=2048, vocab=32000, window=1024),
}
FOVOSUN_KINDS = ["attention_2", "attention", "retention", "attention_2"]


def fovosun_config(z: dict) -> dict:
    kv = max(1, z["heads"] // 8)
    windowed = {"heads": z["heads"], "kv_heads": kv, "dim": 64, "vdim": 128, "scale": 64 ** -0.5, "diff": 0.3,
                "rot": {"base": 10000.0, "dims": 64}, "mask": {"size": z["window"]}}
    conv = {"heads": z["heads"], "kv_heads": kv, "dim": 64, "vdim": 128, "scale": 64 ** -0.5, "diff": 0.3, "conv": 4,
            "q_temp": {"coef": 0.1, "every": 1024}}
    ret = {"heads": z["heads"], "dim": 128, "vdim": 128, "decay": [1.0 - 2.0 ** (-5 - 3 * h / z["heads"]) for h in range(z["heads"])],
           "rot": {"base": 1000000.0, "dims": 64}}
    mlp = {"kind": "moe", "expert": {"ff": z["ff"], "limit": 7.0}, "router": {"experts": z["experts"], "top": z["top"]},
           "shared": {"ff": z["ff"], "limit": 3.0}}
    mixers = {"attention_2": windowed, "attention": conv, "retention": ret}
    layers = [{"type": kind, "mixer": mixers[kind], "mlp": mlp} for kind in FOVOSUN_KINDS[:z["layers"]]]
    return {"architecture": "Fovosun", "vocab": z["vocab"], "width": z["width"], "norm": {"eps": 1e-5}, "embedding": {"scale": 1.0},
            "streams": 4, "layers": layers}


def llama4_like_fovosun(z: dict) -> dict:
    """Llama 4 layers of the same width, heads, kv heads, experts, picks and expert width, chunks of the window's size."""
    cfg = llama4_config_like(z)
    cfg.update({"attention_chunk_size": z["window"]})
    return cfg


def run_fovosun(args) -> int:
    """Prefill of one 2,048-token prompt and decode at batch 8 and 64 for the Fovosun design at two sizes
    (random weights), each beside Llama 4 layers of the same width, heads, experts and expert width, with the
    per-kernel-class tables of one prefill and one decode step of both."""
    rows, P, steps, warm = _beside(args, FOVOSUN_SIZES, (("fovosun", fovosun_config), ("llama4", llama4_like_fovosun)))
    k0 = rows[0]
    out = {"metric": "decode tok/s at batch 8 (Fovosun, width 2048, 4 layers, 2,048-token prompts)", "value": k0["decode_b8_tok_s"],
           "unit": "tok/s", "n_gpus": 1, "steps": steps, "warmup": warm, "ms_per_step": k0["decode_b8_ms_per_step"],
           "higher_is_better": True, "scaling": "weak", "vs_baseline": None, "dtype": "bf16", "data": "synthetic",
           "config": {"model": "fovosun-random beside llama4-random at equal sizes", "global_batch": 8, "seq_len": CONTEXT,
                      "parallelism": "single-gpu", "prompt_len": P, "sizes": FOVOSUN_SIZES},
           "rows": rows}
    print(json.dumps(out), flush=True)
    return 0


# ---------------------------------------------------------------------------
# Pagonex beside Kuvonex and Pazatar at equal sizes
# ---------------------------------------------------------------------------
# width, layers (delta rule, latent attention, latent attention over its neighbour's rows, delta rule), heads (of the
# latent layers: 128 + 64 wide over a latent of 512, queries through a latent of a quarter or half of the width), delta heads of
# 128 key and 128 value channels over half as many key heads, routed experts, picks, expert width (and a shared expert of
# that width with a limit of its own), vocabulary.  Kuvonex has the latent layers' like, Pazatar (one parallel layer in
# two, dense feed-forwards as wide as the picks together) the recurrence's
PAGONEX_SIZES = {
    "w2048": dict(width=2048, layers=4, heads=16, q_rank=768, delta_heads=16, experts=64, top=6, ff=1408, groups=(8, 4), vocab=32000,
                  window=1024, rank=128, kv_heads=4, chunk=1024, decay_rank=128),
    "w4096": dict(width=4096, layers=4, heads=64, q_rank=1536, delta_heads=32, experts=32, top=4, ff=2048, groups=(4, 2), vocab=32000,
                  window=1024, rank=128, kv_heads=8, chunk=1024, decay_rank=128),
}
PAGONEX_KINDS = ["channel_delta", "latent_attention", "latent_attention", "channel_delta"]


def pagonex_config(z: dict) -> dict:
    delta = {"heads": z["delta_heads"], "kv_heads": z["delta_heads"] // 2, "dim": 128, "vdim": 128, "conv": 4, "decay_rank": z["rank"],
             "gate_rank": z["rank"]}
    latent = {"heads": z["heads"], "dim": 128, "rot_dim": 64, "vdim": 128, "q_rank": z["q_rank"], "kv_rank": 512, "scale": 192 ** -0.5,
              "mask": {"size": z["window"]},
              "rot": {"base": 10000.0, "dims": 64, "scaling": {"factor": 8.0, "original": 1024, "fast": 32.0, "slow": 1.0}}}
    mlp = {"kind": "moe", "expert": {"ff": z["ff"], "limit": 7.0}, "router": {"experts": z["experts"], "top": z["top"], "scale": 2.5},
           "shared": {"ff": z["ff"], "limit": 3.0}}
    layers = [{"type": kind, "mixer": dict(delta if kind == "channel_delta" else latent), "mlp": mlp} for kind in PAGONEX_KINDS[:z["layers"]]]
    layers[2]["mixer"]["kv_from"] = 1
    return {"architecture": "Pagonex", "vocab": z["vocab"], "width": z["width"], "norm": {"eps": 1e-5}, "canon": {"taps": 4},
            "embedding": {"bigram": {"buckets": 100003, "mul_prev": 10007, "mul_cur": 257}}, "logit_scale": 1.0, "layers": layers}


def pazatar_like_pagonex(z: dict) -> dict:
    return pazatar_config(dict(z, heads=z["delta_heads"], ff=z["ff"] * z["top"]))


def run_pagonex(args) -> int:
    """Prefill of one 2,048-token prompt and decode at batch 8 and 64 for the Pagonex design at two sizes (random
    weights), each beside Kuvonex layers of the same width, heads, experts and expert width and Pazatar layers with the
    same recurrent heads, with the per-kernel-class tables of one prefill and one decode step of all."""
    pairs = (("pagonex", pagonex_config), ("kuvonex", kuvonex_config), ("pazatar", pazatar_like_pagonex))
    rows, P, steps, warm = _beside(args, PAGONEX_SIZES, pairs[:1] if args.alone else pairs)
    k0 = rows[0]
    out = {"metric": "decode tok/s at batch 8 (Pagonex, width 2048, 4 layers, 2,048-token prompts)", "value": k0["decode_b8_tok_s"],
           "unit": "tok/s", "n_gpus": 1, "steps": steps, "warmup": warm, "ms_per_step": k0["decode_b8_ms_per_step"],
           "higher_is_better": True, "scaling": "weak", "vs_baseline": None, "dtype": "bf16", "data": "synthetic",
           "config": {"model": "pagonex-random beside kuvonex-random and pazatar-random at equal sizes", "global_batch": 8,
                      "seq_len": CONTEXT, "parallelism": "single-gpu", "prompt_len": P, "sizes": PAGONEX_SIZES},
           "rows": rows}
    print(json.dumps(out), flush=True)
    return 0


# ---------------------------------------------------------------------------
# Rigodra beside Kuvonex and Llama 4 at equal sizes
# ---------------------------------------------------------------------------
# the sizes are Kuvonex's; `identity` of the router's `experts` outputs are identity experts.  Attention heads are 192
# wide with values of 128 (the width of a latent layer's heads) and share a key head by eights
RIGODRA_SIZES = {
    "w2048": dict(KUVONEX_SIZES["w2048"], identity=8, window=1024, keep=64, q_rank=768),
    "w4096": dict(KUVONEX_SIZES["w4096"], identity=4, window=1024, keep=64, q_rank=1536),
}
RIGODRA_KINDS = (("latent_attention", "moe"), ("attention", "moe"), ("attention", "moe"), ("latent_attention", "dense"))


def rigodra_config(z: dict) -> dict:
    latent = {"heads": z["heads"], "dim": 128, "rot_dim": 64, "vdim": 128, "q_rank": z["q_rank"], "kv_rank": 512, "scale": 192 ** -0.5,
              "mask": {"size": z["window"]}, "rot": {"base": 10000.0, "dims": 64}}
    attn = {"heads": z["heads"], "kv_heads": max(1, z["heads"] // 8), "dim": 192, "vdim": 128, "scale": 192 ** -0.5, "v_mix": True,
            "mask": {"size": z["window"], "keep_first": z["keep"]}, "rot": {"base": 10000.0, "dims": 64}}
    moe = {"kind": "moe", "expert": {"ff": z["ff"]}, "shared": {"ff": z["ff"]},
           "router": {"experts": z["experts"] - z["identity"], "top": z["top"], "identity": z["identity"],
                      "groups": {"count": z["groups"][0], "keep": z["groups"][1]}}}
    dense = {"kind": "dense", "ff": z["ff"] * z["top"]}
    layers = [{"type": kind, "mixer": dict(latent if kind == "latent_attention" else attn), "mlp": moe if ff == "moe" else dense}
              for kind, ff in RIGODRA_KINDS[:z["layers"]]]
    return {"architecture": "Rigodra", "vocab": z["vocab"], "width": z["width"], "norm": {"eps": 1e-5}, "postln_alpha": 1.7, "layers": layers}


def run_rigodra(args) -> int:
    """Prefill of one 2,048-token prompt and decode at batch 8 and 64 for the Rigodra design at two sizes (random
    weights), each beside Kuvonex and Llama 4 layers of the same width, heads, experts and expert width, with the
    per-kernel-class tables of one prefill and one decode step of all."""
    pairs = (("rigodra", rigodra_config), ("kuvonex", kuvonex_config), ("llama4", llama4_config_like))
    rows, P, steps, warm = _beside(args, RIGODRA_SIZES, pairs[:1] if args.alone else pairs)
    k0 = rows[0]
    out = {"metric": "decode tok/s at batch 8 (Rigodra, width 2048, 4 layers, 2,048-token prompts)", "value": k0["decode_b8_tok_s"],
           "unit": "tok/s", "n_gpus": 1, "steps": steps, "warmup": warm, "ms_per_step": k0["decode_b8_ms_per_step"],
           "higher_is_better": True, "scaling": "weak", "vs_baseline": None, "dtype": "bf16", "data": "synthetic",
           "config": {"model": "rigodra-random beside kuvonex-random and llama4-random at equal sizes", "global_batch": 8,
                      "seq_len": CONTEXT, "parallelism": "single-gpu", "prompt_len": P, "sizes": RIGODRA_SIZES},
           "rows": rows}
    print(json.dumps(out), flush=True)
    return 0


def main() -> int:
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=GEN_LEN - 8, help="timed decode steps (default: with the warm-up, the 256 generated tokens of the baseline's run)")
    ap.add_argument("--warmup", type=int, default=8)
    ap.add_argument("--layers", type=int, default=FULL_LAYERS)
    ap.add_argument("--batch", type=int, default=8)
    ap.add_argument("--page-size", type=int, default=16)
    ap.add_argument("--prompt-len", type=int, default=PROMPT_LEN, help="tokens of every prompt (the contract's run: 2,048)")
    ap.add_argument("--no-points", action="store_true", help="skip the batch-1 and batch-64 points")
    ap.add_argument("--no-graphs", action="store_true", help="launch decode steps kernel by kernel instead of replaying a HIP graph")
    ap.add_argument("--no-peaks", action="store_true", help="skip the two measuring kernels (pure read, matrix-core loop)")
    ap.add_argument("--profile", action="store_true", help="also print ms / bytes / GB/s per kernel class of one prefill and one decode step")
    ap.add_argument("--shape", default="scout", choices=["scout", "maverick8", "long16", "kuvonex", "pazatar", "nosedra", "fovosun", "pagonex", "rigodra"],
                    help="scout: the headline run; maverick8 / long16: two other workloads; kuvonex / pazatar: that design beside "
                         "Llama 4 layers of equal size; nosedra: that design beside Pazatar layers of equal size; fovosun: that design beside "
                         "Llama 4 layers of equal size; pagonex: that design beside Kuvonex and Pazatar layers of equal size; rigodra: that design "
                         "beside Kuvonex and Llama 4 layers of equal size; each prints a JSON "
                         "line of its own")
    ap.add_argument("--alone", action="store_true", help="--shape pagonex or rigodra without the models it is measured beside")
    args = ap.parse_args()
    if args.gpus != 1:
        print("bench.py measures one GPU: this engine has no multi-GPU path (N=1 only)")
        return 2
    if args.shape == "maverick8":
        return run_maverick8(args)
    if args.shape == "long16":
        return run_long16(args)
    if args.shape == "kuvonex":
        return run_kuvonex(args)
    if args.shape == "pazatar":
        return run_pazatar(args)
    if args.shape == "nosedra":
        return run_nosedra(args)
    if args.shape == "fovosun":
        return run_fovosun(args)
    if args.shape == "pagonex":
        return run_pagonex(args)
    if args.shape == "rigodra":
        return run_rigodra(args)

    import torch  # noqa: F401

    rng = random.Random(2)
    max_batch = args.batch if args.no_points else max(args.batch, 64)
    gen_len = max(GEN_LEN, args.warmup + args.steps + 2)      # warm-up, timed steps and the one traced step
    P = args.prompt_len
    eng = build_engine(args.layers, max_batch, args.page_size, graphs=not args.no_graphs, gen_len=gen_len, prompt_len=P)
    cfg = eng.config
    measured = None
    if not args.no_peaks:
        from sharpinference_amd import ops

        measured = ops.measured_peaks("cuda:0", read_bytes=2 << 30)
        log(f"measured on this GPU: pure read {measured['hbm_gbs']:.0f} GB/s (published {PEAK_HBM_GBS:.0f}), "
            f"matrix-core loop {measured['bf16_tflops']:.0f} TFLOP/s bf16 (published {PEAK_DENSE_TFLOPS['bf16']:.0f})")

    # prefill: one prompt (2,048 tokens) alone, once to warm up, then three times timed
    prompt = [rng.randrange(cfg.vocab_size) for _ in range(P)]
    run_prefill(eng, "warm", prompt)
    eng.free_request("warm")
    times = []
    for i in range(3):                                   # the median of three: a single run varies by a per cent or two
        t, _ = run_prefill(eng, f"timed{i}", prompt)
        eng.free_request(f"timed{i}")
        times.append(t)
    pre_s = sorted(times)[1]
    log(f"prefill {P} tokens: {pre_s * 1e3:.1f} ms")
    flops = prefill_flops(cfg, P, args.layers)
    prefill = {"value": P / pre_s, "tokens": P, "ms": pre_s * 1e3,
               "frac": flops / pre_s / (PEAK_DENSE_TFLOPS["bf16"] * 1e12),
               "hbm_frac": prefill_bytes(cfg, args.layers) / pre_s / 1e9 / PEAK_HBM_GBS}

    dt, distinct, ctx, host_ms = decode_run(eng, args.batch, args.steps, args.warmup, rng, count_experts=True, prompt_len=P)
    ms_step = dt / args.steps * 1e3
    value = args.batch * args.steps / dt
    step_bytes = decode_step_bytes(cfg, args.layers, args.batch, ctx, distinct)
    achieved = step_bytes / (ms_step * 1e-3) / 1e9
    log(f"decode b{args.batch}: {ms_step:.2f} ms/step ({host_ms:.2f} ms of it on the host), {value:.1f} tok/s, {achieved:.0f} GB/s "
        f"({distinct:.2f} experts per layer)")

    points, points_roofline, points_host = {}, {}, {}
    if not args.no_points:
        for pb in (1, 64):
            k = max(8, args.steps // 2)
            pdt, pdist, pctx, phost = decode_run(eng, pb, k, max(2, args.warmup // 2), rng, count_experts=True, prompt_len=P)
            points[f"decode_b{pb}"] = pb * k / pdt
            gbs = decode_step_bytes(cfg, args.layers, pb, pctx, pdist) / (pdt / k) / 1e9
            points_roofline[f"decode_b{pb}"] = gbs / PEAK_HBM_GBS
            points_host[f"decode_b{pb}"] = phost
            log(f"decode b{pb}: {pdt / k * 1e3:.2f} ms/step ({phost:.2f} ms on the host), "
                f"{points[f'decode_b{pb}']:.1f} tok/s, {gbs:.0f} GB/s "
                f"({gbs / PEAK_HBM_GBS:.3f} of the roofline; {pdist:.2f} experts per layer)")
    host_cases = None
    if args.profile:
        profile_report(eng, args.batch, P, rng)
        host_cases = host_report(eng, P, rng, batch=max_batch)

    out = {
        "metric": f"decode tok/s at batch {args.batch} (Scout-shaped, {P:,}-token prompts)",
        "value": value, "unit": "tok/s", "n_gpus": 1, "steps": args.steps, "warmup": args.warmup,
        "ms_per_step": ms_step, "higher_is_better": True, "scaling": "weak", "vs_baseline": None,
        "dtype": "bf16", "data": "synthetic",
        "config": {
            "model": "llama4-scout-shaped-random", "global_batch": args.batch, "seq_len": eng.max_model_len,
            "parallelism": "single-gpu", "layers": args.layers, "layers_of_full_model": FULL_LAYERS,
            "hidden_size": cfg.hidden_size, "heads": cfg.num_attention_heads, "kv_heads": cfg.num_key_value_heads,
            "head_dim": cfg.head_dim, "experts": cfg.num_local_experts, "experts_per_tok": cfg.num_experts_per_tok,
            "expert_ffn": cfg.intermediate_size, "shared_ffn": cfg.intermediate_size, "vocab": cfg.vocab_size,
            "attention_chunk": cfg.attention_chunk_size, "prompt_len": P,
            # decoded tokens a request: warm-up, the two steps that time the host, the run-ahead's own warm-up, the
            # timed steps and the traced one
            "generated": args.warmup + 2 + (eng.decode_run_ahead if eng.decode_run_ahead > 1 else 0) + args.steps + 1,
            "page_size": args.page_size,
        },
        "prefill": prefill,
        "roofline": {"bound": "hbm", "achieved": achieved, "peak": PEAK_HBM_GBS, "unit": "GB/s",
                     "frac": achieved / PEAK_HBM_GBS},
        "points": points,
        "points_roofline": points_roofline,
        "host_ms_per_step": host_ms,
        "points_host_ms_per_step": points_host,
    }
    if host_cases is not None:
        out["host_unhidden"] = {k: {a: round(b, 3) for a, b in v.items()} for k, v in host_cases.items()}
    if measured is not None:
        out["measured_peaks"] = {"hbm_gbs": measured["hbm_gbs"], "bf16_tflops": measured["bf16_tflops"],
                                 "roofline_frac_of_measured": achieved / measured["hbm_gbs"]}
    print(json.dumps(out), flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
