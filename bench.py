#!/usr/bin/env python3
"""Decode and prefill throughput of the engine on Llama-3.1-8B shapes with random weights.

  python bench.py [--gpus 1] [--steps K] [--warmup W] [--batch 8] [--context 2048] [--layers L]

A step is one decode step of the whole engine (schedule, batch upload, model, sampling, token ids back).
The engine is set up for sequences of up to 8,192 tokens (--max-context), page size 16; the timed decode steps
run with every sequence at 2,048 tokens (--context).
Prints one JSON line: `value` = decoded tokens per second at the given batch; `prefill` = a 2,048-token
prompt in one step; `roofline` = bytes a decode step has to read (every weight once, and the cache of the
live requests) over its time, against 8 TB/s, and beside it what a plain streaming read reaches on this card
(`measured_peak`); `points` = decode at batch 1 and 64.  The way of reporting
follows the reference's bench tool (bytes per token, effective GB/s, share of the peak:
tools/bench/src/roofline.rs:35-70).  Peaks: MI355X HBM3E 8 TB/s; dense bf16 MFMA 2.5 PFLOP/s."""
import argparse
import gc
import json
import os
import sys
import time

ROOT = os.path.dirname(os.path.abspath(__file__))
if ROOT not in sys.path:
    sys.path.insert(0, ROOT)

HBM_PEAK_GBS = 8000.0
PEAK_FLOPS = {"bf16": 2.5e15, "fp32": 157.3e12}


def build_engine(cfg_json, dtype, batch, context, extra_tokens, layers, seed=0, use_graphs=True, max_context=0,
                 chunk_tokens=2048, pool_tokens=0, set_layers=True):
    """An engine on random weights made directly on the GPU (no model folder is written for 16 GB)."""
    import torch

    from allpaca_amd.config import EngineConfig
    from allpaca_amd.engine.engine import Engine
    from allpaca_amd.models import DecoderModel, describe_model
    from allpaca_amd.parts import Runtime
    from allpaca_amd.weights import random_tensors

    if set_layers:
        cfg_json = dict(cfg_json, num_hidden_layers=layers)
    _, cfg, spec = describe_model(cfg_json)
    model = DecoderModel(spec)
    tdt = torch.bfloat16 if dtype == "bf16" else torch.float32
    page = 16
    # every sequence may grow to `max_context` tokens (positions, block table, pages of the pool)
    per_seq = -(-max(context + extra_tokens, max_context) // page) * page
    ec = EngineConfig(dtype="bfloat16" if dtype == "bf16" else "float32", page_tokens=page,
                      num_pages=(pool_tokens or batch * per_seq) // page + 8, max_active_requests=max(batch, 1),
                      max_batch_tokens=2048, chunk_tokens=chunk_tokens, use_graphs=use_graphs)
    rt = Runtime(torch.device("cuda:0"), tdt, per_seq)
    # weights tensor by tensor on the GPU: nothing of 16 GB passes through host memory
    specs = model.param_specs()
    tensors = {}
    for name, ps in specs.items():
        tensors.update(random_tensors({name: ps}, seed, tdt, 0.02, 0.0, device="cuda:0"))
    model.bind(tensors, rt)
    del tensors
    eng = Engine.from_model(cfg, model, ec)
    return cfg, eng


def weight_bytes(eng):
    """Bytes of every matrix and vector a decode step reads once (the embedding table is read row-wise, a few
    KB, and only counts if the head shares it)."""
    import torch

    from allpaca_amd.kernels.packing import PackedWeight
    seen, total = set(), 0

    def add(v):
        nonlocal total
        if isinstance(v, PackedWeight):
            v = v.data
        elif not isinstance(v, torch.Tensor) and isinstance(getattr(v, "data", None), torch.Tensor):
            v = v.data          # (the tiled matrices of a layer's experts)
        if isinstance(v, (tuple, list)):
            for x in v:
                add(x)
        elif isinstance(v, torch.Tensor) and v.dim() >= 1 and v.data_ptr() not in seen:
            seen.add(v.data_ptr())
            total += v.numel() * v.element_size()

    model = eng.model
    add(model.head.weight)
    add(model.final_norm.weight)
    for b in model.blocks:
        for part in b.parts.values():
            for v in vars(part).values():
                add(v)
    return total


def kv_bytes_per_token(eng):
    """Bytes of cache that one more token of a request takes over all layers: what the engine's own estimate of its
    cache says (`CacheEstimate`, from the needs that the model's parts state), a page's bytes over its positions."""
    import torch
    from allpaca_amd.cache import CacheEstimate
    page = eng.config.page_tokens
    elem = torch.empty((), dtype=eng.runner.storage.paged[0].dtype).element_size()
    est = CacheEstimate.of(eng.model.cache_needs(), page, elem)
    return est.bytes_per_page_of_every_group / page


def decode_during_prefill(batch, context, chunk=2048):
    """Tokens the first request may decode while the other prompts are still running in portions of `chunk`."""
    return batch * -(-context // chunk) + batch


def decode_run(eng, cfg, batch, context, steps, warmup, sampled=False):
    """Fills `batch` requests to `context` tokens, then times `steps` decode steps (greedy, or with `sampled` the
    request options' defaults: temperature 0.8, top-k 40, top-p 0.95)."""
    import numpy as np
    import torch

    from allpaca_amd.sampling import GenerationParams
    rng = np.random.default_rng(0)
    # requests that finish their prompt first decode while the others still prefill: leave room for that
    gp = GenerationParams(max_tokens=warmup + steps + decode_during_prefill(batch, context) + 8,
                          **({} if sampled else {"temperature": 0.0}))
    for _ in range(batch):
        eng.add_request(rng.integers(0, cfg.vocab_size, size=context - 1).tolist(), gp)
    while any(not r.decoding for r in eng.scheduler.running) or eng.scheduler.waiting:
        eng.step()
    for _ in range(warmup):
        eng.step()
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    n = 0
    produced = {}
    for _ in range(steps):
        events = eng.step()
        n += len(events)
        for ev in events:
            produced.setdefault(ev.request_id, []).append(ev.token_id)
    torch.cuda.synchronize()
    dt = time.perf_counter() - t0
    assert n == batch * steps, f"{n} tokens from {steps} steps of batch {batch}"
    for rid in list(eng.requests):
        eng.abort(rid)
    decode_run.ids_hash = ids_hash([produced[k] for k in sorted(produced)])   # of the timed steps' tokens
    return dt / steps


def prefill_run(eng, cfg, tokens, repeats=3):
    """One prompt of `tokens` tokens in one step (logits of its last row), best of `repeats`."""
    import numpy as np
    import torch

    from allpaca_amd.engine.batch import Entry
    rng = np.random.default_rng(1)
    best = None
    for i in range(repeats + 1):
        toks = rng.integers(0, cfg.vocab_size, size=tokens).tolist()
        eng.runner.admit(("prefill", i))
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        eng.runner.step([Entry(("prefill", i), toks, [tokens - 1])])
        torch.cuda.synchronize()
        dt = time.perf_counter() - t0
        eng.runner.release(("prefill", i))
        if i > 0:
            best = dt if best is None else min(best, dt)
    return best


def long_prefill_run(eng, cfg, tokens, portion, repeats=2):
    """One prompt of `tokens` tokens in steps of `portion` tokens (logits of its last row only), best of `repeats`.
    Returns the seconds of the whole prompt and of its last step."""
    import numpy as np
    import torch

    from allpaca_amd.engine.batch import Entry
    rng = np.random.default_rng(1)
    best = None
    for i in range(repeats + 1):
        toks = rng.integers(0, cfg.vocab_size, size=tokens).tolist()
        eng.runner.admit(("prompt", i))
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        for a in range(0, tokens, portion):
            part = toks[a:a + portion]
            if a + portion >= tokens:
                torch.cuda.synchronize()
                t_last = time.perf_counter()
            eng.runner.step([Entry(("prompt", i), part, [len(part) - 1] if a + portion >= tokens else [])])
        torch.cuda.synchronize()
        t1 = time.perf_counter()
        eng.runner.release(("prompt", i))
        if i > 0 and (best is None or t1 - t0 < best[0]):
            best = (t1 - t0, t1 - t_last)
    return best


def ids_hash(token_lists):
    """A short hash of produced token ids (requests in order): the same run gives the same hash."""
    import hashlib
    h = hashlib.sha256()
    for toks in token_lists:
        h.update((",".join(str(int(t)) for t in toks) + ";").encode())
    return h.hexdigest()[:16]


def requests_run(eng, cfg, n_requests, min_prompt, max_prompt, new_tokens, seed=0, sampled=False):
    """`n_requests` requests with prompts of random length arrive at once and run to `new_tokens` tokens each
    through the scheduler: portions of prompts beside decoding rows.  Returns a dict of totals and mean times."""
    import numpy as np
    import torch

    from allpaca_amd.sampling import GenerationParams
    rng = np.random.default_rng(seed)
    lengths = [int(x) for x in rng.integers(min_prompt, max_prompt + 1, size=n_requests)]
    # greedy, or the defaults of the request options (temperature 0.8, top-k 40, top-p 0.95)
    gp = GenerationParams(max_tokens=new_tokens) if sampled else GenerationParams(max_tokens=new_tokens, temperature=0.0)
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    ids = [eng.add_request(rng.integers(0, cfg.vocab_size, size=n).tolist(), gp) for n in lengths]
    reqs = [eng.requests[i] for i in ids]
    steps = 0
    while eng.has_unfinished():
        eng.step()
        steps += 1
    torch.cuda.synchronize()
    dt = time.perf_counter() - t0
    times = [r.timing() for r in reqs]
    out_tokens = sum(len(r.output) for r in reqs)
    assert out_tokens == n_requests * new_tokens, f"{out_tokens} tokens from {n_requests} requests"
    ttft = [1e3 * t["ttft"] for t in times]
    itl = [1e3 * t["itl"] for t in times]
    return {"seconds": dt, "steps": steps, "prompt_tokens": sum(lengths), "output_tokens": out_tokens,
            "ttft_ms": float(np.mean(ttft)), "itl_ms": float(np.mean(itl)),
            "ttft_p50_ms": float(np.percentile(ttft, 50)), "ttft_p95_ms": float(np.percentile(ttft, 95)),
            "itl_p50_ms": float(np.percentile(itl, 50)), "itl_p95_ms": float(np.percentile(itl, 95)),
            "ids_hash": ids_hash([r.output for r in reqs]),
            "preemptions": eng.scheduler.preemption_count}


def prefill_flops(cfg, layers, T):
    D, F, V = cfg.hidden_size, cfg.intermediate_size, cfg.vocab_size
    H, Hk, d = cfg.num_attention_heads, cfg.num_key_value_heads, cfg.head_dim
    linear = 2 * T * D * ((H + 2 * Hk) * d + H * d) + 2 * T * D * 3 * F
    attn = 2 * 2 * H * d * (T * (T + 1) // 2)
    return layers * (linear + attn) + 2 * D * V


# ---- per-kernel times (a pass of its own, never inside the measured steps) -----------------------------------
# entry point -> (indices of M, N, K among its int arguments, matrices read); N of the q/k/v product comes from its heads
_PRODUCTS = {
    "apc_skinny_gemm_bf16": ((2, 3, 4), 1), "apc_skinny_gemm_emit_bf16": ((2, 3, 4), 1),
    "apc_skinny_gemm_pre_bf16": ((3, 4, 5), 1), "apc_skinny_swiglu_bf16": ((2, 3, 4), 2),
    "apc_skinny_swiglu_pre_bf16": ((3, 4, 5), 2), "apc_gemm_bf16": ((2, 3, 4), 1), "apc_gemm_swiglu_bf16": ((2, 3, 4), 2),
    "apc_gemm_splitk_emit_bf16": ((2, 3, 4), 1), "apc_gemm_direct_emit_bf16": ((2, 3, 4), 1),
}


def _product_work(name, ints):
    """(rows, weight bytes read, flops) of one call of a matrix product's entry point, or None."""
    if name in _PRODUCTS:
        (m, n, k), mats = _PRODUCTS[name]
        M, N, K = ints[m], ints[n], ints[k]
    elif name in ("apc_skinny_qkv_rope_bf16", "apc_gemm_splitk_qkv_rope_bf16"):
        M, K, H, Hk, d = ints[3:8]
        N, mats = (H + 2 * Hk) * d, 1
    elif name in ("apc_gemm_pre_bf16", "apc_gemm_splitk_pre_bf16"):
        M, N, K, mode = ints[3:7]
        mats = 2 if mode == 3 else 1
    elif name == "apc_gemm_splitk_bf16":
        M, N, K, mode = ints[2:6]
        mats = 2 if mode == 3 else 1
    else:
        return None
    return M, mats * N * K * 2, 2 * mats * M * N * K


def kernel_table(totals, steps, attention_bytes=0, attention_flops=0):
    """Per entry point: calls and microseconds a step, and for the products and the attention what they read or
    compute and at what rate, against the published peaks."""
    rows = []
    for name, t in sorted(totals.items(), key=lambda kv: -kv[1]["us"]):
        r = {"kernel": name, "calls": round(t["calls"] / steps, 1), "us": round(t["us"] / steps, 1)}
        works = [_product_work(name, a) for a in t["args"]]
        nbytes = flops = 0
        if works and works[0] is not None:
            nbytes, flops = sum(w[1] for w in works) / steps, sum(w[2] for w in works) / steps
            r["rows"] = works[0][0]
        elif name == "apc_attention_decode_bf16":
            nbytes = attention_bytes
        elif name == "apc_attention_prefill_bf16":
            flops = attention_flops
        sec = t["us"] / steps * 1e-6
        if nbytes and (not flops or flops / nbytes < 300):     # below the ridge: bound by reading
            r.update({"GB": round(nbytes / 1e9, 3), "GB/s": round(nbytes / sec / 1e9, 1),
                      "frac_hbm": round(nbytes / sec / 1e9 / HBM_PEAK_GBS, 3)})
        elif flops:
            r.update({"TFLOP": round(flops / 1e12, 3), "TFLOP/s": round(flops / sec / 1e12, 1),
                      "frac_mfma": round(flops / sec / PEAK_FLOPS["bf16"], 3)})
        rows.append(r)
    return rows


def kernel_times(cfg_json, args, layers):
    """Event timers around every kernel launch of a decode step, a 2,048-token prefill and a mixed step (a portion of
    512 tokens beside the decoding rows), run eagerly in passes of their own; and the host's time to launch a mixed step."""
    import numpy as np
    import torch

    from allpaca_amd.engine.batch import Entry
    from allpaca_amd.kernels import lib as klib
    from allpaca_amd.sampling import GenerationParams
    B, ctx = args.batch, args.context
    cfg, eng = build_engine(cfg_json, args.dtype, B + 1, ctx, 600, layers, use_graphs=False, max_context=args.max_context)
    rng = np.random.default_rng(0)
    gp = GenerationParams(max_tokens=64, temperature=0.0)
    for _ in range(B):
        eng.add_request(rng.integers(0, cfg.vocab_size, size=ctx - 1).tolist(), gp)
    while any(not r.decoding for r in eng.scheduler.running) or eng.scheduler.waiting:
        eng.step()
    for _ in range(3):
        eng.step()
    out = {}
    steps = 4
    # The tables come from timers around the entry points as Python calls them, so these passes walk the model's
    # parts in Python (the same kernels with the same arguments as the compiled executor issues); the host's time to
    # launch a step is measured on both.
    native, eng.runner.native = eng.runner.native, None
    with klib.timing() as t:
        for _ in range(steps):
            eng.step()
    kv = kv_bytes_per_token(eng)
    out[f"decode_b{B}_ctx{ctx}"] = kernel_table(t.totals(), steps, attention_bytes=B * (ctx + 5) * kv)
    # a mixed step: a portion of a new prompt beside the B decoding rows, as long as the scheduler makes it (a chunk of
    # 512 tokens, cut back so that the step's rows are whole tiles); host time = until the launches are queued
    ids = [r.id for r in eng.scheduler.running]
    eng.runner.admit("mixed")
    tile = eng.scheduler.row_tile
    portion = 512
    if tile and 0 < (portion + B) % tile <= tile // 4:
        portion -= (portion + B) % tile
    mixed = lambda at: [Entry("mixed", rng.integers(0, cfg.vocab_size, size=portion).tolist(), [portion - 1])] + \
        [Entry(i, [1], [0]) for i in ids]
    def launch_time(reps=3):
        eng.runner.step(mixed(0))
        torch.cuda.synchronize()
        host, gpu = [], []
        for rep in range(reps):
            e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
            batch = mixed(rep)
            t0 = time.perf_counter()
            e0.record()
            eng.runner.step(batch)
            e1.record()
            host.append((time.perf_counter() - t0) * 1e6)
            e1.synchronize()
            gpu.append(e0.elapsed_time(e1) * 1e3)
        return round(min(host), 1), round(min(gpu), 1)

    walk_host, walk_gpu = launch_time()
    with klib.timing() as t:
        eng.runner.step(mixed(9))
    hd = cfg.num_attention_heads * cfg.head_dim
    out[f"mixed_{portion}_plus_b{B}"] = kernel_table(t.totals(), 1, attention_bytes=B * ctx * kv,
                                                     attention_flops=layers * 4 * hd * portion * (portion * 4 + portion // 2))
    eng.runner.native = native
    host, gpu = launch_time() if native is not None else (walk_host, walk_gpu)
    out["host_us_mixed_step"] = {"host_launch_us": host, "gpu_us": gpu, "executor": "compiled" if native is not None else "python",
                                 "python_walk_host_launch_us": walk_host, "python_walk_gpu_us": walk_gpu}
    eng.runner.native = None
    eng.runner.release("mixed")
    # prefill of 2,048 tokens in one step
    T = 2048
    eng.runner.admit("pf")
    eng.runner.step([Entry("pf", rng.integers(0, cfg.vocab_size, size=T).tolist(), [T - 1])])
    eng.runner.release("pf")
    eng.runner.admit("pf2")
    with klib.timing() as t:
        eng.runner.step([Entry("pf2", rng.integers(0, cfg.vocab_size, size=T).tolist(), [T - 1])])
    out[f"prefill_{T}"] = kernel_table(t.totals(), 1, attention_flops=layers * 4 * hd * (T * (T + 1) // 2))
    eng.runner.native = native
    return out


def sampler_times(vocab: int) -> dict:
    """Microseconds to choose the tokens of 1, 8 and 64 rows of random logits under four rules.  `gpu_us`: the
    kernels alone, their launches queued while the GPU is busy with something else (as a serving loop queues them
    behind the step), so that no waiting for the host is in it; `latency_us`: `Sampler.sample` from call to token ids
    on an idle GPU (parameters up, kernels, ids back)."""
    import torch
    from allpaca_amd.kernels import ops
    from allpaca_amd.sampling import GenerationParams
    from allpaca_amd.sampling.sampler import Sampler
    dev = torch.device("cuda:0")
    rules = {"greedy": dict(temperature=0.0, top_k=0, top_p=1.0),
             "temperature": dict(temperature=0.8, top_k=0, top_p=1.0),
             "top_k_40_top_p_0.95": dict(temperature=0.8, top_k=40, top_p=0.95),
             "top_p_0.95": dict(temperature=0.8, top_k=0, top_p=0.95)}
    busy = torch.randn(8192, 8192, device=dev)
    sampler = Sampler(dev, 0)
    out = {}
    for rows in (1, 8, 64):
        logits = torch.randn(rows, vocab, device=dev) * 3.0
        ids = torch.empty(rows, dtype=torch.int32, device=dev)
        u = torch.rand(rows, device=dev)
        for name, rule in rules.items():
            params = [GenerationParams(max_tokens=1, **rule) for _ in range(rows)]
            t = torch.full((rows,), rule["temperature"], device=dev)
            k = torch.full((rows,), rule["top_k"], dtype=torch.int32, device=dev)
            p = torch.full((rows,), rule["top_p"], device=dev)

            def kernels():
                if name == "greedy":
                    ops.argmax_rows(logits, ids)
                else:
                    ops.sample_rows(logits, t, k, p, u, ids, any_top_k=rule["top_k"] > 0, any_top_p=rule["top_p"] < 1.0,
                                    few_after_top_k=0 < rule["top_k"] <= 1024)
            calls = 20
            for _ in range(3):
                kernels()
                sampler.sample(logits, params, [0] * rows)
            e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
            for _ in range(6):
                busy @ busy                                   # a few milliseconds for the launches to queue behind
            e0.record()
            for _ in range(calls):
                kernels()
            e1.record()
            torch.cuda.synchronize()
            t0 = time.perf_counter()
            for i in range(calls):
                sampler.sample(logits, params, [i] * rows)
            wall = time.perf_counter() - t0
            out[f"b{rows}_{name}"] = {"gpu_us": round(e0.elapsed_time(e1) * 1e3 / calls, 1),
                                      "latency_us": round(wall * 1e6 / calls, 1)}
    return out


# ---- the Risizen design beside the llama decoder at equal sizes ---------------------------------------------------
# name -> width, heads, kv heads, head size (keys and values alike), feed-forward width, vocabulary
DESIGN_SIZES = {"1b": (2048, 32, 8, 64, 8192, 128256), "8b": (4096, 32, 8, 128, 14336, 128256)}
# entry points of the new design -> the like entry points of the llama decoder
LIKE_KERNELS = {
    "apc_conv_heads_bf16": ["apc_rope_kv_write_bf16", "apc_rope_kv_write"],
    "apc_attention_masked_prefill_bf16": ["apc_attention_prefill_bf16"],
    "apc_attention_masked_decode_bf16": ["apc_attention_decode_bf16"],
    "apc_streams_step": ["apc_rmsnorm_rows"],
    "apc_embed_streams": ["apc_embed_rows", "apc_embed_rows_tiled"],
    "apc_clamped_glu": ["apc_gemm_swiglu_bf16", "apc_skinny_swiglu_bf16", "apc_skinny_swiglu_pre_bf16"],
}


def design_configs(size: str, layers: int, chunk: int, streams: int = 2, taps: int = 4):
    D, H, G, d, F, V = DESIGN_SIZES[size]
    mixer = dict(heads=H, kv_heads=G, dim=d, vdim=d, scale=d ** -0.5, conv=taps, mask=dict(size=chunk))
    risizen = dict(architecture="Risizen", vocab=V, width=D, streams=streams, norm=dict(eps=1e-6), logit_scale=1.0,
                   layers=[dict(type="attention", mixer=dict(mixer), mlp=dict(kind="dense", ff=F, limit=7.0))
                           for _ in range(layers)])
    llama = dict(architectures=["LlamaForCausalLM"], model_type="llama", vocab_size=V, hidden_size=D,
                 num_hidden_layers=layers, num_attention_heads=H, num_key_value_heads=G, head_dim=d,
                 intermediate_size=F, rms_norm_eps=1e-6, rope_theta=500000.0, rope_scaling=None,
                 tie_word_embeddings=False, max_position_embeddings=8192, hidden_act="silu")
    return {"risizen": risizen, "llama": llama}


# ---- the Gulidra design beside the llama decoder at equal sizes ---------------------------------------------------
GULIDRA_LIKE_KERNELS = {
    "apc_conv_heads_bf16": ["apc_rope_kv_write_bf16", "apc_rope_kv_write"],
    "apc_attention_masked_prefill_bf16": ["apc_attention_prefill_bf16"],
    "apc_attention_masked_decode_bf16": ["apc_attention_decode_bf16"],
    "apc_linear_attention_bf16": ["apc_attention_prefill_bf16"],
    "apc_linear_attention": ["apc_attention_decode_bf16"],
    "apc_routed_experts_bf16": ["apc_gemm_swiglu_bf16", "apc_skinny_swiglu_bf16", "apc_skinny_swiglu_pre_bf16"],
    "apc_rmsnorm_add": ["apc_rmsnorm_rows"],
    "apc_embed_positions": ["apc_embed_rows", "apc_embed_rows_tiled"],
    "apc_diff_combine": [],
    "apc_gated_rmsnorm": [],
    "apc_route_topk": [],
}
GULIDRA_EXPERTS, GULIDRA_IDENTITY, GULIDRA_TOP = 8, 1, 2


def gulidra_configs(size: str, context: int, taps: int = 4):
    """Four layers at the widths of `size`: differential attention (two maps of half a head each, values of a whole
    head) with a dense feed-forward, linear attention with routed experts (2 of 8 + 1, each half as wide as the dense
    feed-forward: the same arithmetic a row), an attention that borrows the first one's keys with routed experts, and
    an attention of its own with a dense feed-forward; the llama decoder with four layers of the same widths."""
    D, H, G, d, F, V = DESIGN_SIZES[size]
    att = dict(heads=H, kv_heads=G, dim=d // 2, vdim=d, scale=(d // 2) ** -0.5, diff=0.3, conv=taps)
    lin = dict(heads=H, dim=d, vdim=d, decay=[1.0 - 2.0 ** -(5 + 3 * i / max(1, H - 1)) for i in range(H)])
    moe = dict(kind="moe", expert=dict(ff=F // GULIDRA_TOP),
               router=dict(experts=GULIDRA_EXPERTS, identity=GULIDRA_IDENTITY, top=GULIDRA_TOP))
    dense = dict(kind="dense", ff=F)
    gulidra = dict(architecture="Gulidra", vocab=V, width=D, max_positions=2 * context + 4096, embedding=dict(scale=1.0),
                   residual_mult=0.5, norm=dict(eps=1e-6),
                   layers=[dict(type="attention", mixer=dict(att), mlp=dense),
                           dict(type="lightning", mixer=lin, mlp=moe),
                           dict(type="attention", mixer=dict(att, kv_from=0), mlp=moe),
                           dict(type="attention", mixer=dict(att), mlp=dense)])
    return {"gulidra": gulidra, "llama": design_configs(size, 4, 2 * context)["llama"]}


def gulidra_rooflines(size, batch, context, T, points):
    """For the kernels the design adds and their like kernels of the llama decoder: the bytes or the arithmetic of the
    launches of a step over the measured time, as a share of the GPU's peak (8 TB/s, 2.5 PFLOP/s)."""
    D, H, G, d, F, V = DESIGN_SIZES[size]
    Fe, E, K = F // GULIDRA_TOP, GULIDRA_EXPERTS, GULIDRA_TOP

    def work(name, model, rows, keys_sum):
        """(bytes, flops) of all of a step's launches of entry point `name` in `model`."""
        att_own, att_all, lin, moe, layers = (2, 3, 1, 2, 4) if model == "gulidra" else (4, 4, 0, 0, 4)
        if name == "apc_conv_heads_bf16":        # rows read, q and the pages' rows written (a borrower: q alone)
            own, q = (H + 2 * G) * d, H * d
            return rows * (att_own * (own + q + 2 * G * d) + (att_all - att_own) * 2 * q) * 2, 0
        if name in ("apc_rope_kv_write_bf16", "apc_rope_kv_write"):
            return layers * rows * ((H + 2 * G) * d + H * d + 2 * G * d) * 2, 0
        if name == "apc_attention_masked_prefill_bf16":      # two maps of d / 2 a head, each over values of d
            return 0, att_all * keys_sum * H * 2 * (2 * (d // 2) + 2 * d)
        if name == "apc_attention_prefill_bf16":
            return 0, att_all * 4 * keys_sum * H * d
        if name in ("apc_attention_masked_decode_bf16", "apc_attention_decode_bf16"):
            return att_all * keys_sum * G * 2 * d * 2, 0
        if name == "apc_linear_attention_bf16":      # a row: scores with and weights over half a chunk of 64 on
            return 0, lin * rows * H * 2 * (32 * d + 32 * d + 2 * d * d)      # average, the state read and moved on
        if name == "apc_linear_attention":           # the state of every row read and written
            return lin * rows * H * d * d * 4 * 2, 0
        if name == "apc_routed_experts_bf16":
            used = min(E, rows * K)
            return moe * used * 3 * Fe * D * 2, moe * rows * K * 3 * 2 * Fe * D
        if name in ("apc_gemm_swiglu_bf16", "apc_skinny_swiglu_bf16", "apc_skinny_swiglu_pre_bf16"):
            return layers * 2 * F * D * 2, layers * rows * 2 * 2 * F * D
        if name == "apc_rmsnorm_add":                # y and x read, x and its copy written
            return (2 * layers) * rows * D * (4 + 4 + 4 + 2), 0
        if name == "apc_rmsnorm_rows":
            return (2 * layers + 1) * rows * D * (4 + 2), 0
        return None

    table = {}
    for phase, rows, keys_sum in (("prefill", T, T * (T + 1) // 2), ("decode", batch, batch * context)):
        for new, likes in GULIDRA_LIKE_KERNELS.items():
            row = {}
            for model, names in (("gulidra", [new]), ("llama", likes)):
                us = sum(points[model][phase + "_kernels_us"].get(n, 0.0) for n in names)
                name = next((n for n in names if n in points[model][phase + "_kernels_us"]), None)
                if not us or name is None:
                    continue
                w = work(name, model, rows, keys_sum)
                row[model] = {"us": round(us, 1)}
                if w:
                    row[model]["share_of_peak"] = round(max(w[0] / (us * 1e-6) / (HBM_PEAK_GBS * 1e9),
                                                            w[1] / (us * 1e-6) / PEAK_FLOPS["bf16"]), 4)
            if row:
                table[f"{phase}: {new}"] = row
    return table


def gulidra_run(args) -> int:
    T, batch, context = 2048, args.batch, args.context
    out = {"metric": "Gulidra beside the llama decoder at equal sizes: prefill tok/s (one prompt of 2048 tokens) and "
                     f"decode tok/s (batch {batch}, context {context})", "unit": "tok/s", "n_gpus": 1,
           "dtype": args.dtype, "data": "synthetic: random N(0, 0.02) weights, uniform random token ids",
           "config": {"layers": "attention + dense, linear attention + experts, borrowing attention + experts, "
                                "attention + dense", "experts": GULIDRA_EXPERTS, "identity": GULIDRA_IDENTITY,
                      "top": GULIDRA_TOP, "conv_taps": 4, "page_tokens": 16},
           "sizes": {}}
    for size in args.design_sizes.split(","):
        cfgs = gulidra_configs(size, context)
        points = {m: design_point(c, args.dtype, batch, context, args.steps, args.warmup, T) for m, c in cfgs.items()}
        out["sizes"][size] = {
            "shape": dict(zip(("width", "heads", "kv_heads", "head_size", "ff", "vocab"), DESIGN_SIZES[size])),
            **points,
            "prefill_gulidra_over_llama": round(points["gulidra"]["prefill_tok_s"] / points["llama"]["prefill_tok_s"], 3),
            "decode_gulidra_over_llama": round(points["gulidra"]["decode_tok_s"] / points["llama"]["decode_tok_s"], 3),
            "like_kernels": gulidra_rooflines(size, batch, context, T, points)}
    print(json.dumps(out), flush=True)
    return 0


# ---- the Lesarax design beside the llama decoder at equal sizes ---------------------------------------------------
LESARAX_LIKE_KERNELS = {
    "apc_rotary_pages_bf16": ["apc_rope_kv_write_bf16", "apc_rope_kv_write"],
    "apc_attention_masked_prefill_bf16": ["apc_attention_prefill_bf16"],
    "apc_attention_masked_decode_bf16": ["apc_attention_decode_bf16"],
    "apc_routed_experts_bf16": ["apc_gemm_swiglu_bf16", "apc_skinny_swiglu_bf16", "apc_skinny_swiglu_pre_bf16"],
    "apc_streams_step": ["apc_rmsnorm_rows"],
    "apc_route_topk": [],
}
LESARAX_EXPERTS, LESARAX_TOP, LESARAX_WINDOW = 8, 2, 1024


def lesarax_configs(size: str, context: int):
    """Two layers that run twice in a row (four layer runs, each with pages of its own): a latent attention (latents of
    3/8 and 1/8 of the width, heads of d unrotated and d/2 rotated key elements, values of d, a window of 1,024) and a
    grouped attention whose values are its keys (heads of d, half of them rotated), each with routed experts (2 of 8,
    each half as wide as the dense feed-forward: the same arithmetic a row); the llama decoder with four layers of the
    same widths."""
    D, H, G, d, F, V = DESIGN_SIZES[size]
    latent = dict(heads=H, dim=d, rot_dim=d // 2, vdim=d, q_rank=3 * D // 8, kv_rank=D // 8, scale=(d + d // 2) ** -0.5,
                  rot=dict(base=10000.0, dims=d // 2), mask=dict(size=LESARAX_WINDOW))
    grouped = dict(heads=H, kv_heads=G, dim=d, vdim=d, scale=d ** -0.5, rot=dict(base=500000.0, dims=d // 2))
    moe = dict(kind="moe", expert=dict(ff=F // LESARAX_TOP, limit=7.0),
               router=dict(experts=LESARAX_EXPERTS, top=LESARAX_TOP))
    lesarax = dict(architecture="Lesarax", vocab=V, width=D, residual_mult=0.5, norm=dict(eps=1e-6),
                   max_positions=2 * context + 4096, loop=dict(start=0, stop=2, times=2),
                   layers=[dict(type="latent_attention", mixer=latent, mlp=moe),
                           dict(type="attention", mixer=grouped, mlp=moe)])
    return {"lesarax": lesarax, "llama": design_configs(size, 4, 2 * context)["llama"]}


def lesarax_rooflines(size, batch, context, T, points):
    """For the kernels the design adds and their like kernels of the llama decoder: the bytes or the arithmetic of the
    launches of a step over the measured time, as a share of the GPU's peak (8 TB/s, 2.5 PFLOP/s)."""
    D, H, G, d, F, V = DESIGN_SIZES[size]
    Fe, E, K, W = F // LESARAX_TOP, LESARAX_EXPERTS, LESARAX_TOP, LESARAX_WINDOW
    dr = d // 2

    def work(name, model, rows, keys_sum, keys_in_window):
        """(bytes, flops) of all of a step's launches of entry point `name` in `model`."""
        if name == "apc_rotary_pages_bf16":      # per run: the projected rows read, q and the pages' rows written
            grouped = (H + G) * d + H * d + 2 * G * d
            latent = H * (d + dr) + 2 * H * d + 2 * dr + H * (d + dr) + H * (2 * d + dr)
            return 2 * rows * (grouped + latent) * 2, 0
        if name in ("apc_rope_kv_write_bf16", "apc_rope_kv_write"):
            return 4 * rows * ((H + 2 * G) * d + H * d + 2 * G * d) * 2, 0
        if name == "apc_attention_masked_prefill_bf16":      # two runs over all earlier keys, two inside the window
            return 0, 2 * keys_sum * H * 4 * d + 2 * keys_in_window * H * (2 * (d + dr) + 2 * d)
        if name == "apc_attention_prefill_bf16":
            return 0, 4 * 4 * keys_sum * H * d
        if name == "apc_attention_masked_decode_bf16":       # keys and values of every kv head; every head has its own
            return (2 * keys_sum * G * 2 * d + 2 * keys_in_window * H * (2 * d + dr)) * 2, 0      # in the latent runs
        if name == "apc_attention_decode_bf16":
            return 4 * keys_sum * G * 2 * d * 2, 0
        if name == "apc_routed_experts_bf16":
            used = min(E, rows * K)
            return 4 * used * 3 * Fe * D * 2, 4 * rows * K * 3 * 2 * Fe * D
        if name in ("apc_gemm_swiglu_bf16", "apc_skinny_swiglu_bf16", "apc_skinny_swiglu_pre_bf16"):
            return 4 * 2 * F * D * 2, 4 * rows * 2 * 2 * F * D
        if name == "apc_streams_step":               # y and x read, x and the next reader's 16-bit copy written
            return 8 * rows * D * (4 + 4 + 4 + 2), 0
        if name == "apc_rmsnorm_rows":
            return 9 * rows * D * (4 + 2), 0
        return None

    table = {}
    in_window = sum(min(p + 1, W) for p in range(T))
    for phase, rows, keys_sum, kw in (("prefill", T, T * (T + 1) // 2, in_window),
                                      ("decode", batch, batch * context, batch * min(context, W))):
        for new, likes in LESARAX_LIKE_KERNELS.items():
            row = {}
            for model, names in (("lesarax", [new]), ("llama", likes)):
                us = sum(points[model][phase + "_kernels_us"].get(n, 0.0) for n in names)
                name = next((n for n in names if n in points[model][phase + "_kernels_us"]), None)
                if not us or name is None:
                    continue
                w = work(name, model, rows, keys_sum, kw)
                row[model] = {"us": round(us, 1)}
                if w:
                    row[model]["share_of_peak"] = round(max(w[0] / (us * 1e-6) / (HBM_PEAK_GBS * 1e9),
                                                            w[1] / (us * 1e-6) / PEAK_FLOPS["bf16"]), 4)
            if row:
                table[f"{phase}: {new}"] = row
    return table


def lesarax_run(args) -> int:
    T, batch, context = 2048, args.batch, args.context
    out = {"metric": "Lesarax beside the llama decoder at equal sizes: prefill tok/s (one prompt of 2048 tokens) and "
                     f"decode tok/s (batch {batch}, context {context})", "unit": "tok/s", "n_gpus": 1,
           "dtype": args.dtype, "data": "synthetic: random N(0, 0.02) weights, uniform random token ids",
           "config": {"layers": "(latent attention + experts, grouped attention + experts) twice in a row",
                      "experts": LESARAX_EXPERTS, "top": LESARAX_TOP, "window": LESARAX_WINDOW, "page_tokens": 16},
           "sizes": {}}
    for size in args.design_sizes.split(","):
        cfgs = lesarax_configs(size, context)
        points = {m: design_point(c, args.dtype, batch, context, args.steps, args.warmup, T) for m, c in cfgs.items()}
        out["sizes"][size] = {
            "shape": dict(zip(("width", "heads", "kv_heads", "head_size", "ff", "vocab"), DESIGN_SIZES[size])),
            **points,
            "prefill_lesarax_over_llama": round(points["lesarax"]["prefill_tok_s"] / points["llama"]["prefill_tok_s"], 3),
            "decode_lesarax_over_llama": round(points["lesarax"]["decode_tok_s"] / points["llama"]["decode_tok_s"], 3),
            "like_kernels": lesarax_rooflines(size, batch, context, T, points)}
    print(json.dumps(out), flush=True)
    return 0


# ---- the Seredra design beside the llama decoder at equal sizes ---------------------------------------------------
SEREDRA_LIKE_KERNELS = {
    "apc_conv_heads_bf16": ["apc_rope_kv_write_bf16", "apc_rope_kv_write"],
    "apc_rotary_pages_bf16": ["apc_rope_kv_write_bf16", "apc_rope_kv_write"],
    "apc_attention_masked_prefill_bf16": ["apc_attention_prefill_bf16"],
    "apc_attention_masked_decode_bf16": ["apc_attention_decode_bf16"],
    "apc_linear_attention_bf16": ["apc_attention_prefill_bf16"],
    "apc_linear_attention": ["apc_attention_decode_bf16"],
    "apc_selective_scan_bf16": ["apc_attention_prefill_bf16"],
    "apc_selective_scan": ["apc_attention_decode_bf16"],
    "apc_conv_channels": ["apc_rope_kv_write_bf16", "apc_rope_kv_write"],
    "apc_routed_experts_bf16": ["apc_gemm_swiglu_bf16", "apc_skinny_swiglu_bf16", "apc_skinny_swiglu_pre_bf16"],
    "apc_act_rows": [],
    "apc_streams_step": ["apc_rmsnorm_rows"],
    "apc_gated_rmsnorm": [],
    "apc_weighted_pair": [],
}
SEREDRA_EXPERTS, SEREDRA_TOP, SEREDRA_STATES, SEREDRA_TAPS = 8, 2, 16, 4


def seredra_configs(size: str, context: int):
    """Four layers: the convolution attention (4 taps, temperature, distance penalty) with the squared-relu
    feed-forward; a retention (heads of d) with routed experts (2 of 8, each half as wide as the dense feed-forward: the
    same arithmetic a row); the side-by-side mixer (grouped attention whose values are its keys, half of a head rotated
    under the frequency rule, soft cap; a selective scan of 2 x width channels with 16 states) with the dense
    feed-forward; an attention that borrows the first one's keys and values, with experts.  The llama decoder with four
    layers of the same widths."""
    D, H, G, d, F, V = DESIGN_SIZES[size]
    att = dict(heads=H, kv_heads=G, dim=d, vdim=d, scale=d ** -0.5, conv=SEREDRA_TAPS, q_temp=dict(coef=0.1, every=256))
    left = dict(heads=H, kv_heads=G, dim=d, vdim=d, scale=d ** -0.5, softcap=50.0,
                rot=dict(base=500000.0, dims=d // 2, scaling=dict(factor=4.0, original=2048, fast=32.0, slow=1.0)))
    right = dict(inner=2 * D, state=SEREDRA_STATES, dt_rank=D // 16, conv=SEREDRA_TAPS)
    ret = dict(heads=H, dim=d, vdim=d, decay=[1.0 - 2.0 ** (-5 - 5 * h / H) for h in range(H)],
               rot=dict(base=10000.0, dims=d))
    moe = dict(kind="moe", expert=dict(ff=F // SEREDRA_TOP), router=dict(experts=SEREDRA_EXPERTS, top=SEREDRA_TOP))
    dense = dict(kind="dense", ff=F)
    seredra = dict(architecture="Seredra", vocab=V, width=D, embedding=dict(scale=1.0), norm=dict(eps=1e-6),
                   max_positions=2 * context + 4096,
                   layers=[dict(type="attention", mixer=att, mlp=dense),
                           dict(type="retention", mixer=ret, mlp=moe),
                           dict(type="parallel", mixer=dict(left=left, right=right, left_scale=0.7, right_scale=0.7),
                                mlp=dense),
                           dict(type="attention", mixer=dict(att, kv_from=0), mlp=moe)])
    return {"seredra": seredra, "llama": design_configs(size, 4, 2 * context)["llama"]}


def seredra_work(size, name, rows, keys_sum, prefill):
    """(bytes, flops) of all launches of entry point `name` in a step of the Seredra model (or, for an entry point of the
    llama decoder, of that one)."""
    D, H, G, d, F, V = DESIGN_SIZES[size]
    Fe, E, K, N, C = F // SEREDRA_TOP, SEREDRA_EXPERTS, SEREDRA_TOP, SEREDRA_STATES, 2 * D
    if name == "apc_conv_heads_bf16":        # an owner (q, k, v) and a borrower (q): rows read, q and pages written
        return 2 * rows * ((H + 2 * G) * d + H * d) * 2 * 2 - 2 * rows * 2 * G * d * 2 * 2 // 2, 0
    if name == "apc_rotary_pages_bf16":      # q and k read, q and the pages' keys and values written
        return rows * ((H + G) * d + H * d + 2 * G * d) * 2, 0
    if name in ("apc_rope_kv_write_bf16", "apc_rope_kv_write"):
        return 4 * rows * ((H + 2 * G) * d + H * d + 2 * G * d) * 2, 0
    if name == "apc_attention_masked_prefill_bf16":      # three attentions over all earlier keys
        return 0, 3 * keys_sum * H * 4 * d
    if name == "apc_attention_prefill_bf16":
        return 0, 4 * 4 * keys_sum * H * d
    if name == "apc_attention_masked_decode_bf16":
        return 3 * keys_sum * G * 2 * d * 2, 0
    if name == "apc_attention_decode_bf16":
        return 4 * keys_sum * G * 2 * d * 2, 0
    if name == "apc_linear_attention_bf16":  # a row: scores and weights over half a chunk of 64, 2 dk dv for the state
        return 0, rows * H * (2 * 32 * 2 * d + 2 * 2 * d * d)
    if name == "apc_linear_attention":       # the state of every row read and written
        return rows * H * d * d * 4 * 2, 0
    if name in ("apc_selective_scan", "apc_selective_scan_bf16"):
        # x, z, the step sizes read, y written; decoded rows: the state both ways
        return rows * C * (2 + 2 + 4 + 2) + (0 if prefill else rows * C * N * 4 * 2), 0
    if name == "apc_conv_channels":
        return rows * C * (2 + 2), 0
    if name == "apc_routed_experts_bf16":
        used = min(E, rows * K)
        return 2 * used * 3 * Fe * D * 2, 2 * rows * K * 3 * 2 * Fe * D
    if name in ("apc_gemm_swiglu_bf16", "apc_skinny_swiglu_bf16", "apc_skinny_swiglu_pre_bf16"):
        return 4 * 2 * F * D * 2, 4 * rows * 2 * 2 * F * D
    if name == "apc_act_rows":               # the float32 sums read, the activations written
        return 2 * rows * F * (4 + 2), 0
    if name == "apc_streams_step":           # y and x read, x and the next reader's 16-bit copy written
        return 9 * rows * D * (4 + 4 + 4 + 2), 0
    if name == "apc_rmsnorm_rows":
        return 9 * rows * D * (4 + 2), 0
    if name == "apc_gated_rmsnorm":
        return rows * H * d * (4 + 2 + 2), 0
    if name == "apc_weighted_pair":
        return rows * D * 12, 0
    return None


def seredra_rooflines(size, batch, context, T, points):
    """For the kernels the design adds and their like kernels of the llama decoder: the bytes or the arithmetic of the
    launches of a step over the measured time, as a share of the GPU's peak (8 TB/s, 2.5 PFLOP/s)."""
    table = {}
    for phase, rows, keys_sum in (("prefill", T, T * (T + 1) // 2), ("decode", batch, batch * context)):
        for new, likes in SEREDRA_LIKE_KERNELS.items():
            row = {}
            for model, names in (("seredra", [new]), ("llama", likes)):
                times = points[model][phase + "_kernels_us"]
                us = sum(times.get(n, 0.0) for n in names)
                name = next((n for n in names if n in times), None)
                if not us or name is None:
                    continue
                w = seredra_work(size, name, rows, keys_sum, phase == "prefill")
                row[model] = {"us": round(us, 1)}
                if w:
                    row[model]["share_of_peak"] = round(max(w[0] / (us * 1e-6) / (HBM_PEAK_GBS * 1e9),
                                                            w[1] / (us * 1e-6) / PEAK_FLOPS["bf16"]), 4)
            if "seredra" in row:
                table[f"{phase}: {new}"] = row
    return table


def seredra_run(args) -> int:
    T, batch, context = 2048, args.batch, args.context
    out = {"metric": "Seredra beside the llama decoder at equal sizes: prefill tok/s (one prompt of 2048 tokens) and "
                     f"decode tok/s (batch {batch}, context {context})", "unit": "tok/s", "n_gpus": 1,
           "dtype": args.dtype, "data": "synthetic: random N(0, 0.02) weights, uniform random token ids",
           "config": {"layers": "convolution attention + dense, retention + experts, (attention | selective scan) + "
                                "dense, borrowing attention + experts",
                      "experts": SEREDRA_EXPERTS, "top": SEREDRA_TOP, "states": SEREDRA_STATES, "taps": SEREDRA_TAPS,
                      "page_tokens": 16},
           "sizes": {}}
    for size in args.design_sizes.split(","):
        cfgs = seredra_configs(size, context)
        points = {m: design_point(c, args.dtype, batch, context, args.steps, args.warmup, T) for m, c in cfgs.items()}
        out["sizes"][size] = {
            "shape": dict(zip(("width", "heads", "kv_heads", "head_size", "ff", "vocab"), DESIGN_SIZES[size])),
            **points,
            "prefill_seredra_over_llama": round(points["seredra"]["prefill_tok_s"] / points["llama"]["prefill_tok_s"], 3),
            "decode_seredra_over_llama": round(points["seredra"]["decode_tok_s"] / points["llama"]["decode_tok_s"], 3),
            "like_kernels": seredra_rooflines(size, batch, context, T, points)}
    print(json.dumps(out), flush=True)
    return 0


# ---- the Muvorax design beside the llama and Seredra decoders at equal sizes ---------------------------------------
# like kernels: of the llama decoder, and of Seredra (which shares the scan, the linear attention and the router)
MUVORAX_LIKE_KERNELS = {
    "apc_latent_attention_bf16": (["apc_attention_prefill_bf16", "apc_attention_decode_bf16"],
                                  ["apc_attention_masked_prefill_bf16", "apc_attention_masked_decode_bf16"]),
    "apc_latent_rows_bf16": (["apc_rope_kv_write_bf16", "apc_rope_kv_write"], ["apc_rotary_pages_bf16"]),
    "apc_heads_gemm_bf16": (["apc_gemm_bf16", "apc_skinny_gemm_bf16"], []),
    "apc_tanh_norm_add": (["apc_rmsnorm_rows"], ["apc_streams_step"]),
    "apc_act_rows": ([], ["apc_act_rows"]),
    "apc_routed_experts_bf16": (["apc_gemm_swiglu_bf16", "apc_gemm_pre_bf16", "apc_skinny_swiglu_pre_bf16"],
                                ["apc_routed_experts_bf16"]),
    "apc_route_topk": ([], ["apc_route_topk"]),
    "apc_linear_attention_bf16": (["apc_attention_prefill_bf16"], ["apc_linear_attention_bf16"]),
    "apc_linear_attention": (["apc_attention_decode_bf16"], ["apc_linear_attention"]),
    "apc_selective_scan_bf16": (["apc_attention_prefill_bf16"], ["apc_selective_scan_bf16"]),
    "apc_selective_scan": (["apc_attention_decode_bf16"], ["apc_selective_scan"]),
    "apc_conv_channels": (["apc_rope_kv_write_bf16"], ["apc_conv_channels"]),
    "apc_gated_rmsnorm": ([], ["apc_gated_rmsnorm"]),
}
MUVORAX_EXPERTS, MUVORAX_TOP, MUVORAX_STATES, MUVORAX_TAPS = 8, 2, 16, 4


def muvorax_configs(size: str, context: int):
    """Four layers: an attention over cached latents (H heads of d unrotated and d/2 rotated elements, a latent of 4 d)
    with the dense feed-forward; a selective scan of 2 x width channels with 16 states and a lightning attention (heads
    of d), both with routed experts (2 of 8 in 4 groups of which 2 are kept, each half as wide as the dense
    feed-forward); an attention on the first layer's latents with the dense feed-forward.  The llama decoder and the
    Seredra decoder (see there) with four layers of the same widths."""
    D, H, G, d, F, V = DESIGN_SIZES[size]
    lat = dict(heads=H, dim=d, rot_dim=d // 2, vdim=d, kv_rank=4 * d, scale=(d + d // 2) ** -0.5,
               rot=dict(base=500000.0, dims=d // 2, scaling=dict(factor=4.0, original=2048, fast=32.0, slow=1.0)))
    scan = dict(inner=2 * D, state=MUVORAX_STATES, dt_rank=D // 16, conv=MUVORAX_TAPS)
    lig = dict(heads=H, dim=d, vdim=d, decay=[1.0 - 2.0 ** (-5 - 5 * h / H) for h in range(H)])
    moe = dict(kind="moe", expert=dict(ff=F // MUVORAX_TOP),
               router=dict(experts=MUVORAX_EXPERTS, top=MUVORAX_TOP, scale=1.5, groups=dict(count=4, keep=2)))
    dense = dict(kind="dense", ff=F)
    muvorax = dict(architecture="Muvorax", vocab=V, width=D, norm=dict(eps=1e-6), max_positions=2 * context + 4096,
                   layers=[dict(type="latent_attention", mixer=lat, mlp=dense), dict(type="mamba1", mixer=scan, mlp=moe),
                           dict(type="lightning", mixer=lig, mlp=moe),
                           dict(type="latent_attention", mixer=dict(lat, kv_from=0), mlp=dense)])
    return {"muvorax": muvorax, **seredra_configs(size, context)}


def muvorax_rooflines(size, batch, context, T, points):
    """For the kernels the design uses beside plain products and their like kernels: the bytes or the arithmetic of the
    launches of a step over the measured time, as a share of the GPU's peak (8 TB/s, 2.5 PFLOP/s)."""
    D, H, G, d, F, V = DESIGN_SIZES[size]
    R, dr = 4 * d, d // 2
    Fe, E, K, N, C = F // MUVORAX_TOP, MUVORAX_EXPERTS, MUVORAX_TOP, MUVORAX_STATES, 2 * D

    def work(model, name, rows, keys_sum, prefill):
        """(bytes, flops) of all of a step's launches of entry point `name`."""
        if name == "apc_latent_attention_bf16":  # two layers; decoded rows: the cached rows of their requests
            return (0, 2 * keys_sum * H * 2 * (2 * R + dr)) if prefill else (2 * keys_sum * (R + dr) * 2,
                                                                            2 * keys_sum * H * 2 * (2 * R + dr))
        if name == "apc_latent_rows_bf16":       # the rotated parts of q in two layers, latents and key part of one
            return rows * (2 * H * dr * 2 + (R + dr) * 2) * 2, 0
        if name == "apc_heads_gemm_bf16":        # queries and outputs of two layers
            return (2 * 2 * H * d * R * 2 + 2 * rows * H * (d + 2 * R + dr + d) * 2, 2 * 2 * rows * H * 2 * d * R)
        if name == "apc_tanh_norm_add":          # x and y read, x and the next reader's 16-bit copy written
            return 8 * rows * D * (4 + 4 + 4 + 2), 0
        if name == "apc_routed_experts_bf16" and model == "muvorax":
            return 2 * min(E, rows * K) * 2 * Fe * D * 2, 2 * rows * K * 2 * 2 * Fe * D
        if name == "apc_gemm_pre_bf16":          # llama: the gate and up products of four layers (and q, k, v of three)
            return 4 * 2 * F * D * 2 + 3 * (H + 2 * G) * d * D * 2, rows * 2 * (4 * 2 * F * D + 3 * (H + 2 * G) * d * D)
        if name == "apc_gemm_bf16" and model == "llama":         # q, k, v of the first layer
            return 0, rows * 2 * (H + 2 * G) * d * D
        if name == "apc_skinny_gemm_bf16" and model == "llama":  # the head
            return V * D * 2, 0
        if name == "apc_gated_rmsnorm":
            return rows * H * d * (4 + 2 + 2), 0
        return seredra_work(size, name, rows, keys_sum, prefill)

    table = {}
    for phase, rows, keys_sum in (("prefill", T, T * (T + 1) // 2), ("decode", batch, batch * context)):
        for new, (llama, seredra) in MUVORAX_LIKE_KERNELS.items():
            row = {}
            for model, names in (("muvorax", [new]), ("llama", llama), ("seredra", seredra)):
                times = points[model][phase + "_kernels_us"]
                name = next((n for n in names if n in times), None)
                if name is None or not times[name]:
                    continue
                us = times[name]
                w = work(model, name, rows, keys_sum, phase == "prefill")
                row[model] = {"us": round(us, 1)}
                if w:
                    row[model]["share_of_peak"] = round(max(w[0] / (us * 1e-6) / (HBM_PEAK_GBS * 1e9),
                                                            w[1] / (us * 1e-6) / PEAK_FLOPS["bf16"]), 4)
            if "muvorax" in row:
                table[f"{phase}: {new}"] = row
    return table


def muvorax_run(args) -> int:
    T, batch, context = 2048, args.batch, args.context
    out = {"metric": "Muvorax beside the llama and Seredra decoders at equal sizes: prefill tok/s (one prompt of 2048 "
                     f"tokens) and decode tok/s (batch {batch}, context {context})", "unit": "tok/s", "n_gpus": 1,
           "dtype": args.dtype, "data": "synthetic: random N(0, 0.02) weights, uniform random token ids",
           "config": {"layers": "latent attention + dense, selective scan + experts, lightning + experts, borrowing "
                                "latent attention + dense",
                      "experts": MUVORAX_EXPERTS, "top": MUVORAX_TOP, "states": MUVORAX_STATES, "taps": MUVORAX_TAPS,
                      "page_tokens": 16},
           "sizes": {}}
    for size in args.design_sizes.split(","):
        cfgs = muvorax_configs(size, context)
        points = {m: design_point(c, args.dtype, batch, context, args.steps, args.warmup, T) for m, c in cfgs.items()}
        out["sizes"][size] = {
            "shape": dict(zip(("width", "heads", "kv_heads", "head_size", "ff", "vocab"), DESIGN_SIZES[size])),
            **points,
            **{f"{phase}_muvorax_over_{m}": round(points["muvorax"][phase + "_tok_s"] / points[m][phase + "_tok_s"], 3)
               for phase in ("prefill", "decode") for m in ("llama", "seredra")},
            "like_kernels": muvorax_rooflines(size, batch, context, T, points)}
    print(json.dumps(out), flush=True)
    return 0


# ---- the Natenex design beside the llama, Muvorax and Seredra decoders at equal sizes ------------------------------
# like kernels: of the llama decoder, of Muvorax (latents, linear attention) and of Seredra (mixers side by side, scan)
NATENEX_LIKE_KERNELS = {
    "apc_attention_masked_prefill_bf16": (["apc_attention_prefill_bf16"], [], ["apc_attention_masked_prefill_bf16"]),
    "apc_attention_masked_decode_bf16": (["apc_attention_decode_bf16"], [], ["apc_attention_masked_decode_bf16"]),
    "apc_rotary_pages_bf16": (["apc_rope_kv_write_bf16", "apc_rope_kv_write"], [], ["apc_rotary_pages_bf16"]),
    "apc_latent_attention_bf16": (["apc_attention_prefill_bf16", "apc_attention_decode_bf16"],
                                  ["apc_latent_attention_bf16"], []),
    "apc_latent_rows_bf16": (["apc_rope_kv_write_bf16", "apc_rope_kv_write"], ["apc_latent_rows_bf16"], []),
    "apc_heads_gemm_bf16": (["apc_gemm_bf16", "apc_skinny_gemm_bf16"], ["apc_heads_gemm_bf16"], []),
    "apc_delta_rule_bf16": (["apc_attention_prefill_bf16"], ["apc_linear_attention_bf16"], []),
    "apc_delta_rule": (["apc_attention_decode_bf16"], ["apc_linear_attention"], []),
    "apc_gated_recurrence_bf16": (["apc_attention_prefill_bf16"], ["apc_selective_scan_bf16"], ["apc_selective_scan_bf16"]),
    "apc_gated_recurrence": (["apc_attention_decode_bf16"], ["apc_selective_scan"], ["apc_selective_scan"]),
    "apc_conv_channels": (["apc_rope_kv_write_bf16"], ["apc_conv_channels"], ["apc_conv_channels"]),
    "apc_gated_rmsnorm": ([], ["apc_gated_rmsnorm"], ["apc_gated_rmsnorm"]),
    "apc_rmsnorm_add": (["apc_rmsnorm_rows"], ["apc_tanh_norm_add"], ["apc_streams_step"]),
}
NATENEX_TAPS, NATENEX_BLOCKS, NATENEX_KEEP = 4, 16, 64


def natenex_configs(size: str, context: int):
    """Four layers: mixers side by side (grouped attention over a window of half the context with 64 kept first tokens,
    half of a head rotated, beside a gated recurrence of the model's width) with the dense feed-forward; an attention
    over cached latents (H heads of d unrotated and d/2 rotated elements, latents of 12 d for the queries and 4 d for
    keys and values, an output gate) with the dense feed-forward; a gated delta rule (H heads over H/2 key heads of d)
    without one; the first layer's weights once more.  The llama, Muvorax and Seredra decoders (see there) with four
    layers of the same widths."""
    D, H, G, d, F, V = DESIGN_SIZES[size]
    left = dict(heads=H, kv_heads=G, dim=d, vdim=d, scale=d ** -0.5, mask=dict(size=context // 2, keep_first=NATENEX_KEEP),
                rot=dict(base=500000.0, dims=d // 2, scaling=dict(factor=4.0, low=1.0, high=4.0, original=2048)))
    right = dict(width=D, blocks=NATENEX_BLOCKS, conv=NATENEX_TAPS)
    par = dict(left=left, right=right, left_scale=0.7, right_scale=0.7)
    lat = dict(heads=H, dim=d, rot_dim=d // 2, vdim=d, q_rank=12 * d, kv_rank=4 * d, scale=(d + d // 2) ** -0.5,
               rot=dict(base=500000.0, dims=d // 2))
    delta = dict(heads=H, kv_heads=H // 2, dim=d, vdim=d, conv=NATENEX_TAPS)
    dense = dict(kind="dense", ff=F)
    natenex = dict(architecture="Natenex", vocab=V, width=D, embedding=dict(scale=1.0), norm=dict(eps=1e-6),
                   max_positions=2 * context + 4096,
                   layers=[dict(type="parallel", mixer=par, mlp=dense), dict(type="latent_attention", mixer=lat, mlp=dense),
                           dict(type="delta", mixer=delta, mlp=None),
                           dict(type="parallel", mixer=par, mlp=dense, weights_of=0)])
    return {"natenex": natenex, **muvorax_configs(size, context)}


def natenex_rooflines(size, batch, context, T, points):
    """For the kernels the design uses beside plain products and their like kernels: the bytes or the arithmetic of the
    launches of a step over the measured time, as a share of the GPU's peak (8 TB/s, 2.5 PFLOP/s)."""
    D, H, G, d, F, V = DESIGN_SIZES[size]
    R, dr, Q, C, w = 4 * d, d // 2, 12 * d, D, D // NATENEX_BLOCKS
    window, keep = context // 2, NATENEX_KEEP

    def work(name, rows, keys_sum, prefill):
        """(bytes, flops) of all of a step's launches of entry point `name` in the Natenex model."""
        seen = (sum(min(t + 1, window + keep) for t in range(rows)) if prefill
                else rows * min(context, window + keep))                 # keys of the windows and the kept first tokens
        if name == "apc_attention_masked_prefill_bf16":
            return 0, 2 * seen * H * 4 * d
        if name == "apc_attention_masked_decode_bf16":
            return 2 * seen * G * 2 * d * 2, 0
        if name == "apc_rotary_pages_bf16":          # q, k, v read, q and the pages' keys and values written
            return 2 * rows * ((H + 2 * G) * d * 2) * 2, 0
        if name == "apc_latent_attention_bf16":
            return (0, keys_sum * H * 2 * (2 * R + dr)) if prefill else (keys_sum * (R + dr) * 2, keys_sum * H * 2 * (2 * R + dr))
        if name == "apc_latent_rows_bf16":
            return rows * (2 * H * dr * 2 + 2 * (R + dr) * 2), 0
        if name == "apc_heads_gemm_bf16":            # the latents' queries and outputs; the gates of two recurrences
            gates = 2 * (2 * C * w * 2 + rows * (C * 2 + 2 * C * 4))
            return 2 * H * d * R * 2 + rows * H * (d + 2 * R + dr + 2 * d) * 2 + gates, 2 * rows * H * 2 * d * R + 2 * rows * 2 * 2 * C * w
        if name == "apc_delta_rule_bf16":            # a row: products with keys, its chunk's systems, the state both ways
            return 0, rows * H * (2 * 2 * 32 * d + 2 * 2 * 32 * d + 3 * 2 * d * d)
        if name == "apc_delta_rule":
            return rows * H * d * d * 4 * 2, 0
        if name in ("apc_gated_recurrence", "apc_gated_recurrence_bf16"):     # u, both gates, y read, the output written
            return 2 * rows * C * (2 + 8 + 2 + 2), 0
        if name == "apc_conv_channels":              # the recurrences' and the delta rule's channels
            return rows * (2 * C + 2 * H * d) * (2 + 2), 0
        if name == "apc_gated_rmsnorm":
            return rows * H * d * (4 + 2 + 2), 0
        if name == "apc_rmsnorm_add":                # y and x read, x and the next reader's 16-bit copy written
            return 7 * rows * D * (4 + 4 + 4 + 2), 0
        return None

    def muvorax_work(name, rows, keys_sum, prefill):
        if name == "apc_latent_attention_bf16":
            return (0, 2 * keys_sum * H * 2 * (2 * R + dr)) if prefill else (2 * keys_sum * (R + dr) * 2, 0)
        if name == "apc_latent_rows_bf16":
            return rows * (2 * H * dr * 2 + (R + dr) * 2) * 2, 0
        if name == "apc_heads_gemm_bf16":
            return 2 * 2 * H * d * R * 2 + 2 * rows * H * (d + 2 * R + dr + d) * 2, 2 * 2 * rows * H * 2 * d * R
        if name == "apc_tanh_norm_add":
            return 8 * rows * D * (4 + 4 + 4 + 2), 0
        return seredra_work(size, name, rows, keys_sum, prefill)

    table = {}
    for phase, rows, keys_sum in (("prefill", T, T * (T + 1) // 2), ("decode", batch, batch * context)):
        for new, (llama, muvorax, seredra) in NATENEX_LIKE_KERNELS.items():
            row = {}
            for model, names in (("natenex", [new]), ("llama", llama), ("muvorax", muvorax), ("seredra", seredra)):
                times = points[model][phase + "_kernels_us"]
                name = next((n for n in names if n in times), None)
                if name is None or not times[name]:
                    continue
                us, pre = times[name], phase == "prefill"
                w_ = (work(name, rows, keys_sum, pre) if model == "natenex" else muvorax_work(name, rows, keys_sum, pre)
                      if model == "muvorax" else seredra_work(size, name, rows, keys_sum, pre))
                row[model] = {"us": round(us, 1)}
                if w_:
                    row[model]["share_of_peak"] = round(max(w_[0] / (us * 1e-6) / (HBM_PEAK_GBS * 1e9),
                                                            w_[1] / (us * 1e-6) / PEAK_FLOPS["bf16"]), 4)
            if "natenex" in row:
                table[f"{phase}: {new}"] = row
    return table


def natenex_run(args) -> int:
    T, batch, context = 2048, args.batch, args.context
    out = {"metric": "Natenex beside the llama, Muvorax and Seredra decoders at equal sizes: prefill tok/s (one prompt of "
                     f"2048 tokens) and decode tok/s (batch {batch}, context {context})", "unit": "tok/s", "n_gpus": 1,
           "dtype": args.dtype, "data": "synthetic: random N(0, 0.02) weights, uniform random token ids",
           "config": {"layers": "(windowed attention | gated recurrence) + dense, latent attention + dense, gated delta "
                                "rule, the first layer's weights again",
                      "window": context // 2, "keep_first": NATENEX_KEEP, "taps": NATENEX_TAPS, "blocks": NATENEX_BLOCKS,
                      "page_tokens": 16},
           "sizes": {}}
    for size in args.design_sizes.split(","):
        cfgs = natenex_configs(size, context)
        points = {m: design_point(c, args.dtype, batch, context, args.steps, args.warmup, T) for m, c in cfgs.items()}
        out["sizes"][size] = {
            "shape": dict(zip(("width", "heads", "kv_heads", "head_size", "ff", "vocab"), DESIGN_SIZES[size])),
            **points,
            **{f"{phase}_natenex_over_{m}": round(points["natenex"][phase + "_tok_s"] / points[m][phase + "_tok_s"], 3)
               for phase in ("prefill", "decode") for m in ("llama", "muvorax", "seredra")},
            "like_kernels": natenex_rooflines(size, batch, context, T, points)}
    print(json.dumps(out), flush=True)
    return 0


def design_point(cfg_json, dtype, batch, context, steps, warmup, T):
    """Prefill tok/s (one prompt of T tokens in one step), decode tok/s (batch x context, graphs) and the time of
    every kernel in an eager prefill step and an eager decode step of one model."""
    import numpy as np
    import torch

    from allpaca_amd.engine.batch import Entry
    from allpaca_amd.kernels import lib as klib
    from allpaca_amd.sampling import GenerationParams
    extra = warmup + steps + decode_during_prefill(batch, context) + 16
    _, eng = build_engine(cfg_json, dtype, batch + 1, context, extra, 0, max_context=context + extra, set_layers=False)
    V = eng.model.spec.vocab_size
    rng = np.random.default_rng(0)
    r = eng.runner

    def prefill_once(tag):
        toks = rng.integers(0, V, size=T).tolist()
        r.admit(tag)
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        r.step([Entry(tag, toks, [T - 1])])
        torch.cuda.synchronize()
        dt = time.perf_counter() - t0
        r.release(tag)
        return dt

    prefill_once("w")
    psec = min(prefill_once(("p", i)) for i in range(3))
    native, r.native = r.native, None          # the timers sit around the entry points as Python calls them
    with klib.timing() as t:
        prefill_once("k")
    prefill_kernels = {k: round(v["us"], 1) for k, v in t.totals().items()}
    r.native = native
    gp = GenerationParams(max_tokens=extra, temperature=0.0)
    for _ in range(batch):
        eng.add_request(rng.integers(0, V, size=context - 1).tolist(), gp)
    while any(not q.decoding for q in eng.scheduler.running) or eng.scheduler.waiting:
        eng.step()
    for _ in range(warmup):
        eng.step()
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    for _ in range(steps):
        eng.step()
    torch.cuda.synchronize()
    dsec = (time.perf_counter() - t0) / steps
    # one eager decode step of as many rows at the same context, under the timers (requests of their own)
    for q in list(eng.scheduler.running):
        eng.abort(q.id)
    eng.step()
    torch.cuda.synchronize()
    ids = [("d", i) for i in range(batch)]
    native, r.native = r.native, None
    graphs, r.use_graphs = r.use_graphs, False
    for i in ids:
        r.admit(i)
        r.step([Entry(i, rng.integers(0, V, size=context).tolist(), [])])
    entries = [Entry(i, [1], [0]) for i in ids]
    r.step(entries)
    with klib.timing() as t:
        r.step(entries)
    decode_kernels = {k: round(v["us"], 1) for k, v in t.totals().items()}
    r.native, r.use_graphs = native, graphs
    out = {"prefill_tok_s": round(T / psec, 1), "prefill_ms": round(psec * 1e3, 3),
           "decode_tok_s": round(batch / dsec, 1), "decode_ms_per_step": round(dsec * 1e3, 4),
           "weight_bytes": weight_bytes(eng), "prefill_kernels_us": prefill_kernels, "decode_kernels_us": decode_kernels}
    del eng, r
    gc.collect()
    torch.cuda.empty_cache()
    return out


def design_rooflines(size, layers, streams, batch, context, T, points):
    """For the kernels the new design adds and their like kernels of the llama decoder: the bytes or the arithmetic
    of the launches of a step, over the measured time, as a share of the GPU's peak (8 TB/s, 2.5 PFLOP/s)."""
    D, H, G, d, F, V = DESIGN_SIZES[size]
    qkv = (H + 2 * G) * d

    def work(name, rows, keys_sum):
        """(bytes, flops) of all of a step's launches of entry point `name`."""
        if name in ("apc_conv_heads_bf16", "apc_rope_kv_write_bf16", "apc_rope_kv_write"):
            return layers * rows * (qkv + H * d + 2 * G * d) * 2, 0       # rows read, q and the pages' rows written
        if name in ("apc_attention_masked_prefill_bf16", "apc_attention_prefill_bf16"):
            return 0, layers * 4 * keys_sum * H * d
        if name in ("apc_attention_masked_decode_bf16", "apc_attention_decode_bf16"):
            return layers * keys_sum * G * 2 * d * 2, 0
        if name == "apc_streams_step":       # per sublayer: the streams read and written, the output read, h written
            return layers * 2 * rows * (2 * streams * D * 4 + D * 4 + D * 2), 0
        return None

    table = {}
    for phase, rows, keys_sum in (("prefill", T, T * (T + 1) // 2), ("decode", batch, batch * context)):
        for new, likes in LIKE_KERNELS.items():
            row = {}
            for model, names in (("risizen", [new]), ("llama", likes)):
                us = sum(points[model][phase + "_kernels_us"].get(n, 0.0) for n in names)
                name = next((n for n in names if n in points[model][phase + "_kernels_us"]), None)
                if not us or name is None:
                    continue
                w = work(name, rows, keys_sum)
                row[model] = {"us": round(us, 1)}
                if w:
                    row[model]["share_of_peak"] = round(max(w[0] / (us * 1e-6) / (HBM_PEAK_GBS * 1e9),
                                                            w[1] / (us * 1e-6) / PEAK_FLOPS["bf16"]), 4)
            if row:
                table[f"{phase}: {new}"] = row
    return table


def design_run(args) -> int:
    layers = args.layers or 4
    T, batch, context = 2048, args.batch, args.context
    out = {"metric": "Risizen beside the llama decoder at equal sizes: prefill tok/s (one prompt of 2048 tokens) and "
                     f"decode tok/s (batch {batch}, context {context})", "unit": "tok/s", "n_gpus": 1,
           "dtype": args.dtype, "data": "synthetic: random N(0, 0.02) weights, uniform random token ids",
           "config": {"layers": layers, "streams": 2, "conv_taps": 4, "chunk": 2 * context, "page_tokens": 16},
           "sizes": {}}
    for size in args.design_sizes.split(","):
        cfgs = design_configs(size, layers, 2 * context)
        points = {m: design_point(c, args.dtype, batch, context, args.steps, args.warmup, T) for m, c in cfgs.items()}
        out["sizes"][size] = {
            "shape": dict(zip(("width", "heads", "kv_heads", "head_size", "ff", "vocab"), DESIGN_SIZES[size])),
            **points,
            "prefill_risizen_over_llama": round(points["risizen"]["prefill_tok_s"] / points["llama"]["prefill_tok_s"], 3),
            "decode_risizen_over_llama": round(points["risizen"]["decode_tok_s"] / points["llama"]["decode_tok_s"], 3),
            "like_kernels": design_rooflines(size, layers, 2, batch, context, T, points)}
    print(json.dumps(out), flush=True)
    return 0


def main() -> int:
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=64)
    ap.add_argument("--warmup", type=int, default=8)
    ap.add_argument("--batch", type=int, default=8)
    ap.add_argument("--context", type=int, default=2048, help="tokens every sequence holds when the decode steps are timed")
    ap.add_argument("--max-context", type=int, default=8192,
                    help="tokens a sequence may grow to: positions, block tables and the page pool are made for it")
    ap.add_argument("--layers", type=int, default=0, help="fewer layers than the configuration (0: all)")
    ap.add_argument("--dtype", default="bf16", choices=["bf16", "fp32"])
    ap.add_argument("--preset", default="llama-3.1-8b")
    ap.add_argument("--no-points", action="store_true", help="skip the batch-1 and batch-64 points and the prefill")
    ap.add_argument("--no-graphs", action="store_true")
    ap.add_argument("--requests", type=int, default=0,
                    help="instead of the decode steps: this many requests with prompts of --min-prompt..--max-prompt "
                         "tokens arrive at once and decode --new-tokens tokens each under chunked prefill")
    ap.add_argument("--min-prompt", type=int, default=128)
    ap.add_argument("--max-prompt", type=int, default=4096)
    ap.add_argument("--new-tokens", type=int, default=256)
    ap.add_argument("--chunk", type=int, default=512, help="largest portion of a prompt in a step (with --requests)")
    ap.add_argument("--sampled", action="store_true",
                    help="tokens drawn with temperature 0.8, top-k 40, top-p 0.95 instead of greedy (the decode steps, or "
                         "with --requests the requests)")
    ap.add_argument("--kernel-times", action="store_true",
                    help="instead of the measured steps: event timers around every kernel of a decode step, a mixed step "
                         "and a 2,048-token prefill (eager passes of their own), and the host's time to launch a mixed step")
    ap.add_argument("--prompt", type=int, default=0,
                    help="with --only prefill: a prompt of this many tokens in steps of --portion tokens instead of the "
                         "2,048-token prompt in one step")
    ap.add_argument("--portion", type=int, default=2048)
    ap.add_argument("--only", choices=["decode", "prefill", "sampler"], default=None,
                    help="for profiling: only the decode steps at --batch (as --no-points), only the 2,048-token "
                         "prefill (prints its figures as the line's value), or only the sampler over the preset's "
                         "vocabulary (microseconds a step's rows take on the GPU and on the host)")
    ap.add_argument("--design", choices=["risizen", "gulidra", "lesarax", "seredra", "muvorax", "natenex"], default=None,
                    help="instead of the default workload: the named design beside the llama decoder at equal sizes "
                         "(--design-sizes), prefill and decode throughput and the times of their like kernels")
    ap.add_argument("--design-sizes", default="1b,8b", help="with --design: sizes of the comparison, of " + ",".join(DESIGN_SIZES))
    args = ap.parse_args()
    if args.gpus != 1:
        print(f"bench.py: this engine runs on one GPU; --gpus {args.gpus} is not supported", flush=True)
        return 2

    import torch

    from allpaca_amd.config import preset
    from allpaca_amd.kernels import lib as klib
    cfg_json = preset(args.preset)
    full_layers = cfg_json["num_hidden_layers"]
    layers = args.layers or full_layers
    klib.load("plain")
    klib.load("tuned")

    if args.design == "gulidra":
        return gulidra_run(args)
    if args.design == "lesarax":
        return lesarax_run(args)
    if args.design == "seredra":
        return seredra_run(args)
    if args.design == "muvorax":
        return muvorax_run(args)
    if args.design == "natenex":
        return natenex_run(args)
    if args.design:
        return design_run(args)
    if args.kernel_times:
        print(json.dumps({"metric": "microseconds per kernel and step (event timers, eager passes)", "unit": "us",
                          "n_gpus": 1, "dtype": args.dtype,
                          "config": {"model": args.preset, "layers": layers, "layers_of_configuration": full_layers,
                                     "global_batch": args.batch, "seq_len": args.context},
                          "kernel_times": kernel_times(cfg_json, args, layers)}), flush=True)
        return 0
    if args.requests:
        n = args.requests
        top = args.max_prompt + args.new_tokens
        cfg, eng = build_engine(cfg_json, args.dtype, n, top, 0, layers, use_graphs=not args.no_graphs,
                                max_context=top, chunk_tokens=args.chunk, pool_tokens=n * (top + 16))
        t0 = time.perf_counter()
        captured = eng.warm_up()                                                                    # decode graphs
        requests_run(eng, cfg, min(n, 4), args.min_prompt, min(args.max_prompt, 512), 8, seed=1)   # first launches
        warm = time.perf_counter() - t0
        r = requests_run(eng, cfg, n, args.min_prompt, args.max_prompt, args.new_tokens, sampled=args.sampled)
        print(json.dumps({
            "metric": f"output tok/s, {n} requests at once, prompts {args.min_prompt}-{args.max_prompt}, "
                      f"{args.new_tokens} new tokens each, chunked prefill"
                      + (", sampled (temperature 0.8, top-k 40, top-p 0.95)" if args.sampled else ""),
            "value": round(r["output_tokens"] / r["seconds"], 1), "unit": "tok/s", "n_gpus": 1,
            "seconds": round(r["seconds"], 3), "steps": r["steps"], "prompt_tokens": r["prompt_tokens"],
            "output_tokens": r["output_tokens"], "all_tokens_per_s": round((r["prompt_tokens"] + r["output_tokens"]) / r["seconds"], 1),
            "mean_ttft_ms": round(r["ttft_ms"], 1), "mean_itl_ms": round(r["itl_ms"], 2),
            "ttft_p50_ms": round(r["ttft_p50_ms"], 1), "ttft_p95_ms": round(r["ttft_p95_ms"], 1),
            "itl_p50_ms": round(r["itl_p50_ms"], 2), "itl_p95_ms": round(r["itl_p95_ms"], 2),
            "ids_hash": r["ids_hash"], "preemptions": r["preemptions"],
            "graphs_captured_before": captured, "warm_up_seconds": round(warm, 2),
            "dtype": args.dtype, "data": "synthetic: random N(0, 0.02) weights, uniform random token ids",
            "config": {"model": args.preset, "layers": layers, "layers_of_configuration": full_layers,
                       "chunk_tokens": args.chunk, "max_batch_tokens": 2048, "page_tokens": 16}}), flush=True)
        return 0
    if args.only == "sampler":
        print(json.dumps({"metric": "microseconds to choose a step's tokens (GPU time, launches queued behind other work)",
                          "unit": "us", "n_gpus": 1, "config": {"model": args.preset, "vocab": cfg_json["vocab_size"]},
                          "sampler": sampler_times(cfg_json["vocab_size"])}), flush=True)
        return 0
    if args.only == "decode":
        args.no_points = True
    if args.only == "prefill" and args.prompt > 0:
        T = args.prompt
        cfg, eng = build_engine(cfg_json, args.dtype, 1, T, 64, layers, use_graphs=not args.no_graphs,
                                max_context=max(args.max_context, T + 64))
        psec, last = long_prefill_run(eng, cfg, T, args.portion)
        fl = prefill_flops(cfg, layers, T)
        print(json.dumps({"metric": f"prefill tok/s, one prompt of {T} tokens in steps of {args.portion}",
                          "value": round(T / psec, 1), "unit": "tok/s", "n_gpus": 1, "seconds": round(psec, 4),
                          "last_step_ms": round(last * 1e3, 3), "dtype": args.dtype,
                          "frac_of_mfma_peak": round(fl / psec / PEAK_FLOPS[args.dtype], 4),
                          "config": {"model": args.preset, "layers": layers, "prompt_tokens": T,
                                     "portion": args.portion}}), flush=True)
        return 0
    if args.only == "prefill":
        T = 2048
        cfg, eng = build_engine(cfg_json, args.dtype, 1, T, 64, layers, use_graphs=not args.no_graphs,
                                max_context=args.max_context)
        psec = prefill_run(eng, cfg, T)
        fl = prefill_flops(cfg, layers, T)
        print(json.dumps({"metric": "prefill tok/s @ 2048 tokens", "value": round(T / psec, 1), "unit": "tok/s",
                          "n_gpus": 1, "ms_per_step": round(psec * 1e3, 3), "dtype": args.dtype,
                          "frac_of_mfma_peak": round(fl / psec / PEAK_FLOPS[args.dtype], 4),
                          "config": {"model": args.preset, "layers": layers}}), flush=True)
        return 0

    # what this card delivers: a streaming read of 8 GiB and a loop of MFMAs from registers (allpaca_amd/csrc/probe.hip)
    from allpaca_amd.kernels import probe
    measured_gbs = probe.read_bandwidth(8.0)
    measured_tflops = probe.mfma_rate() if args.dtype == "bf16" else None
    points = {}
    batches = [args.batch] + ([] if args.no_points else [b for b in (1, 64) if b != args.batch])
    ms = {}
    prefill = None
    roof = None
    for b in batches:
        extra = args.warmup + args.steps + decode_during_prefill(b, args.context) + 16
        cfg, eng = build_engine(cfg_json, args.dtype, max(b, 1), args.context, extra, layers,
                                use_graphs=not args.no_graphs, max_context=args.max_context)
        sec = decode_run(eng, cfg, b, args.context, args.steps, args.warmup, sampled=args.sampled)
        ms[b] = sec * 1e3
        if b == args.batch:
            main_hash = decode_run.ids_hash
            wbytes = weight_bytes(eng)
            ctx_mid = args.context + args.warmup + args.steps // 2
            total = wbytes + b * ctx_mid * kv_bytes_per_token(eng)
            gbs = total / sec / 1e9
            roof = {"bound": "hbm", "achieved": round(gbs, 1), "peak": HBM_PEAK_GBS, "unit": "GB/s",
                    "frac": round(gbs / HBM_PEAK_GBS, 4), "measured_peak": round(measured_gbs, 1),
                    "frac_of_measured": round(gbs / measured_gbs, 4)}
            if not args.no_points:
                T = 2048
                psec = prefill_run(eng, cfg, T)
                fl = prefill_flops(cfg, layers, T)
                prefill = {"value": round(T / psec, 1), "tokens": T, "ms": round(psec * 1e3, 3),
                           "frac": round(fl / psec / PEAK_FLOPS[args.dtype], 4)}
                if measured_tflops:
                    prefill["measured_peak_tflops"] = round(measured_tflops, 1)
        else:
            points[f"decode_b{b}"] = round(b / sec, 1)
        del eng
        gc.collect()                 # an engine holds cycles (graphs, parts): without this the next one is built beside it
        torch.cuda.empty_cache()

    sec = ms[args.batch] / 1e3
    out = {
        "metric": f"decode tok/s @ batch {args.batch}, context {args.context} ({args.preset} shapes)"
                  + (", sampled (temperature 0.8, top-k 40, top-p 0.95)" if args.sampled else ""),
        "value": round(args.batch / sec, 1), "unit": "tok/s", "n_gpus": 1, "steps": args.steps, "warmup": args.warmup,
        "ms_per_step": round(ms[args.batch], 4), "higher_is_better": True, "scaling": "weak", "vs_baseline": None,
        "dtype": args.dtype, "data": "synthetic: random N(0, 0.02) weights, uniform random token ids",
        "config": {
            "model": args.preset, "layers": layers, "layers_of_configuration": full_layers,
            "hidden_size": cfg.hidden_size, "heads": cfg.num_attention_heads, "kv_heads": cfg.num_key_value_heads,
            "head_dim": cfg.head_dim, "intermediate_size": cfg.intermediate_size, "vocab_size": cfg.vocab_size,
            "rope_theta": cfg.rope_theta, "rope_scaling_factor": cfg.rope_scaling.factor if cfg.rope_scaling else 1.0,
            "rms_norm_eps": cfg.rms_norm_eps, "tied_head": cfg.tie_word_embeddings, "global_batch": args.batch,
            "seq_len": args.context, "max_context": max(args.max_context, args.context), "page_tokens": 16,
            "parallelism": "single GPU",
            "graphs": not args.no_graphs,
        },
    }
    out["ids_hash"] = main_hash      # of the tokens the timed steps produced (greedy): the same run, the same hash
    if prefill:
        out["prefill"] = prefill
    if roof:
        out["roofline"] = roof
    if points:
        out["points"] = points
    print(json.dumps(out), flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
