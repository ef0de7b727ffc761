#!/usr/bin/env python3
"""Benchmark of the native-hip sub-2-bit hot path on one MI355X.

    python bench.py [--gpus 1] [--steps K] [--warmup W]

Workload: the Q1_0_g128 GEMV set of a Qwen3-8B layer at
batch 1: fused QKV 6144x4096, gate||up 24576x4096, down 4096x12288.  One step = one
pass over the three GEMVs (one kernel each: it quantises the fp32 activations in its
prologue) with the inputs already resident in HBM; the steps are replayed from a HIP
graph, as the decode path launches them.  Every single matrix fits the 256 MB Infinity Cache, so the
weights rotate through enough distinct resident copies (> 512 MB) that each launch
streams data that is not cached.

Prints ONE JSON line: whole-step throughput in algorithmic GB/s, the roofline of the
dominant kernel (the gate||up GEMV) and the CPU SIMD baseline of the same set.
"""
from __future__ import annotations

import argparse
import ctypes as C
import json
import os
import sys
import time

import numpy as np

ROOT = os.path.dirname(os.path.abspath(__file__))
sys.path.insert(0, ROOT)

HBM_PEAK_GBPS = 8000.0
# HBM bytes one gate||up GEMV launch moves come from the committed counter profile named here: rocprofv3 FETCH_SIZE and
# WRITE_SIZE (KiB per dispatch) of the kernel row named beside it, each times the factor the same file derives from a
# 256 MiB copy.  The algorithmic figure is 14 270 464.
GATE_UP_HBM_TRAFFIC_SOURCE = "profiles/gemv_q1_qwen3_8b_set_hbm_traffic.txt"
GATE_UP_KERNEL_ROW = "gemv_f4_kernel<0, 1, 3, 0>"
GATE_UP_KERNEL = "gemv_f4_kernel<0, 1, 3, 0> (Q1 weights, one activation vector, one superblock of K per wave, three row tiles in flight, fp32 input) gate||up 24576x4096"
SHAPES = [("qkv", 6144, 4096), ("gate_up", 24576, 4096), ("down", 4096, 12288)]
FMT_Q1 = 0
FMT_TQ2 = 1


def traffic_from_profile(path: str, kernel_row: str):
    """HBM bytes per launch of `kernel_row` from a counter summary under profiles/: the per-dispatch averages of its
    FETCH_SIZE and WRITE_SIZE rows (KiB), each scaled by the 'factor' the summary states for that counter.  None when
    the file or a row is missing (the figure is then left out rather than guessed)."""
    import re
    try:
        text = open(os.path.join(ROOT, path)).read()
    except OSError:
        return None
    total = 0.0
    for counter in ("FETCH_SIZE", "WRITE_SIZE"):
        row = re.search(r"^.*%s\(OxbGemvParams\)\s+%s\s+\d+\s+\d+\s+([0-9.]+)" % (re.escape(kernel_row), counter), text, flags=re.M)
        fac = re.search(r"^\s*%s reads .*factor ([0-9.]+)" % counter, text, flags=re.M)
        if not row or not fac:
            return None
        total += float(row.group(1)) * float(fac.group(1)) * 1024.0
    return int(round(total))


def algorithmic_bytes(n_rows: int, k: int, batch: int = 1, block_bytes: int = 18) -> int:
    """weights + input + output bytes, the reference's own effective-bandwidth count
    (crates/oxibonsai-kernels/examples/gemv_benchmark.rs:72-73)."""
    return n_rows * (k // 128) * block_bytes + batch * k * 4 + batch * n_rows * 4


def cpu_baseline(blocks: dict, xs: dict, budget_s: float = 12.0) -> dict:
    """The reference's best x86 tier restated in C++ (oracle/oxb_simd.cpp), all host cores,
    timed on the same three matrices and inputs."""
    from oracle import oracle
    outs = {n: np.zeros(r, dtype=np.float32) for n, r, _ in SHAPES}

    def one_pass():
        for name, n_rows, k in SHAPES:
            oracle.simd_gemv(FMT_Q1, blocks[name], xs[name], n_rows, k, out=outs[name])

    one_pass()
    t0 = time.perf_counter()
    one_pass()
    per = max(time.perf_counter() - t0, 1e-6)
    reps = int(max(5, min(20000, budget_s / per)))
    times = []
    for _ in range(reps):
        t0 = time.perf_counter()
        one_pass()
        times.append(time.perf_counter() - t0)
    med = float(np.median(times))
    total = sum(algorithmic_bytes(r, k) for _, r, k in SHAPES)
    # the reference's scalar tier on one thread: two passes over the same set, the faster one
    oracle.set_threads(1)
    t_scalar = []
    for _ in range(2):
        t0 = time.perf_counter()
        for name, n_rows, k in SHAPES:
            oracle.gemv(FMT_Q1, blocks[name], xs[name], n_rows, k)
        t_scalar.append(time.perf_counter() - t0)
    oracle.set_threads(0)
    return {"value": round(total / med / 1e9, 3), "unit": "GB/s", "cores": oracle.simd_threads(),
            "kind": "port", "tier": oracle.simd_tier(),
            "sample": f"{reps} passes over the same 3-GEMV set (median), {sum(times):.1f} s of CPU time",
            "scalar_tier_1_thread_GBps": round(total / min(t_scalar) / 1e9, 3)}


DECODE_CFG = dict(fmt=FMT_Q1, n_layers=36, h=4096, inter=12288, nq=32, nkv=8, hd=128, vocab=151936,
                  max_seq=32768, eps=1e-6, rope_theta=1e6)   # Qwen3-8B shape, Q1_0_g128


def decode_leg(be, prompt_len: int, n_tokens: int, with_cpu: bool, batches=(8, 32), with_gguf: bool = True,
               long_context: int = 0, long_only: str = "", long_batches=(8,)) -> dict:
    """Greedy batch-1 decode of the random-init 8B-shape Q1 model: one batched prefill of `prompt_len` random
    token ids fills the context (timed on its own), then `n_tokens` greedy steps are timed.  The per-token time
    is what the caller of the fused entry point sees: embedding row H2D, the replayed HIP graph (36 layers,
    final norm, LM head, argmax), token id D2H."""
    from oxibonsai_amd import synth
    from oxibonsai_amd.model import HipModel
    cfg = DECODE_CFG
    w = synth.make_model(cfg, 0xB0A5A104)
    m = HipModel(be, cfg, w, batch=1)
    weight_bytes = sum(len(lw[k]) for lw in w["layers"] for k in ("q", "k", "v", "o", "gate", "up", "down")) + len(w["lm_head"])
    ids = (synth.splitmix64(0xB0A5A1040F, prompt_len) % np.uint64(cfg["vocab"])).astype(np.int64)
    table = {}

    def emb(t):
        if t not in table:
            table[t] = synth.embedding_rows(0xE3B, [t], cfg["h"])[0] * 50.0
        return table[t]

    rows = np.stack([emb(int(t)) for t in ids])
    m.prefill(rows, want_logits=False)      # untimed: allocates the workspaces
    samples = []
    for _ in range(3):      # median of three host-timed calls
        t0 = time.perf_counter()
        _, tok = m.prefill(rows, want_logits=False)
        samples.append(time.perf_counter() - t0)
    t_prefill = sorted(samples)[1]
    layer_macs = sum(r * k for r, k in ((6144, 4096), (4096, 4096), (24576, 4096), (4096, 12288)))
    prefill_flop = 2.0 * prompt_len * cfg["n_layers"] * layer_macs \
        + 4.0 * cfg["n_layers"] * cfg["nq"] * cfg["hd"] * prompt_len * (prompt_len + 1) / 2
    tokens, spent = [], 0.0
    for i in range(n_tokens):
        hidden = emb(tok)
        t0 = time.perf_counter()
        _, out = m.forward(hidden, prompt_len + i, want_logits=False)
        spent += time.perf_counter() - t0
        tok = int(out[0])
        tokens.append(tok)
    res = {"model": "random-init Qwen3-8B shape, Q1_0_g128 (36 layers, h 4096, 32/8 heads, inter 12288, vocab 151936)",
           "batch": 1, "context_before": prompt_len, "prefill_ms": round(t_prefill * 1e3, 2),
           "prefill_tok_per_s": round(prompt_len / t_prefill, 1),
           "prefill_TFLOPs": round(prefill_flop / t_prefill / 1e12, 1),
           "tokens": n_tokens, "tok_per_s": round(n_tokens / spent, 2),
           "ms_per_token": round(spent / n_tokens * 1e3, 4), "hip_graph": m.uses_graph(),
           "weight_bytes_per_token": weight_bytes,
           "kv_bytes_per_token_at_end": 2 * cfg["n_layers"] * cfg["nkv"] * cfg["hd"] * 2 * (prompt_len + n_tokens),
           "weight_stream_GBps": round(weight_bytes / (spent / n_tokens) / 1e9, 1),
           "distinct_tokens": len(set(tokens))}
    # HBM bound of a token: every weight block once, plus the K and V rows of the context (fp16) at the mean position
    # of the timed tokens; norms, activations and the embedding row are below 1 MB and left out
    kv_mean = 2 * cfg["n_layers"] * cfg["nkv"] * cfg["hd"] * 2 * (prompt_len + (n_tokens + 1) // 2)
    bound_us = (weight_bytes + kv_mean) / (HBM_PEAK_GBPS * 1e9) * 1e6
    res["roofline"] = {"bound": "hbm", "bytes_per_token": weight_bytes + kv_mean, "weight_bytes": weight_bytes,
                       "kv_bytes_at_mean_context": kv_mean, "bound_us": round(bound_us, 1), "peak": HBM_PEAK_GBPS, "unit": "GB/s",
                       "achieved": round((weight_bytes + kv_mean) / (spent / n_tokens) / 1e9, 1),
                       "frac": round(bound_us / (spent / n_tokens * 1e6), 4)}
    # the same loop without a host round trip per token: embedding lookup (a Q1_0_g128 table here), forward and
    # argmax stay on the device, the host gets all ids at the end (oxb_hip_decode_tokens)
    from oxibonsai_amd.model import Embedding
    emb_blocks = synth.make_q1_blocks(0xB0A5A104E0, cfg["vocab"] * (cfg["h"] // 128), 0.01, 0.1)
    emb_tab = Embedding(emb_blocks, 41, cfg["vocab"], cfg["h"])
    # the prompt as token ids: the embedding rows are gathered on the device instead of crossing PCIe (33 MB per 2048 tokens)
    m.prefill_tokens(emb_tab, ids, want_logits=False)
    samples = []
    for _ in range(3):
        t0 = time.perf_counter()
        m.prefill_tokens(emb_tab, ids, want_logits=False)
        samples.append(time.perf_counter() - t0)
    t_pft = sorted(samples)[1]
    res["prefill_from_token_ids_ms"] = round(t_pft * 1e3, 2)
    res["prefill_from_token_ids_tok_per_s"] = round(prompt_len / t_pft, 1)
    m.prefill(rows, want_logits=False)      # the cache the decode loops below continue on
    m.generate(emb_tab, [tok], [prompt_len + n_tokens], 2)
    t0 = time.perf_counter()
    ids_dev = m.generate(emb_tab, [tok], [prompt_len + n_tokens], n_tokens)
    t_dev = time.perf_counter() - t0
    t0 = time.perf_counter()
    m.generate_sampled(emb_tab, [tok], [prompt_len + n_tokens], n_tokens, 0.7, 40, 0.9, [0xB0A5A1])   # the reference's defaults
    t_smp = time.perf_counter() - t0
    # the Creative preset: top-k off, softmax / sort / top-p over the whole vocabulary of 151 936 logits
    t0 = time.perf_counter()
    m.generate_sampled(emb_tab, [tok], [prompt_len + 2 * n_tokens], n_tokens, 1.0, 0, 0.95, [0xB0A5A1])
    t_full = time.perf_counter() - t0
    res["device_loop"] = {"tokens": n_tokens, "tok_per_s": round(n_tokens / t_dev, 2),
                          "ms_per_token": round(t_dev / n_tokens * 1e3, 4), "embedding": "Q1_0_g128 table on the device",
                          "sampled_tok_per_s": round(n_tokens / t_smp, 2), "sampling": "temperature 0.7, top-k 40, top-p 0.9",
                          "sampled_filter_off_tok_per_s": round(n_tokens / t_full, 2),
                          "sampling_filter_off": "temperature 1.0, top-k 0 (filter off), top-p 0.95 over the 151936 logits"}
    m.close()
    if with_gguf:
        # checkpoint file -> device: the same tensors written as a GGUF file (page cache), loaded by oxb_hip_load_gguf
        import tempfile
        from oxibonsai_amd.gguf import model_gguf
        with tempfile.TemporaryDirectory() as td:
            path = os.path.join(td, "bonsai8b_shape_q1.gguf")
            with open(path, "wb") as f:
                f.write(model_gguf(cfg, w, 41, emb_blocks))
            size = os.path.getsize(path)
            t0 = time.perf_counter()
            mg, eg, _ = HipModel.from_gguf(be, path, max_seq=prompt_len + 2 * n_tokens + 8)
            t_load = time.perf_counter() - t0
        mg.prefill_tokens(eg, ids, want_logits=False)
        ids_file = mg.generate(eg, [int(ids_dev[0, 0])], [prompt_len], 16)
        mg.close()
        eg.close()
        res["gguf_load"] = {"file_bytes": size, "seconds": round(t_load, 3), "GB_per_s": round(size / t_load / 1e9, 2),
                            "first_tokens": [int(t) for t in ids_file[:4, 0]]}
    emb_tab.close()
    # the same model decoding several sequences at once (weights stream once per step for the whole batch); each
    # sequence gets its own prefilled context of `prompt_len` positions
    res["batched"] = []
    for B in batches:
        cfg_b = dict(cfg, max_seq=prompt_len + 64)
        mb = HipModel(be, cfg_b, w, batch=B)
        for cache, kv_mode in (("fp16", 0), ("int8", 1)) if B == max(batches) else (("fp16", 0),):
            mb.set_attention(kv_mode, 0, 0)
            for sq in range(B):
                mb.prefill(np.roll(rows, sq, axis=0), seq=sq, want_logits=False)
            toks = [int(ids[sq]) for sq in range(B)]
            steps_b, spent = 32, 0.0
            for i in range(steps_b + 2):
                hidden = np.stack([emb(t) for t in toks])
                t0 = time.perf_counter()
                _, out = mb.forward(hidden, np.full(B, prompt_len + i, dtype=np.uint32), want_logits=False)
                if i >= 2:      # the first step records the graph, the second replays it for the first time
                    spent += time.perf_counter() - t0
                toks = [int(t) for t in out]
            res["batched"].append({"batch": B, "context_before": prompt_len, "kv_cache": cache, "steps": steps_b,
                                   "ms_per_step": round(spent / steps_b * 1e3, 4),
                                   "tok_per_s": round(B * steps_b / spent, 1), "hip_graph": mb.uses_graph()})
        mb.close()
    if long_context:
        # one sequence deep into the 32 768-position context: fp16 cache, quantised caches, sliding window
        from oxibonsai_amd.model import KV_F16, KV_FP8_E4M3, KV_I8
        ml = HipModel(be, dict(cfg, max_seq=long_context + 64), w, batch=1)
        reps = -(-long_context // prompt_len)
        res["long_context"] = []
        n_pages16 = -(-(long_context + 64) // 16)
        for name, mode, window, sinks, page, pages in (
                ("fp16 cache", KV_F16, 0, 0, 0, 0), ("int8 cache", KV_I8, 0, 0, 0, 0), ("fp8-e4m3 cache", KV_FP8_E4M3, 0, 0, 0, 0),
                ("fp16 cache, window 4096 + 4 sinks", KV_F16, 4096, 4, 0, 0),
                ("fp16 cache in pages of 16 positions", KV_F16, 0, 0, 16, n_pages16),
                ("int8 cache in pages of 128 positions", KV_I8, 0, 0, 128, -(-(long_context + 64) // 128))):
            if long_only and name != long_only:
                continue
            ml.set_attention(mode, window, sinks, page, pages)
            t0 = time.perf_counter()
            for c in range(reps):       # the prompt rows again and again until the context is full
                n = min(prompt_len, long_context - c * prompt_len)
                ml.prefill(rows[:n], pos_start=c * prompt_len, want_logits=False)
            t_fill = time.perf_counter() - t0
            t, spent, steps_l = int(ids[0]), 0.0, 32
            for i in range(steps_l + 2):
                hidden = emb(t)
                t0 = time.perf_counter()
                _, out = ml.forward(hidden, long_context + i, want_logits=False)
                if i >= 2:
                    spent += time.perf_counter() - t0
                t = int(out[0])
            kv_row = cfg["hd"] * (2 if mode == KV_F16 else 1) + (0 if mode == KV_F16 else 4)
            seen = long_context if not window else min(window, long_context)
            res["long_context"].append({"cache": name, "context_before": long_context, "fill_s": round(t_fill, 2),
                                        "ms_per_token": round(spent / steps_l * 1e3, 4), "tok_per_s": round(steps_l / spent, 1),
                                        "kv_bytes_read_per_token": 2 * cfg["n_layers"] * cfg["nkv"] * kv_row * seen})
        ml.close()
        # several sequences at once, each deep in its own context: the cache reads dominate the step
        res["long_context_batched"] = []
        def deep_batch(B: int) -> dict:
            mlb = HipModel(be, dict(cfg, max_seq=long_context + 64), w, batch=B)
            try:
                t0 = time.perf_counter()
                for sq in range(B):
                    for c in range(reps):
                        n = min(prompt_len, long_context - c * prompt_len)
                        mlb.prefill(rows[:n], pos_start=c * prompt_len, seq=sq, want_logits=False)
                t_fill = time.perf_counter() - t0
                toks, spent, steps_l = [int(ids[sq]) for sq in range(B)], 0.0, 16
                for i in range(steps_l + 2):
                    hidden = np.stack([emb(t) for t in toks])
                    t0 = time.perf_counter()
                    _, out = mlb.forward(hidden, np.full(B, long_context + i, dtype=np.uint32), want_logits=False)
                    if i >= 2:
                        spent += time.perf_counter() - t0
                    toks = [int(t) for t in out]
                kv_bytes = B * 2 * cfg["n_layers"] * cfg["nkv"] * cfg["hd"] * 2 * long_context
                return {"batch": B, "cache": "fp16 cache", "context_before": long_context, "fill_s": round(t_fill, 2),
                        "ms_per_step": round(spent / steps_l * 1e3, 4), "tok_per_s": round(B * steps_l / spent, 1),
                        "kv_bytes_read_per_step": kv_bytes, "kv_read_GBps": round(kv_bytes / (spent / steps_l) / 1e9, 1)}
            finally:
                mlb.close()

        from oxibonsai_amd import GpuError
        for B in (() if long_only else long_batches):
            try:        # 32 sequences hold 151 GB of cache: a GPU that cannot spare them reports that instead of a figure
                res["long_context_batched"].append(deep_batch(B))
            except GpuError as e:
                if e.kind != "OutOfMemory":
                    raise
                res["long_context_batched"].append({"batch": B, "context_before": long_context, "error": str(e)[:200]})
    if with_cpu:
        # CPU SIMD tier on the same matrices: linear layers only (one layer x 36 + LM head), an upper bound on its tok/s
        from oracle import oracle
        lw = w["layers"][0]
        x_h, x_q, x_i = synth.normal_f32(1, cfg["h"]), synth.normal_f32(2, cfg["nq"] * cfg["hd"]), synth.normal_f32(3, cfg["inter"])
        mats = [(np.concatenate([lw["q"], lw["k"], lw["v"]]), x_h, 6144, 4096), (lw["o"], x_q, 4096, 4096),
                (np.concatenate([lw["gate"], lw["up"]]), x_h, 24576, 4096), (lw["down"], x_i, 4096, 12288)]
        def layer():
            for b, x, n, k in mats:
                oracle.simd_gemv(FMT_Q1, b, x, n, k)
        layer()
        t0 = time.perf_counter()
        for _ in range(5):
            layer()
        t_layer = (time.perf_counter() - t0) / 5
        oracle.simd_gemv(FMT_Q1, w["lm_head"], x_h, cfg["vocab"], cfg["h"])
        t0 = time.perf_counter()
        oracle.simd_gemv(FMT_Q1, w["lm_head"], x_h, cfg["vocab"], cfg["h"])
        t_lm = time.perf_counter() - t0
        res["cpu_linear_layers_only_tok_per_s"] = round(1.0 / (36 * t_layer + t_lm), 2)
        res["cpu_cores"] = oracle.simd_threads()
    return res


TERNARY_CFG = dict(fmt=FMT_TQ2, n_layers=28, h=2048, inter=6144, nq=16, nkv=8, hd=128, vocab=151936,
                   max_seq=4096, eps=1e-6, rope_theta=1e6)   # Qwen3-1.7B shape, TQ2_0_g128


def decode_ternary_leg(be, prompt_len: int, n_tokens: int) -> dict:
    """Greedy batch-1 decode of the random-init ternary 1.7B-shape model after a batched prefill, as decode_leg."""
    from oxibonsai_amd import synth
    from oxibonsai_amd.model import HipModel
    cfg = TERNARY_CFG
    w = synth.make_model(cfg, 0xB0A5A103)
    m = HipModel(be, cfg, w, batch=1)
    ids = (synth.splitmix64(0xB0A5A1030F, prompt_len) % np.uint64(cfg["vocab"])).astype(np.int64)
    table = {}

    def emb(t):
        if t not in table:
            table[t] = synth.embedding_rows(0xE3C, [t], cfg["h"])[0] * 50.0
        return table[t]

    rows = np.stack([emb(int(t)) for t in ids])
    m.prefill(rows, want_logits=False)
    samples = []
    for _ in range(3):      # median of three: one call is a few ms of host-timed work
        t0 = time.perf_counter()
        _, tok = m.prefill(rows, want_logits=False)
        samples.append(time.perf_counter() - t0)
    t_prefill = sorted(samples)[1]
    spent = 0.0
    for i in range(n_tokens):
        hidden = emb(tok)
        t0 = time.perf_counter()
        _, out = m.forward(hidden, prompt_len + i, want_logits=False)
        spent += time.perf_counter() - t0
        tok = int(out[0])
    m.close()
    return {"model": "random-init Qwen3-1.7B shape, TQ2_0_g128 (28 layers, h 2048, 16/8 heads, inter 6144, vocab 151936)",
            "batch": 1, "context_before": prompt_len, "prefill_ms": round(t_prefill * 1e3, 2),
            "prefill_tok_per_s": round(prompt_len / t_prefill, 1), "tokens": n_tokens,
            "tok_per_s": round(n_tokens / spent, 2), "ms_per_token": round(spent / n_tokens * 1e3, 4)}


# Fulirax at sizes that resemble a real model's layers, next to the Q1 Qwen3 model of the same width, heads, feed-forward
# width, vocabulary and layer count.
FULIRAX_SHAPES = [dict(width=2048, heads=16, ff=6144), dict(width=4096, heads=32, ff=12288)]
FULIRAX_LATENT = dict(dim=128, rot_dim=64, vdim=128, kv_rank=512)


def fulirax_model(be, shape: dict, layers: int, vocab: int, max_seq: int, batch: int):
    """Random weights: every matrix is a window of one random buffer (bf16 bit patterns), scaled by its fan-in."""
    from oxibonsai_amd.model import HipModel
    w, ff, m = shape["width"], shape["ff"], dict(heads=shape["heads"], **FULIRAX_LATENT)
    base = np.random.default_rng(0xF01).standard_normal(1 << 22, dtype=np.float32)

    def tensor(*dims, std):
        n = int(np.prod(dims))
        return np.resize((base * std).view(np.uint32) >> 16, n).astype(np.uint16).reshape(dims)

    def norm(out, name):
        out[name], out[name + ".b"] = np.full(w, 0x3F80, np.uint16), np.zeros(w, np.uint16)
        out[name + ".alpha"] = np.uint16(0x3F00)

    t = {"embed": tensor(vocab, w, std=1.0), "loop.in": tensor(w, 2 * w, std=(2 * w) ** -0.5), "loop.step": tensor(1, w, std=0.1)}
    kinds = {"q": (m["heads"] * (m["dim"] + m["rot_dim"]), w), "dkv": (m["kv_rank"] + m["rot_dim"], w), "uk": (m["heads"] * m["dim"], m["kv_rank"]),
             "uv": (m["heads"] * m["vdim"], m["kv_rank"]), "o": (w, m["heads"] * m["vdim"]), "up": (ff, w), "down": (w, ff)}
    shared = {k: tensor(*d, std=d[1] ** -0.5) for k, d in kinds.items()}
    for i in range(layers):
        p = f"l{i}."
        norm(t, p + "norm1")
        norm(t, p + "norm2")
        t[p + "mix.dkv.norm"], t[p + "mix.sink"] = np.full(m["kv_rank"], 0x3F80, np.uint16), np.zeros(m["heads"], np.uint16)
        for k in ("q", "dkv", "uk", "uv", "o"):
            t[p + "mix." + k] = shared[k]
        t[p + "mlp.up"], t[p + "mlp.down"] = shared["up"], shared["down"]
    norm(t, "final.norm")
    layer = {"type": "latent_attention", "mlp": {"kind": "dense", "ff": ff},
             "mixer": dict(m, rot={"base": 10000.0, "dims": m["rot_dim"]}, scale=(m["dim"] + m["rot_dim"]) ** -0.5)}
    cfg = {"architecture": "Fulirax", "width": w, "vocab": vocab, "layers": [layer] * layers, "loop": {"start": 0, "stop": 1, "times": 1},
           "norm": {"eps": 1e-6}, "logit_scale": 1.0}
    model, emb = HipModel.from_tensors(be, cfg, t, max_seq=max_seq, batch=batch)
    macs = sum(a * b for a, b in kinds.values())
    return model, emb, macs


MUVONEX_SHAPES = [dict(width=2048, heads=16, kv_heads=8, ff=6144), dict(width=4096, heads=32, kv_heads=8, ff=12288)]


def muvonex_model(be, shape: dict, layers: int, vocab: int, max_seq: int, batch: int):
    """Random weights as above: three gated-delta layers for one of grouped attention beside a state space, heads of 128 (64
    in the state space, twice as many, 128 states)."""
    from oxibonsai_amd.model import HipModel
    w, ff, h, g = shape["width"], shape["ff"], shape["heads"], shape["kv_heads"]
    base = np.random.default_rng(0xF02).standard_normal(1 << 22, dtype=np.float32)

    def tensor(*dims, std):
        n = int(np.prod(dims))
        return np.resize((base * std).view(np.uint32) >> 16, n).astype(np.uint16).reshape(dims)

    def flat(n, value):
        return np.full(n, np.float32(value).view(np.uint32) >> 16, np.uint16)

    delta = {"heads": h, "kv_heads": h, "dim": 128, "vdim": 128, "conv": 4}
    left = {"heads": h, "kv_heads": g, "dim": 128, "vdim": 128, "scale": 128 ** -0.5,
            "rot": {"base": 500000.0, "dims": 128, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}}}
    right = {"heads": 2 * h, "vdim": 64, "state": 128, "groups": 1, "norm_groups": 1, "conv": 4}
    inner, channels = 128 * h, 128 * h + 256
    kinds = {"mlp.gate": (ff, w), "mlp.up": (ff, w), "mlp.down": (w, ff)}
    d_kinds = {"mix." + k: (inner, w) for k in "qkvg"} | {"mix.b": (h, w), "mix.a": (h, w), "mix.o": (w, inner)}
    p_kinds = {"mix.left.q": (inner, w), "mix.left.k": (128 * g, w), "mix.left.v": (128 * g, w), "mix.left.o": (w, inner),
               "mix.right.in": (inner + channels + 2 * h, w), "mix.right.o": (w, inner)}
    shared = {k: tensor(*d, std=d[1] ** -0.5) for k, d in (kinds | d_kinds | p_kinds).items()}
    shared |= {f"mix.{k}.conv": tensor(inner, 4, std=0.5) for k in "qkv"} | {"mix.right.conv": tensor(channels, 4, std=0.5)}
    t = {"embed": tensor(vocab, w, std=1.0), "final.norm": flat(w, 0.0)}
    cfg_layers, macs = [], 0
    for i in range(layers):
        p, parallel = f"l{i}.", i % 4 == 3
        t[p + "norm1"] = flat(w, 0.0)
        names = kinds | (p_kinds if parallel else d_kinds)
        macs += sum(a * b for a, b in names.values())
        for k in names:
            t[p + k] = shared[k]
        if parallel:
            t |= {p + "mix.left.sink": flat(h, 0.0), p + "mix.right.conv": shared["mix.right.conv"], p + "mix.right.conv.b": flat(channels, 0.0),
                  p + "mix.right.dt_bias": flat(2 * h, -2.0), p + "mix.right.A_log": flat(2 * h, -1.0), p + "mix.right.D": flat(2 * h, 1.0),
                  p + "mix.right.norm": flat(inner, 1.0)}
        else:
            t |= {p + f"mix.{k}.conv": shared[f"mix.{k}.conv"] for k in "qkv"}
            t |= {p + "mix.A_log": flat(h, -1.0), p + "mix.dt_bias": flat(h, -2.0), p + "mix.norm": flat(128, 1.0)}
        cfg_layers.append({"type": "parallel", "mixer": {"left": left, "right": right, "left_scale": 0.7, "right_scale": 0.7}} if parallel
                          else {"type": "delta", "mixer": delta})
        cfg_layers[-1]["mlp"] = {"kind": "dense", "ff": ff}
    cfg = {"architecture": "Muvonex", "width": w, "vocab": vocab, "layers": cfg_layers, "norm": {"eps": 1e-6}, "embedding": {"scale": 1.0},
           "residual_mult": 0.5}
    model, emb = HipModel.from_tensors(be, cfg, t, max_seq=max_seq, batch=batch)
    return model, emb, macs


def design_leg(be, name: str, layers: int, vocab: int, prompt: int, steps: int, batches, long_context: int, only: str = "", which: int = -1) -> list:
    """Prefill and decode of a configured design and of the Q1 Qwen3 model of equal size from token ids, the token loops on the device; host-timed around whole calls."""
    from oxibonsai_amd import synth
    from oxibonsai_amd.model import Embedding, HipModel
    ids = (synth.splitmix64(0xF0120F, max(prompt, long_context)) % np.uint64(vocab)).astype(np.int64)
    chunk = 2048

    def fill(m, e, n, seq, first=0):
        t0 = 0.0
        for at in range(first, n, chunk):
            t0 = time.perf_counter()
            m.prefill_tokens(e, ids[at:min(n, at + chunk)], at, seq, want_logits=False)
        return time.perf_counter() - t0

    def measure(build) -> dict:
        r = {}
        m, e = build(prompt + 2 * steps, 1)
        fill(m, e, prompt, 0)
        samples = []
        for _ in range(5):
            t0 = time.perf_counter()
            m.prefill_tokens(e, ids[:prompt], 0, 0, want_logits=False)
            samples.append(time.perf_counter() - t0)
        t = sorted(samples)[2]
        r["prefill_ms"], r["prefill_tok_per_s"] = round(t * 1e3, 3), round(prompt / t, 1)

        def decode(m, e, n, batch):
            m.generate(e, np.arange(batch), np.full(batch, n), 2)
            t0 = time.perf_counter()
            m.generate(e, np.arange(batch), np.full(batch, n + 2), steps)
            return (time.perf_counter() - t0) / steps

        t = decode(m, e, prompt, 1)
        r["decode_batch1"] = {"ms_per_step": round(t * 1e3, 4), "tok_per_s": round(1 / t, 1)}
        m.close()
        for b in batches:
            m2, e2 = build(prompt + 2 * steps, b)
            for q in range(b):
                fill(m2, e2, prompt, q)
            t = decode(m2, e2, prompt, b)
            r[f"decode_batch{b}"] = {"ms_per_step": round(t * 1e3, 4), "tok_per_s": round(b / t, 1)}
            m2.close()
            e2.close()
        if long_context:
            m3, e3 = build(long_context + 2 * steps, 1)
            fill(m3, e3, long_context - chunk, 0)
            tp = fill(m3, e3, long_context, 0, long_context - chunk)
            t = decode(m3, e3, long_context, 1)
            r[f"context_{long_context}"] = {"last_2048_prefill_ms": round(tp * 1e3, 3), "decode_ms_per_step": round(t * 1e3, 4)}
            m3.close()
            e3.close()
        e.close()
        return r

    out = []
    shapes, build = (FULIRAX_SHAPES, fulirax_model) if name == "fulirax" else (MUVONEX_SHAPES, muvonex_model)
    for shape in shapes if which < 0 else shapes[which:which + 1]:
        cfg = dict(fmt=FMT_Q1, n_layers=layers, h=shape["width"], inter=shape["ff"], nq=shape["heads"], nkv=8, hd=128, vocab=vocab,
                   max_seq=0, eps=1e-6, rope_theta=1e6)
        row = {"shape": dict(shape, layers=layers, vocab=vocab)}
        if only != "qwen3":
            n = 1 if name == "fulirax" else layers
            m, e, macs = build(be, shape, n, 64, 64, 1)
            m.close()
            e.close()
            macs *= layers // n
            row[name] = measure(lambda n, b: build(be, shape, layers, vocab, n, b)[:2])
            # products of attention alone beside the matrices (a recurrence's own are not counted)
            per_layer = layers * (192 + 128) if name == "fulirax" else (layers // 4) * 256
            flop = 2.0 * prompt * macs + 2.0 * per_layer * shape["heads"] * prompt * (prompt + 1) / 2
            row[name]["prefill_TFLOPs"] = round(flop / row[name]["prefill_ms"] / 1e9, 1)
            row[name]["weight_bytes_per_token"] = 2 * (macs + vocab * shape["width"] + (2 * shape["width"] ** 2 if name == "fulirax" else 0))
        if only != name:
            weights = synth.make_model(dict(cfg, max_seq=prompt), 0xF012)
            table = synth.make_q1_blocks(0xF0E, vocab * (shape["width"] // 128), 0.01, 0.1)
            row["qwen3_q1"] = measure(lambda n, b: (HipModel(be, dict(cfg, max_seq=n), weights, batch=b), Embedding(table, 41, vocab, shape["width"])))
        out.append(row)
        print(json.dumps(row), file=sys.stderr, flush=True)
    return out


PREFILL_SHAPES = [("qkv", 5120, 2560), ("gate_up", 19456, 2560), ("down", 2560, 9728)]
MFMA_F16_PEAK_TFLOPS = 2500.0


def prefill_gemm_leg(be, L, torch, m_tokens: int = 512) -> dict:
    """TQ2_0_g128 prefill GEMM at Qwen3-4B shapes, M = 512 tokens: the GEMM kernel alone (activations already
    packed to fp16), timed with HIP events on the library's stream; 2 * M * N * K flops per launch."""
    from oxibonsai_amd import _lib, synth
    res = {"workload": f"TQ2_0_g128 prefill GEMM, Qwen3-4B shapes, M = {m_tokens}", "dtype": "fp16 MFMA, fp32 accumulate",
           "peak_TFLOPs": MFMA_F16_PEAK_TFLOPS, "per_kernel": {}}
    total_flop = total_us = 0.0
    for i, (name, n, k) in enumerate(PREFILL_SHAPES):
        a = synth.make_blocks(FMT_TQ2, 0xB0A5A10200 + i, n, k)
        h = be.upload_weights_ternary(a, n, k)
        x = torch.randn(m_tokens, k, device="cuda", dtype=torch.float32)
        y = torch.empty(m_tokens, n, device="cuda", dtype=torch.float32)
        torch.cuda.synchronize()
        us = C.c_float(0.0)
        rc = L.oxb_hip_profile_gemm(int(h), x.data_ptr(), y.data_ptr(), m_tokens, n, k, 5, 50, C.byref(us))
        be.free_weights(h)
        if rc:
            raise RuntimeError(_lib.last_error())
        flop = 2.0 * m_tokens * n * k
        total_flop += flop
        total_us += us.value
        res["per_kernel"][name] = {"us": round(us.value, 2), "TFLOPs": round(flop / us.value * 1e-6, 1),
                                   "frac_of_mfma_peak": round(flop / us.value * 1e-6 / MFMA_F16_PEAK_TFLOPS, 4)}
    res["TFLOPs"] = round(total_flop / total_us * 1e-6, 1)
    res["frac_of_mfma_peak"] = round(total_flop / total_us * 1e-6 / MFMA_F16_PEAK_TFLOPS, 4)
    return res


def measure_launch_context(torch, stream, nbytes: int, copies: int) -> dict:
    """What any launch of this size costs on this GPU, to read roofline.frac against: a kernel that does next to
    nothing, and a device copy that moves the same number of bytes (half read, half written), each replayed from a
    HIP graph of `copies` launches over rotating buffers - the way the GEMV itself is timed."""
    tiny = torch.zeros(64, device="cuda")
    half = nbytes // 8
    src = [torch.ones(half, dtype=torch.float32, device="cuda") for _ in range(copies)]
    dst = [torch.empty(half, dtype=torch.float32, device="cuda") for _ in range(copies)]

    def timed(fn) -> float:
        for i in range(3):
            fn(i)
        torch.cuda.synchronize()
        g = torch.cuda.CUDAGraph()
        with torch.cuda.graph(g, stream=stream):
            for i in range(copies):
                fn(i)
        g.replay()
        torch.cuda.synchronize()
        e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
        e0.record(stream)
        for _ in range(8):
            g.replay()
        e1.record(stream)
        torch.cuda.synchronize()
        return e0.elapsed_time(e1) * 1e3 / (8 * copies)

    empty_us = timed(lambda i: tiny.add_(1.0))
    copy_us = timed(lambda i: dst[i].copy_(src[i]))
    return {"near_empty_kernel_us": round(empty_us, 3), "device_copy_same_bytes_us": round(copy_us, 3),
            "device_copy_GB/s": round(half * 8 / (copy_us * 1e-6) / 1e9, 1),
            "note": "torch elementwise kernels in a replayed HIP graph; the copy moves the GEMV's algorithmic byte count"}


def main() -> int:
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=240)
    ap.add_argument("--warmup", type=int, default=20)
    ap.add_argument("--copies", type=int, default=24, help="distinct resident copies of the weight set")
    ap.add_argument("--no-cpu", action="store_true", help="skip the CPU baseline leg")
    ap.add_argument("--no-decode", action="store_true", help="skip the 8B-shape decode leg")
    ap.add_argument("--no-prefill-gemm", action="store_true", help="skip the prefill GEMM leg")
    ap.add_argument("--no-batch8", action="store_true",
                    help="skip the batch-8 run of the set (counter runs: its launches carry the same kernel names as batch 1)")
    ap.add_argument("--calibrate", action="store_true",
                    help="also run a plain 256 MiB device copy, the known-size kernel that hardware-counter runs are scaled by")
    ap.add_argument("--decode-context", type=int, default=2048)
    ap.add_argument("--decode-tokens", type=int, default=128)
    ap.add_argument("--decode-batches", type=str, default="8,32", help="batch sizes of the batched decode runs ('' = none)")
    ap.add_argument("--no-gguf", action="store_true", help="skip the checkpoint-file load of the decode leg")
    ap.add_argument("--long-context", type=int, default=32000,
                    help="context of the long-context decode runs (fp16 / int8 / fp8 cache, sliding window); 0 = skip")
    ap.add_argument("--long-context-only", type=str, default="", help="run only the long-context option of this name")
    ap.add_argument("--long-context-batches", type=str, default="8,32",
                    help="batch sizes decoded with every sequence at the long context (fp16 cache; 32 sequences hold 151 GB of cache)")
    ap.add_argument("--no-ternary", action="store_true", help="skip the ternary 1.7B-shape decode leg")
    ap.add_argument("--fulirax", action="store_true",
                    help="instead of the default workload: prefill and decode of Fulirax at real layer sizes, next to the Q1 Qwen3 model of equal size")
    ap.add_argument("--muvonex", action="store_true", help="the same for Muvonex")
    ap.add_argument("--design-layers", "--fulirax-layers", type=int, default=8)
    ap.add_argument("--design-shape", "--fulirax-shape", type=int, default=-1, help="one of the shapes alone")
    ap.add_argument("--design-only", "--fulirax-only", choices=["", "design", "fulirax", "muvonex", "qwen3"], default="", help="one of the two models alone (profiling)")
    args = ap.parse_args()
    if args.gpus != 1:
        print("bench.py: this build targets one GPU; run with --gpus 1 (multi-GPU sharding is design-only)",
              file=sys.stderr)
        return 2

    import torch

    import oxibonsai_amd as ox
    from oxibonsai_amd import _lib, synth

    if not torch.cuda.is_available():
        print("bench.py: no GPU visible", file=sys.stderr)
        return 1
    torch.cuda.set_device(0)
    be = ox.NativeHipBackend(0)
    if args.fulirax or args.muvonex:
        design = "fulirax" if args.fulirax else "muvonex"
        rows = design_leg(be, design, args.design_layers, 32768, args.decode_context, args.decode_tokens,
                          tuple(int(b) for b in args.decode_batches.split(",") if b), args.long_context,
                          args.design_only if args.design_only in ("", "qwen3") else design, args.design_shape)
        print(json.dumps({"metric": f"{design.capitalize()} prefill and decode", "n_gpus": 1, "dtype": "bf16", "data": "synthetic, random weights",
                          "prompt": args.decode_context, "steps": args.decode_tokens, "shapes": rows}), flush=True)
        return 0
    L = _lib.lib()
    stream = torch.cuda.Stream()          # a real stream: handle 0 would mean "the library's own"
    torch.cuda.set_stream(stream)
    assert L.oxb_hip_set_stream(C.c_void_p(stream.cuda_stream)) == 0

    # --- synthetic inputs: one seeded set, uploaded `copies` times under distinct handles ----------
    blocks, xs, d_x, d_y, ids = {}, {}, {}, {}, {}
    for i, (name, n_rows, k) in enumerate(SHAPES):
        blocks[name] = synth.make_q1_blocks(0xB0A5A10100 + i, n_rows * (k // 128), 0.01, 0.1)
        xs[name] = synth.normal_f32(0xB0A5A10180 + i, k)
        d_x[name] = torch.from_numpy(xs[name]).cuda()
        d_y[name] = torch.zeros(n_rows, dtype=torch.float32, device="cuda")
        ids[name] = [be.upload_weights_raw(blocks[name], n_rows, k) for _ in range(args.copies)]
    set_bytes = sum(algorithmic_bytes(r, k) for _, r, k in SHAPES)
    resident = sum(len(blocks[n]) for n, _, _ in SHAPES) * args.copies

    def step(i: int) -> None:
        c = i % args.copies
        for name, n_rows, k in SHAPES:
            rc = L.oxb_hip_gemv_dev(ids[name][c], d_x[name].data_ptr(), d_y[name].data_ptr(), n_rows, k, 1)
            if rc:
                raise RuntimeError(_lib.last_error())

    # --- parity spot check before timing ---------------------------------------------------------
    step(0)
    torch.cuda.synchronize()
    from oracle import oracle
    for name, n_rows, k in SHAPES:
        want = oracle.simd_gemv(FMT_Q1, blocks[name], xs[name], n_rows, k)
        got = d_y[name].cpu().numpy()
        err = np.abs(got - want) / np.maximum(np.maximum(np.abs(got), np.abs(want)), 1e-3)
        if not (np.max(np.minimum(err, np.abs(got - want))) < 1e-3):
            print(f"bench.py: parity check failed on {name}", file=sys.stderr)
            return 1

    # --- timed region: exactly K steps, replayed from HIP graphs of `copies` consecutive steps -----
    for i in range(args.warmup):
        step(i)
    torch.cuda.synchronize()

    def capture(n_steps: int):
        g = torch.cuda.CUDAGraph()
        with torch.cuda.graph(g, stream=stream):
            for i in range(n_steps):
                step(i)
        return g

    # The K steps are captured (step i reads weight copy i % copies) - several times over in one graph when K is small,
    # so that a graph holds 240 steps or more and the host's gap between two graph launches weighs the same whatever K
    # is - and the graph is replayed `replays` times so that the timed region lasts a few milliseconds; the figure is the
    # mean over all replayed steps.
    per_graph = max(1, -(-240 // max(args.steps, 1)))
    g_steps = capture(args.steps * per_graph)
    assert L.oxb_hip_set_stream(C.c_void_p(stream.cuda_stream)) == 0
    e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
    g_steps.replay()
    e0.record(stream)
    g_steps.replay()
    e1.record(stream)
    torch.cuda.synchronize()
    replays = int(max(1, min(2000, np.ceil(5.0 / max(e0.elapsed_time(e1), 1e-3)))))
    t0 = time.perf_counter()
    e0.record(stream)
    for _ in range(replays):
        g_steps.replay()
    e1.record(stream)
    torch.cuda.synchronize()
    wall_ms = (time.perf_counter() - t0) * 1e3 / replays
    ms_per_step = max(e0.elapsed_time(e1), 1e-9) / (replays * per_graph * args.steps)
    value = set_bytes / (ms_per_step * 1e-3) / 1e9

    # the same set at batch 8: eight activation vectors, two passes over the weights
    # (four vectors per pass); algorithmic bytes count the weights once
    B8 = 8
    d_x8 = {n: torch.from_numpy(np.stack([synth.normal_f32(0xB0A5A10190 + 16 * i + b, k) for b in range(B8)])).cuda()
            for i, (n, _, k) in enumerate(SHAPES)}
    d_y8 = {n: torch.zeros(B8, r, dtype=torch.float32, device="cuda") for n, r, _ in SHAPES}

    def step8(i: int) -> None:
        c = i % args.copies
        for name, n_rows, k in SHAPES:
            rc = L.oxb_hip_gemv_dev(ids[name][c], d_x8[name].data_ptr(), d_y8[name].data_ptr(), n_rows, k, B8)
            if rc:
                raise RuntimeError(_lib.last_error())

    for i in range(0 if args.no_batch8 else 3):
        step8(i)
    torch.cuda.synchronize()
    g8 = torch.cuda.CUDAGraph()
    if args.no_batch8:
        ms8 = float("nan")
    else:
        with torch.cuda.graph(g8, stream=stream):
            for i in range(args.copies):
                step8(i)
        assert L.oxb_hip_set_stream(C.c_void_p(stream.cuda_stream)) == 0
        g8.replay()
        e0.record(stream)
        for _ in range(8):
            g8.replay()
        e1.record(stream)
        torch.cuda.synchronize()
        ms8 = e0.elapsed_time(e1) / (8 * args.copies)
    set_bytes8 = sum(algorithmic_bytes(r, k, B8) for _, r, k in SHAPES)
    batch8 = {"batch": B8, "ms_per_step": round(ms8, 6), "algorithmic_bytes_per_step": set_bytes8,
              "GB/s": round(set_bytes8 / (ms8 * 1e-3) / 1e9, 1), "frac_of_hbm_peak": round(set_bytes8 / (ms8 * 1e-3) / 1e9 / HBM_PEAK_GBPS, 4),
              "weight_passes_per_gemv": 1, "launches_per_gemv": 2,
              "note": "exact GEMV route: a pack launch quantises the eight vectors once, the GEMV loads its int8 MFMA operands "
                      "and streams the weights once for all eight"}
    if not args.no_batch8:
        # the same step with every workgroup quantising the vectors in its prologue, four vectors per pass over the weights
        L.oxb_hip_set_gemv_packed_min_batch(0)
        for i in range(3):
            step8(i)
        torch.cuda.synchronize()
        g8k = torch.cuda.CUDAGraph()
        with torch.cuda.graph(g8k, stream=stream):
            for i in range(args.copies):
                step8(i)
        L.oxb_hip_set_gemv_packed_min_batch(1)
        assert L.oxb_hip_set_stream(C.c_void_p(stream.cuda_stream)) == 0
        g8k.replay()
        e0.record(stream)
        for _ in range(8):
            g8k.replay()
        e1.record(stream)
        torch.cuda.synchronize()
        ms8k = e0.elapsed_time(e1) / (8 * args.copies)
        batch8["quantised_in_every_workgroup_route"] = {"ms_per_step": round(ms8k, 6), "GB/s": round(set_bytes8 / (ms8k * 1e-3) / 1e9, 1),
                                                        "note": "two passes of four vectors, no pack launch (the route batches of two to four take at K <= 4096)"}
    if not args.no_batch8:
        # the same eight vectors through the route the decode pipeline takes from five sequences on: activations packed
        # to fp16, one pass over the weights on the fp16 matrix cores (prefill tolerance instead of fp32-exact products)
        def step8g(i: int) -> None:
            c = i % args.copies
            for name, n_rows, k in SHAPES:
                rc = L.oxb_hip_gemm_dev(ids[name][c], d_x8[name].data_ptr(), d_y8[name].data_ptr(), B8, n_rows, k)
                if rc:
                    raise RuntimeError(_lib.last_error())

        for i in range(3):
            step8g(i)
        torch.cuda.synchronize()
        g8g = torch.cuda.CUDAGraph()
        with torch.cuda.graph(g8g, stream=stream):
            for i in range(args.copies):
                step8g(i)
        assert L.oxb_hip_set_stream(C.c_void_p(stream.cuda_stream)) == 0
        g8g.replay()
        e0.record(stream)
        for _ in range(8):
            g8g.replay()
        e1.record(stream)
        torch.cuda.synchronize()
        ms8g = e0.elapsed_time(e1) / (8 * args.copies)
        batch8["fp16_matrix_core_route"] = {"ms_per_step": round(ms8g, 6), "GB/s": round(set_bytes8 / (ms8g * 1e-3) / 1e9, 1),
                                            "note": "packer + narrow GEMM per matrix, one pass over the weights, fp16 activations (1e-2 gate)"}

    # --- roofline of the dominant kernel: the gate||up GEMV alone, HIP events on its stream --------
    name, n_rows, k = SHAPES[1]
    idarr = (C.c_uint64 * args.copies)(*[int(h) for h in ids[name]])
    avg_us = C.c_float(0.0)
    rc = L.oxb_hip_profile_gemv(idarr, args.copies, d_x[name].data_ptr(), d_y[name].data_ptr(), n_rows, k,
                                20, max(200, args.steps), C.byref(avg_us))
    if rc:
        raise RuntimeError(_lib.last_error())
    kbytes = algorithmic_bytes(n_rows, k)
    achieved = kbytes / (avg_us.value * 1e-6) / 1e9
    per_kernel = {}
    for nm, r, kk in SHAPES:
        arr = (C.c_uint64 * args.copies)(*[int(h) for h in ids[nm]])
        us = C.c_float(0.0)
        L.oxb_hip_profile_gemv(arr, args.copies, d_x[nm].data_ptr(), d_y[nm].data_ptr(), r, kk, 20, 200, C.byref(us))
        per_kernel[nm] = {"us": round(us.value, 3), "GB/s": round(algorithmic_bytes(r, kk) / (us.value * 1e-6) / 1e9, 1)}
    # what a kernel that only reads the same codes and scales (same grid, waves and load ring) takes: the floor of each launch
    floors = {}
    for nm, r, kk in SHAPES:
        arr = (C.c_uint64 * args.copies)(*[int(h) for h in ids[nm]])
        us = C.c_float(0.0)
        took = []
        for _ in range(3):  # the K = 4096 shapes read 2.8 / 4.2 us in some runs and about 5 us in others: best of three, both ends shown
            if L.oxb_hip_profile_gemv_floor(arr, args.copies, r, kk, 20, 200, C.byref(us)):
                raise RuntimeError(_lib.last_error())
            took.append(us.value)
        floors[nm] = {"us": round(min(took), 3), "us_slowest_of_3": round(max(took), 3),
                      "GB/s": round(len(blocks[nm]) / (min(took) * 1e-6) / 1e9, 1)}
    # the same kernel on a matrix large enough to amortise the launch: the LM head 151936x4096 (3 rotating copies, 262 MB)
    lm_rows, lm_k = 151936, 4096
    lm_blocks = synth.make_q1_blocks(0xB0A5A101F0, lm_rows * (lm_k // 128), 0.01, 0.1)
    lm_ids = [be.upload_weights_raw(lm_blocks, lm_rows, lm_k) for _ in range(3)]
    lm_y = torch.zeros(lm_rows, dtype=torch.float32, device="cuda")
    arr = (C.c_uint64 * 3)(*[int(h) for h in lm_ids])
    us = C.c_float(0.0)
    L.oxb_hip_profile_gemv(arr, 3, d_x["qkv"].data_ptr(), lm_y.data_ptr(), lm_rows, lm_k, 6, 60, C.byref(us))
    per_kernel["lm_head_151936x4096"] = {"us": round(us.value, 3),
                                         "GB/s": round(algorithmic_bytes(lm_rows, lm_k) / (us.value * 1e-6) / 1e9, 1)}
    L.oxb_hip_profile_gemv_floor(arr, 3, lm_rows, lm_k, 6, 60, C.byref(us))
    floors["lm_head_151936x4096"] = {"us": round(us.value, 3), "GB/s": round(len(lm_blocks) / (us.value * 1e-6) / 1e9, 1)}
    for h in lm_ids:
        be.free_weights(h)
    # the same three shapes with ONE resident copy: every launch re-reads what the last one left in the caches
    # (a cache-resident figure, reported apart from the rotating-copies one above)
    cache_resident = {}
    for nm, r, kk in SHAPES:
        arr = (C.c_uint64 * 1)(int(ids[nm][0]))
        L.oxb_hip_profile_gemv(arr, 1, d_x[nm].data_ptr(), d_y[nm].data_ptr(), r, kk, 20, 200, C.byref(us))
        cache_resident[nm] = {"us": round(us.value, 3), "GB/s": round(algorithmic_bytes(r, kk) / (us.value * 1e-6) / 1e9, 1)}
    # TQ2_0_g128 GEMV 12288 x 2048, batch 1, 96 rotating copies (642 MB)
    c0_rows, c0_k, c0_copies = 12288, 2048, 96
    c0_blocks = synth.make_tq2_blocks(0xB0A5A10000, c0_rows * (c0_k // 128))
    c0_ids = [be.upload_weights_ternary(c0_blocks, c0_rows, c0_k) for _ in range(c0_copies)]
    c0_x = torch.from_numpy(synth.normal_f32(0xB0A5A10080, c0_k)).cuda()
    c0_y = torch.zeros(c0_rows, dtype=torch.float32, device="cuda")
    arr = (C.c_uint64 * c0_copies)(*[int(h) for h in c0_ids])
    L.oxb_hip_profile_gemv(arr, c0_copies, c0_x.data_ptr(), c0_y.data_ptr(), c0_rows, c0_k, 20, 400, C.byref(us))
    c0_bytes = algorithmic_bytes(c0_rows, c0_k, 1, 34)
    per_kernel["tq2_12288x2048"] = {"us": round(us.value, 3), "GB/s": round(c0_bytes / (us.value * 1e-6) / 1e9, 1),
                                    "bytes_per_launch": c0_bytes}
    for h in c0_ids:
        be.free_weights(h)
    # the ternary LM head 151936 x 2048 (configs[3]'s last GEMV; 3 rotating copies, 242 MB)
    tl_rows, tl_k = 151936, 2048
    tl_blocks = synth.make_tq2_blocks(0xB0A5A103F0, tl_rows * (tl_k // 128))
    tl_ids = [be.upload_weights_ternary(tl_blocks, tl_rows, tl_k) for _ in range(3)]
    arr = (C.c_uint64 * 3)(*[int(h) for h in tl_ids])
    L.oxb_hip_profile_gemv(arr, 3, c0_x.data_ptr(), lm_y.data_ptr(), tl_rows, tl_k, 6, 60, C.byref(us))
    tl_bytes = algorithmic_bytes(tl_rows, tl_k, 1, 34)
    per_kernel["tq2_lm_head_151936x2048"] = {"us": round(us.value, 3), "GB/s": round(tl_bytes / (us.value * 1e-6) / 1e9, 1),
                                             "bytes_per_launch": tl_bytes}
    for h in tl_ids:
        be.free_weights(h)
    for v in per_kernel.values():
        v["frac"] = round(v["GB/s"] / HBM_PEAK_GBPS, 4)
    slowest = max((nm for nm, _, _ in SHAPES), key=lambda nm: per_kernel[nm]["us"])

    launch_context = measure_launch_context(torch, stream, kbytes, args.copies)
    launch_context["streaming_read_floor"] = floors
    launch_context["streaming_read_floor_note"] = ("a kernel that only reads each matrix's codes and scales with the GEMV's own grid, "
                                                   "waves and load ring (oxb_hip_profile_gemv_floor), rotating copies")

    out = {
        "metric": "quant GEMV HBM GB/s", "value": round(value, 2), "unit": "GB/s",
        "n_gpus": 1, "steps": args.steps, "warmup": args.warmup, "ms_per_step": round(ms_per_step, 6),
        "higher_is_better": True, "scaling": "weak", "vs_baseline": None,
        "dtype": "fp4 (E2M1) MFMA on sixteen base-4 digits of 32-bit fixed-point activations (exact block sums), fp32 scales and accumulation; int8 MFMA on four base-256 digits for two to four vectors",
        "data": "synthetic",
        "config": {"workload": "Q1_0_g128 GEMV set, Qwen3-8B shapes (6144x4096, 24576x4096, 4096x12288), batch 1",
                   "algorithmic_bytes_per_step": set_bytes, "weight_copies": args.copies,
                   "resident_weight_bytes": resident, "pct_of_hbm_peak": round(100 * value / HBM_PEAK_GBPS, 2),
                   "host_wall_ms_per_step": round(wall_ms / (per_graph * args.steps), 6), "timed_replays_of_the_k_steps": replays * per_graph,
                   "steps_per_replayed_graph": per_graph * args.steps,
                   "batch8": batch8},
        "roofline": {"bound": "hbm", "achieved": round(achieved, 1), "peak": HBM_PEAK_GBPS, "unit": "GB/s",
                     "frac": round(achieved / HBM_PEAK_GBPS, 4), "traffic": traffic_from_profile(GATE_UP_HBM_TRAFFIC_SOURCE, GATE_UP_KERNEL_ROW),
                     "traffic_source": GATE_UP_HBM_TRAFFIC_SOURCE, "kernel": GATE_UP_KERNEL, "bytes_per_launch": kbytes,
                     "avg_launch_us": round(avg_us.value, 3), "launch_context": launch_context, "per_kernel": per_kernel,
                     "slowest_kernel_of_the_step": {"name": slowest, **per_kernel[slowest]},
                     "per_kernel_cache_resident": cache_resident},
    }
    if not args.no_cpu:
        out["cpu_baseline"] = cpu_baseline(blocks, xs)
    for name, _, _ in SHAPES:
        for h in ids[name]:
            be.free_weights(h)
    L.oxb_hip_set_stream(None)
    torch.cuda.synchronize()
    if args.calibrate:
        src = torch.ones(64 * 2**20, dtype=torch.float32, device="cuda")
        dst = torch.empty_like(src)
        for _ in range(3):
            dst.copy_(src)
        torch.cuda.synchronize()
    if not args.no_prefill_gemm:
        out["prefill_gemm"] = prefill_gemm_leg(be, L, torch)
    if not args.no_decode:
        out["decode"] = decode_leg(be, args.decode_context, args.decode_tokens, not args.no_cpu,
                                   tuple(int(b) for b in args.decode_batches.split(",") if b), not args.no_gguf,
                                   args.long_context, args.long_context_only,
                                   tuple(int(b) for b in args.long_context_batches.split(",") if b))
        if not args.no_ternary:
            out["decode_ternary_1p7b"] = decode_ternary_leg(be, args.decode_context, args.decode_tokens)
    print(json.dumps(out), flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
