"""Prefill and decode throughput of list-of-layers models (Nokuvik, Ludalix) at sizes that resemble a real model's
layers, beside transformers of the same widths on the framework's per-projection path (`bench.py --design NAME`).

Random weights. Decode: greedy steps replayed from a graph, behind a prompt that fills the attention window. Prefill:
a prompt on an empty cache, without the LM head, wall clock around the call. The two sides are measured in turn and
the best of the rounds is kept.
"""
from __future__ import annotations

import time

import numpy as np

from . import synth, synth_model
from .runtime import DTYPE_BF16, Context

HBM_PEAK_GBS = 8000.0
# width -> (window, transformer of the same width on one launch per projection)
SIZES = {"1024": (1024, "qwen3-0.6b"), "2048": (2048, "tinyllama-1.1b")}
PROMPT = 2048
SEED = 0xB10C


def transformer(name: str):
    import dataclasses
    if name == "qwen3-0.6b":
        return dataclasses.replace(synth_model.QWEN3_0P6B, max_position_embeddings=4096, vocab_size=32000), True
    return dataclasses.replace(synth_model.listed_shape(name), max_position_embeddings=4096), False


def kernel_table(model, rounds: int) -> list[dict]:
    out = []
    for r in model.time_kernels(rounds):
        us, nbytes = r["ms"] * 1e3 / r["launches"], r["bytes"] / r["launches"]
        gbs = nbytes / us * 1e-3
        out.append({"kernel": r["label"], "launches_per_step": r["launches"] // rounds, "avg_us": round(us, 2), "bytes_per_launch": int(nbytes),
                    "GBps": round(gbs, 1), "frac": round(gbs / HBM_PEAK_GBS, 4)})
    return out


def measure(ctx: Context, models: dict, prompt: np.ndarray, steps: int, rounds: int) -> dict:
    """models: name -> model. Prefill and decode of each, in turn."""
    res = {n: {"prefill_s": 1e9, "decode_ms": 1e9} for n in models}
    for _ in range(rounds):
        for name, m in models.items():
            m.reset_kv_cache()
            ctx.sync()
            t0 = time.perf_counter()
            m.prefill(prompt, want_logits=False)
            ctx.sync()
            res[name]["prefill_s"] = min(res[name]["prefill_s"], time.perf_counter() - t0)
            m.bench_decode(1, 4)
            ms, _ = m.bench_decode(2, steps)
            res[name]["decode_ms"] = min(res[name]["decode_ms"], ms / steps)
    return res


SHAPES = {"nokuvik": synth_model.nokuvik_shape, "ludalix": synth_model.ludalix_shape}


def run_size(ctx: Context, design: str, name: str, steps: int, rounds: int, kernels: bool = True) -> dict:
    window, other = SIZES[name]
    cfg = SHAPES[design](name)
    block = synth_model.build_block_model(ctx, cfg, SEED, PROMPT + 512)
    tcfg, qk_norm = transformer(other)
    tw = synth_model.synth_weights(tcfg, SEED + 1, DTYPE_BF16, has_qk_norm=qk_norm)
    tr = synth_model.build_model(ctx, tcfg, tw, PROMPT + 512, DTYPE_BF16, has_qk_norm=qk_norm)
    del tw
    if tr.whole_step_available():
        tr.set_whole_step(False)   # the path that other shapes take, too
    models = {design: block, other: tr}
    for m in models.values():
        m.set_graph(True)
    prompt = synth.token_ids(SEED + 2, PROMPT, 32000)
    res = measure(ctx, models, prompt, steps, rounds)
    out = {"width": int(name), "layers": len(cfg["layers"]), "window": window, "prompt_tokens": PROMPT}
    for n, m in models.items():
        r = res[n]
        table = kernel_table(m, 5) if kernels else []
        step_bytes = sum(k["bytes_per_launch"] * k["launches_per_step"] for k in table)
        out[n] = {"prefill_tok_s": round(PROMPT / r["prefill_s"], 1), "prefill_ms": round(r["prefill_s"] * 1e3, 3),
                  "decode_tok_s": round(1e3 / r["decode_ms"], 1), "decode_ms": round(r["decode_ms"], 4), "launches_per_step": m.launches_per_step(),
                  "decode_bytes": step_bytes, "decode_frac_of_hbm": round(step_bytes / (r["decode_ms"] * 1e-3) / 1e9 / HBM_PEAK_GBS, 4), "kernels": table}
    for pieces in (3,):
        block.set_prefill_pieces(pieces)
        best = min(_prefill_time(ctx, block, prompt) for _ in range(rounds))
        out[design][f"prefill_tok_s_bf16x{pieces}"] = round(PROMPT / best, 1)
    for m in models.values():
        m.close()
    return out


def _prefill_time(ctx, m, prompt):
    m.reset_kv_cache()
    ctx.sync()
    t0 = time.perf_counter()
    m.prefill(prompt, want_logits=False)
    ctx.sync()
    return time.perf_counter() - t0


def run_all(ctx: Context, design: str, steps: int = 64, rounds: int = 3) -> dict:
    return {name: run_size(ctx, design, name, steps, rounds) for name in SIZES}
