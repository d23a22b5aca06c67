"""Prefill and decode throughput of a model design beside the closest other family at
equal width, depth and feed-forward (``bench.py --compare``): random-init weights, the
engine's own scheduler, step loop and decode graphs.

    prefill   ``n`` fresh prompts of ``len`` tokens, generated to their first token
    decode    ``batch`` sequences at context ``ctx``: steady pipelined decode steps
"""
from __future__ import annotations

import gc
import random
import time

import torch

PAIRS = {"sivadra": [("sivadra-1b", "llama-1b-shape"), ("sivadra-8b", "llama-3-8b")],
         "sekazen": [("sekazen-3b", "mixtral-3b-shape"), ("sekazen-8x7b", "mixtral-8x7b")],
         "bisuzen": [("bisuzen-3b", "sekazen-3b"), ("bisuzen-8b", "sivadra-8b")],
         "tarunex": [("tarunex-3b", "sekazen-3b"), ("tarunex-8b", "sivadra-8b")]}
PREFILL = [(1, 8192), (8, 2048), (32, 512)]
DECODE = [(1, 2048), (32, 1024), (128, 1024), (256, 512)]


MAX_LEN = 16384


def _engine(model: str, device: str, max_batch: int):
    from ..models.config import resolve
    from .engine import EngineConfig, LLMEngine

    return LLMEngine(EngineConfig(model=model, device=device, max_batch=max_batch,
                                  max_model_len=MAX_LEN, share_prefix=False, kv_fraction=0.5),
                     resolve(model, max_position=MAX_LEN))


def _sync(eng):
    if eng.device.type == "cuda":
        torch.cuda.synchronize()


def _prompts(eng, n, length, rng):
    v = min(250, eng.model_cfg.vocab_size - 1)
    return [[rng.randrange(v) for _ in range(length)] for _ in range(n)]


def prefill_rate(eng, n: int, length: int, reps: int, rng) -> float:
    from .sampling_params import SamplingParams

    p = SamplingParams(temperature=0.0, max_tokens=1, ignore_eos=True)
    best = float("inf")
    for r in range(reps + 1):
        ps = _prompts(eng, n, length, rng)
        _sync(eng)
        t0 = time.perf_counter()
        for x in ps:
            eng.add_request(x, p)
        eng.run_until_done()
        _sync(eng)
        if r:
            best = min(best, time.perf_counter() - t0)
    return n * length / best


def decode_step_ms(eng, batch: int, ctx: int, steps: int, rng) -> float:
    from .sampling_params import SamplingParams

    p = SamplingParams(temperature=0.0, max_tokens=steps + 24, ignore_eos=True)
    seqs = [eng.add_request(x, p) for x in _prompts(eng, batch, ctx, rng)]
    while any(s.n_real < 8 for s in seqs):  # prefill, graph capture, first steps
        eng.step()
    _sync(eng)
    n0, t0 = seqs[0].n_real, time.perf_counter()
    while seqs[0].n_real < n0 + steps:
        eng.step()
    _sync(eng)
    dt = (time.perf_counter() - t0) / (seqs[0].n_real - n0)
    eng.run_until_done()
    return dt * 1e3


def run(design: str, device: str = "cuda", pairs=None, prefill=None, decode=None,
        reps: int = 3, steps: int = 48) -> dict:
    rng = random.Random(7)
    out = {"metric": f"{design} prefill / decode tokens/s beside the closest model",
           "unit": "tokens/s", "data": "random-init weights, random tokens", "rows": []}
    for pair in pairs or PAIRS[design]:
        for model in pair:
            eng = _engine(model, device, max(b for b, _ in decode or DECODE))
            row = {"model": model, "params_b": round(eng.model_cfg.num_params() / 1e9, 2),
                   "prefill_tok_s": {}, "decode_tok_s": {}, "decode_step_ms": {}}
            for n, length in prefill or PREFILL:
                row["prefill_tok_s"][f"{n}x{length}"] = round(
                    prefill_rate(eng, n, length, reps, rng))
            for b, ctx in decode or DECODE:
                ms = decode_step_ms(eng, b, ctx, steps, rng)
                row["decode_step_ms"][f"b{b}@{ctx}"] = round(ms, 3)
                row["decode_tok_s"][f"b{b}@{ctx}"] = round(b / ms * 1e3)
            print(f"[compare] {row}", flush=True)
            out["rows"].append(row)
            eng.shutdown()
            del eng
            gc.collect()
            if device == "cuda":
                torch.cuda.empty_cache()
    return out
