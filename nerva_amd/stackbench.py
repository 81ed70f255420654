"""Prefill and decode throughput of a mixed layer stack (Retorax) beside the uniform decoder at equal sizes.

    python bench.py --stack [all | "4096 wide" | ...] [--prompt N] [--steps K] [--warmup W]

Both models have the same width, heads, feed-forward width, vocabulary and number of layers, random bf16 weights
generated on the device, one sequence. The stack alternates attention (every other one on the keys of the one before
it) and minGRU; the uniform decoder is the Qwen3 shape. One JSON line per size. `model bytes` are what a decode step
has to read: every weight once and the visible keys and values.
"""
import json
import sys
import time

import numpy as np

from . import DecodeSession, stacks
from .runtime import Device

HBM_PEAK = 8e12
SEED = 0x4E45525641

# name: width, heads, kv heads, feed-forward, minGRU width, layers, chunk (16384: longer than the context, so that the
# attention layers of both models see the same keys)
SIZES = {
    "4096 wide": (4096, 32, 8, 12288, 4096, 12, 16384),
    "2048 wide": (2048, 16, 8, 6144, 2048, 12, 16384),
    "4096 wide, chunks of 1536": (4096, 32, 8, 12288, 4096, 12, 1536),
}
VOCAB, HEAD = 151936, 128


def stack_config(width, heads, kv_heads, ff, channels, layers, chunk):
    out = []
    for i in range(layers):
        if i % 2:
            out.append((stacks.MinGru(channels), stacks.XieluFeedForward(ff)))
        else:
            out.append((stacks.Attention(heads, kv_heads, HEAD, HEAD, HEAD, 1e6, HEAD ** -0.5, chunk,
                                         i - 2 if i % 4 == 2 else None), stacks.XieluFeedForward(ff)))
    return stacks.StackConfig(width, VOCAB, 1e-6, out)


def measure(session, prompt, steps, warmup):
    """Seconds of the second prefill, seconds per decoded token."""
    prefill = None
    for _ in range(2):
        t0 = time.perf_counter()
        rc, _ = session.start(prompt)
        assert rc == 0
        rc, _, _ = session.advance(1)
        assert rc == 0
        prefill = time.perf_counter() - t0
    rc, _, _ = session.advance(warmup)
    assert rc == 0
    Device.synchronize()
    t0 = time.perf_counter()
    rc, res, _ = session.advance(steps)
    step = (time.perf_counter() - t0) / steps
    assert rc == 0 and res.observed_tokens == steps and res.hot_path_allocations == 0
    return prefill, step, int(res.graph_nodes)


def run(prompt_tokens, steps, warmup, sizes=None):
    for name in sizes or SIZES:
        width, heads, kv_heads, ff, channels, layers, chunk = SIZES[name]
        prompt = np.random.default_rng(SEED).integers(0, VOCAB, prompt_tokens).astype(np.uint32)
        context = prompt_tokens + warmup + steps + 8
        line = dict(metric="mixed stack beside the uniform decoder", size=name, prompt_tokens=prompt_tokens, steps=steps,
                    dtype="bf16", data="synthetic", layers=layers,
                    config="width %d, %dq/%dkv x %d, ff %d, vocab %d; stack: minGRU width %d in every other layer, chunk %d"
                           % (width, heads, kv_heads, HEAD, ff, VOCAB, channels, chunk))
        config = stack_config(width, heads, kv_heads, ff, channels, layers, chunk)
        uniform = dict(dtype=1, hidden=width, heads=heads, kv_heads=kv_heads, head_dim=HEAD, intermediate=ff, vocab=VOCAB,
                       layers=layers, rms_eps=1e-6, rope_theta=1e6)
        position = prompt_tokens + warmup + steps // 2
        for key, create, visible, readers in (
                ("retorax", lambda: DecodeSession.create_stack_synthetic(config, context), position % chunk + 1, (layers + 1) // 2),
                ("qwen3", lambda: DecodeSession.create_synthetic(uniform, context), position + 1, layers)):
            session = create()
            prefill, step, nodes = measure(session, prompt, steps, warmup)
            moved = session.create_result.resident_weight_bytes + readers * visible * 2 * kv_heads * HEAD * 2
            if key == "qwen3":
                moved -= VOCAB * width * 2   # the embedding table beside the head is not read
            line[key] = dict(prefill_s=round(prefill, 4), prefill_tok_s=round(prompt_tokens / prefill, 1),
                             decode_ms=round(step * 1e3, 4), decode_tok_s=round(1 / step, 1), model_bytes=int(moved),
                             hbm_frac=round(moved / step / HBM_PEAK, 4), graph_nodes=nodes)
            print("[stack] %s %s: prefill %.1f tok/s, decode %.3f ms (%.1f%% of HBM peak)"
                  % (name, key, prompt_tokens / prefill, step * 1e3, 100 * moved / step / HBM_PEAK), file=sys.stderr, flush=True)
            session.destroy()
        print(json.dumps(line), flush=True)
