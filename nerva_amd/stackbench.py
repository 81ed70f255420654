"""Prefill and decode throughput of mixed layer stacks (Retorax, Kavuvik) beside the uniform decoder at equal sizes.

    python bench.py --stack [all | "4096 wide" | "kavuvik 4096 wide" | ...] [--prompt N] [--steps K] [--warmup W]

Both models have the same width, heads, feed-forward width, vocabulary and number of layers, random bf16 weights
generated on the device, one sequence. Retorax alternates attention (every other one on the keys of the one before
it) and minGRU. Kavuvik is latent attention beside routed experts; the experts a token uses and the shared one are
together as wide as the uniform decoder's feed-forward. The uniform decoder is the Qwen3 shape. One JSON line per size.
`model bytes` are what a decode step has to read: every weight it uses once and the visible keys and values.
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
# name: width, heads, kv heads and feed-forward (of the uniform decoder), experts, experts a token, expert width, shared
# width, query rank, latent rank, layers, window
EXPERT_SIZES = {
    "kavuvik 4096 wide": (4096, 32, 8, 12288, 64, 6, 1536, 3072, 1536, 512, 12, 16384),
    "kavuvik 2048 wide": (2048, 16, 8, 6144, 64, 6, 768, 1536, 768, 512, 12, 16384),
    "kavuvik 4096 wide, windows of 1024": (4096, 32, 8, 12288, 64, 6, 1536, 3072, 1536, 512, 12, 1024),
}
VOCAB, HEAD, ROTARY = 151936, 128, 64


def stack_config(width, heads, kv_heads, ff, channels, layers, chunk):
    out = []
    for i in range(layers):
        if i % 2:
            out.append((stacks.MinGru(channels), stacks.XieluFeedForward(ff)))
        else:
            out.append((stacks.Attention(heads, kv_heads, HEAD, HEAD, HEAD, 1e6, HEAD ** -0.5, chunk,
                                         i - 2 if i % 4 == 2 else None), stacks.XieluFeedForward(ff)))
    return stacks.StackConfig(width, VOCAB, 1e-6, out)


def expert_stack_config(width, heads, experts, top, ff, shared, q_rank, kv_rank, layers, window):
    mixer = stacks.LatentAttention(heads, HEAD, ROTARY, HEAD, q_rank, kv_rank, ROTARY, 1e6, (HEAD + ROTARY) ** -0.5, window)
    return stacks.StackConfig(width, VOCAB, 1e-6, [(mixer, stacks.ExpertFeedForward(experts, top, ff, 7.0, shared, 7.0))] * layers,
                              stacks.PARALLEL, 1.0, 1.0)


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
    for name in sizes or list(SIZES) + list(EXPERT_SIZES):
        prompt = np.random.default_rng(SEED).integers(0, VOCAB, prompt_tokens).astype(np.uint32)
        context = prompt_tokens + warmup + steps + 8
        position = prompt_tokens + warmup + steps // 2
        if name in SIZES:
            width, heads, kv_heads, ff, channels, layers, chunk = SIZES[name]
            own, about = "retorax", "minGRU width %d in every other layer, chunk %d" % (channels, chunk)
            config = stack_config(width, heads, kv_heads, ff, channels, layers, chunk)
            cached, unread = (layers + 1) // 2 * (position % chunk + 1) * 2 * kv_heads * HEAD * 2, 0
        else:
            width, heads, kv_heads, ff, experts, top, expert, shared, q_rank, kv_rank, layers, window = EXPERT_SIZES[name]
            own = "kavuvik"
            about = "ranks %d and %d, %d of %d experts of %d, shared %d, window %d" % (q_rank, kv_rank, top, experts, expert, shared, window)
            config = expert_stack_config(width, heads, experts, top, expert, shared, q_rank, kv_rank, layers, window)
            cached = layers * min(position + 1, window) * (kv_rank + ROTARY) * 2
            unread = VOCAB * width * 2 + layers * (experts - top) * 3 * expert * width * 2   # embedding table, other experts
        line = dict(metric="mixed stack beside the uniform decoder", size=name, prompt_tokens=prompt_tokens, steps=steps,
                    dtype="bf16", data="synthetic", layers=layers,
                    config="width %d, %dq/%dkv x %d, ff %d, vocab %d; stack: %s" % (width, heads, kv_heads, HEAD, ff, VOCAB, about))
        uniform = dict(dtype=1, hidden=width, heads=heads, kv_heads=kv_heads, head_dim=HEAD, intermediate=ff, vocab=VOCAB,
                       layers=layers, rms_eps=1e-6, rope_theta=1e6)
        for key, create, keys, idle in (
                (own, lambda: DecodeSession.create_stack_synthetic(config, context), cached, unread),
                ("qwen3", lambda: DecodeSession.create_synthetic(uniform, context), layers * (position + 1) * 2 * kv_heads * HEAD * 2,
                 VOCAB * width * 2)):   # (the embedding table beside the head is not read)
            session = create()
            prefill, step, nodes = measure(session, prompt, steps, warmup)
            moved = session.create_result.resident_weight_bytes + keys - idle
            line[key] = dict(prefill_s=round(prefill, 4), prefill_tok_s=round(prompt_tokens / prefill, 1),
                             decode_ms=round(step * 1e3, 4), decode_tok_s=round(1 / step, 1), model_bytes=int(moved),
                             hbm_frac=round(moved / step / HBM_PEAK, 4), graph_nodes=nodes)
            print("[stack] %s %s: prefill %.1f tok/s, decode %.3f ms (%.1f%% of HBM peak)"
                  % (name, key, prompt_tokens / prefill, step * 1e3, 100 * moved / step / HBM_PEAK), file=sys.stderr, flush=True)
            session.destroy()
        print(json.dumps(line), flush=True)
