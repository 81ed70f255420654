"""Sessions over parallel layers of latent attention and routed experts (Kavuvik) on the GPU against the plain statement of
oracle/mixed_stack.py: every mechanism alone, whole prompts, portions, decoding, window edges, reused and forked sessions,
sizes that take the wide kernels, generation."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import stack_models as M
from oracle import mixed_stack as O

pytestmark = pytest.mark.gpu

EXACT, HALF = 3e-5, 0.05        # 32-bit and 16-bit sessions, relative to the logits' spread
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
EVERYTHING = [M.latent(), M.latent(heads=1, dim=5, rot_dim=4, vdim=9, q_rank=7, kv_rank=33, window=1, experts=0),
              M.latent(heads=5, dim=16, rot_dim=8, rot=4, vdim=8, q_rank=24, kv_rank=24, window=30, experts=9, top=4, ff=13, shared=0),
              M.latent(heads=2, rot_dim=2, window=17, base=5.0, experts=3, top=1, ff=40, limit=0.3, shared=33, shared_limit=0.4)]
PRECISIONS = pytest.mark.parametrize("precision", [1, 0], ids=["f32", "bf16"])


def tokens_of(cfg, n, seed=1):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).astype(np.uint32)


def weights(cfg, seed, precision):
    """16-bit sessions route by features that rounding cannot turn, 32-bit ones by anything."""
    tensors = M.weights(cfg, seed=seed)
    return tensors if precision else M.clear_routes(cfg, tensors, seed)


def check(cfg, tensors, tokens, sizes, precision, max_context=None):
    s = M.session(cfg, tensors, max_context or len(tokens), precision)
    got = M.feed(s, tokens, sizes)
    want, _ = M.oracle_model(cfg, tensors).run(tokens)
    s.destroy()
    worst = M.errors(got, want)
    assert worst.max() < (EXACT if precision else HALF), "position %d: %.2e" % (int(worst.argmax()), worst.max())


ALONE = {
    "attention": [M.latent(experts=0)],
    "one head": [M.latent(heads=1, experts=0)],
    "no rotation": [M.latent(rot=0, experts=0)],
    "partial rotation": [M.latent(rot_dim=10, rot=4, experts=0)],
    "window of one": [M.latent(window=1, experts=0)],
    "window of two": [M.latent(window=2, experts=0)],
    "window of a block": [M.latent(window=16, experts=0)],
    "window not reached": [M.latent(window=1000, experts=0)],
    "negative scale": [M.latent(scale=-0.6, experts=0)],
    "wide ranks": [M.latent(heads=2, q_rank=300, kv_rank=520, experts=0)],
    "narrow ranks": [M.latent(q_rank=1, kv_rank=3, rot_dim=2, dim=1, vdim=1, experts=0)],
    "experts": [M.latent(heads=1, dim=2, rot_dim=2, vdim=1)],
    "one expert": [M.latent(experts=1, top=1)],
    "one of many": [M.latent(experts=70, top=1, ff=5)],
    "all of them": [M.latent(experts=4, top=4)],
    "no shared expert": [M.latent(shared=0)],
    "tight limits": [M.latent(limit=0.05, shared_limit=0.0)],
    "wide limits": [M.latent(limit=50.0, shared_limit=50.0)],
    "everything": EVERYTHING,
}


@PRECISIONS
@pytest.mark.parametrize("name", ALONE)
def test_mechanism(name, precision):
    cfg = M.parallel_config(ALONE[name])
    check(cfg, weights(cfg, 3, precision), tokens_of(cfg, 45), [45], precision)


@PRECISIONS
def test_residual_rows_after_every_layer(precision):
    cfg = M.parallel_config(EVERYTHING)
    tensors, tokens = weights(cfg, 4, precision), tokens_of(cfg, 30)
    s = M.session(cfg, tensors, 64, precision)
    rc, _, logits, rows = s.extend(tokens, [29], residual_layers=len(EVERYTHING))
    assert rc == 0
    want, trail = M.oracle_model(cfg, tensors).run(tokens)
    spread = np.sqrt((trail ** 2).mean())
    for l in range(len(EVERYTHING)):
        assert np.sqrt(((rows[l] - trail[l]) ** 2).mean()) / spread < (1e-5 if precision else 0.02), l
    assert M.errors(logits, want[29:]).max() < (EXACT if precision else HALF)
    rc, _, after, _ = s.extend(tokens[:1], [0])   # reading the rows back changes nothing that comes after
    want, _ = M.oracle_model(cfg, tensors).run(np.append(tokens, tokens[0]))
    assert rc == 0 and M.errors(after, want[30:]).max() < (EXACT if precision else HALF)
    s.destroy()


@PRECISIONS
@pytest.mark.parametrize("sizes", [[1], [2], [3, 1, 7, 2], [16], [40, 1, 1, 1], [17, 13, 29], [1, 60]], ids=str)
def test_portions(sizes, precision):
    cfg = M.parallel_config(EVERYTHING)
    check(cfg, weights(cfg, 5, precision), tokens_of(cfg, 80, seed=2), sizes, precision)


@pytest.mark.parametrize("change", [dict(eps=1e-12), dict(eps=0.3), dict(embedding_scale=1.0), dict(embedding_scale=-20.0),
                                    dict(logit_scale=1.0), dict(logit_scale=-4.0), dict(vocab=1), dict(width=1, eps=0.5), dict(width=130)], ids=str)
def test_constants_of_the_model(change):
    cfg = M.parallel_config([M.latent(), M.latent(experts=0, window=5)], **change)
    tensors, tokens = M.weights(cfg, seed=6), tokens_of(cfg, 20)
    if cfg["vocab"] == 1:   # one logit: its value, not its place among others
        s = M.session(cfg, tensors, 20, 1)
        assert np.abs(M.feed(s, tokens, [20]) - M.oracle_model(cfg, tensors).run(tokens)[0]).max() < 1e-3
        s.destroy()
        return
    got = M.session(cfg, tensors, 20, 1)
    logits = M.feed(got, tokens, [7, 1, 12])
    want, _ = M.oracle_model(cfg, tensors).run(tokens)
    assert M.errors(logits, want).max() < EXACT
    assert np.abs(logits - want).max() < 1e-3 * np.abs(want).max()   # the scale itself, which the relative measure cannot see
    got.destroy()


@pytest.mark.parametrize("width", [16, 50, 136, 520, 1024, 1030, 4100])
def test_model_widths(width):
    cfg = M.parallel_config([M.latent(), M.latent(experts=3, top=3, shared=0, ff=9)], width=width, vocab=33)
    tokens = tokens_of(cfg, 21)
    for precision in (1, 0):
        check(cfg, weights(cfg, 7, precision), tokens, [11, 1, 9], precision)


def needle_model(window, heads, dim, rot_dim, vdim, kv_rank, layers=1, width=64, vocab=40):
    """Token 1 asks, token 0 answers: where token 0 is visible its key outscores everything, and its value is large."""
    cfg = M.parallel_config([M.latent(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, q_rank=32, kv_rank=kv_rank, window=window, experts=0)
                             for _ in range(layers)], width=width, vocab=vocab)
    tensors = M.weights(cfg, seed=8)
    rng = np.random.default_rng(9)
    embed = M.value(tensors["embed"]) * 0.3
    embed[:, :2] = 0.0
    embed[1, 0] = embed[0, 1] = 6.0
    tensors["embed"] = M.bf16(embed)
    for l in range(layers):
        name = "l%d." % l
        tensors[name + "norm1"] = M.bf16(np.ones(width))
        dq = rng.normal(0, 0.02, (32, width))
        dq[0, 0] += 3.0                                # the query latent's first element: this token asks
        uq = rng.normal(0, 0.05, (heads, dim + rot_dim, 32))
        uq[:, 0, 0] += 2.0
        dkv = rng.normal(0, 0.05, (kv_rank + rot_dim, width))
        dkv[0, 1] += 3.0                               # the latent's first element: this token answers
        uk = rng.normal(0, 0.05, (heads, dim, kv_rank))
        uk[:, 0, 0] += 1.5
        uv = rng.normal(0, 0.3, (heads * vdim, kv_rank))
        uv[:, 0] *= 8.0
        for key, a in (("dq", dq), ("dq.norm", np.ones(32)), ("uq", uq.reshape(-1, 32)), ("dkv", dkv), ("dkv.norm", np.ones(kv_rank)),
                       ("uk", uk.reshape(-1, kv_rank)), ("uv", uv)):
            tensors[name + "mix." + key] = M.bf16(a)
    return cfg, tensors


@pytest.mark.parametrize("shape", [(4, 16, 8, 16, 24), (4, 32, 64, 16, 128), (40, 32, 64, 16, 128), (16, 64, 64, 32, 256)],
                         ids=["general", "rank 128", "rank 128, 40 heads", "rank 256"])
@pytest.mark.parametrize("window", [1, 16, 37, 48])
def test_one_key_at_a_windows_edge(window, shape):
    """A key that decides the answer, just inside and just outside the window, near and far, asked for from a prompt and from a
    decoded token; and the plain statement itself must tell the cases apart."""
    cfg, tensors = needle_model(window, *shape)
    oracle = M.oracle_model(cfg, tensors)
    s = M.session(cfg, tensors, 4 * window + 40)
    fill = np.random.default_rng(3).integers(2, cfg["vocab"], 4 * window + 40)
    for ask, back in ((window + 20, window - 1), (window + 20, window), (window + 20, window + 1), (3 * window + 7, window - 1),
                      (3 * window + 7, window), (15, 15), (16, 16), (17, 1), (window, window), (window - 1, window - 1), (32, 2)):
        needle = ask - back
        if back <= 0 or needle < 0:
            continue
        tokens = fill[:ask + 1].copy()
        tokens[needle], tokens[ask] = 0, 1
        oracle.reset()
        want = oracle.run(tokens)[0][-1:]
        tokens[needle] = fill[needle]
        oracle.reset()
        without = oracle.run(tokens)[0][-1:]
        tokens[needle] = 0
        told = M.errors(without, want).max()
        assert told > 0.12 if back < window else told < 1e-9, (told, ask, back)
        for sizes in ([ask + 1], [ask, 1], [max(1, ask - 2), 3]):
            s.release_sequence()
            got = M.feed(s, tokens.astype(np.uint32), sizes)[-1:]
            assert M.errors(got, want).max() < 0.03, (needle, ask, sizes)
    s.destroy()


def test_the_block_ring_wraps():
    """Contexts far longer than a layer's ring of cache blocks, prompts and decoding."""
    cfg = M.parallel_config([M.latent(heads=2, dim=6, rot_dim=4, vdim=4, q_rank=8, kv_rank=8, window=24, experts=0),
                             M.latent(heads=1, dim=6, rot_dim=4, vdim=4, q_rank=8, kv_rank=16, window=90, experts=2, top=1, ff=6, shared=0)],
                            width=24, vocab=31)
    tensors, tokens = M.weights(cfg, seed=11), tokens_of(cfg, 6000)
    s = M.session(cfg, tensors, 6100, 1)
    assert s.create_result.resident_kv_bytes < 6100 * (12 + 20) * 4 / 1.8
    want, _ = M.oracle_model(cfg, tensors).run(tokens)
    for sizes in ([6000], [700, 511, 513, 2, 512, 2048, 40, 1, 1, 1700, 400]):
        s.release_sequence()
        assert M.errors(M.feed(s, tokens, sizes), want).max() < EXACT
    s.destroy()


def test_sessions_are_reused_and_forked():
    """Sequences of unequal length on sessions of one set of weights, released and started again in between."""
    cfg = M.parallel_config(EVERYTHING)
    tensors = M.weights(cfg, seed=12)
    oracle = M.oracle_model(cfg, tensors)
    root = M.session(cfg, tensors, 128, 1)
    pool = [root, root.fork_shared_weights()]
    for i, n in enumerate((61, 3, 128, 1, 2, 77)):
        tokens = tokens_of(cfg, n, seed=20 + i)
        oracle.reset()
        want, _ = oracle.run(tokens)
        s = pool[i % 2]
        s.release_sequence()
        assert M.errors(M.feed(s, tokens, [5, 1, 30]), want).max() < EXACT, n
    tokens = tokens_of(cfg, 50, seed=30)   # a fork carries the cache over, and both go on by themselves
    root.release_sequence()
    M.feed(root, tokens[:40], [40])
    child = root.fork_shared_weights()
    oracle.reset()
    want, _ = oracle.run(tokens)
    assert M.errors(M.feed(child, tokens[40:], [1]), want[40:]).max() < EXACT
    assert M.errors(M.feed(root, tokens[40:], [4, 6]), want[40:]).max() < EXACT
    for s in pool + [child]:
        s.destroy()


def test_long_decoding():
    cfg = M.parallel_config([M.latent(window=50), M.latent(window=300, experts=6, top=3)])
    for precision, n in ((1, 700), (0, 400)):
        check(cfg, weights(cfg, 13, precision), tokens_of(cfg, n), [20, 1], precision)


WIDE = {   # heads, key dim, value dim, rank, window
    "3 heads, rank 128": (3, 32, 16, 128, 40), "16 heads, rank 128": (16, 32, 16, 128, 1000), "40 heads, rank 128": (40, 32, 48, 128, 65),
    "33 heads, rank 256": (33, 64, 32, 256, 100), "5 heads, rank 512": (5, 128, 128, 512, 77), "100 heads, rank 128": (100, 32, 16, 128, 31),
}


@pytest.mark.parametrize("name", WIDE)
def test_wide_attention(name):
    from nerva_amd import abi
    heads, dim, vdim, rank, window = WIDE[name]
    cfg = M.parallel_config([M.latent(heads=heads, dim=dim, rot_dim=64, rot=rot, vdim=vdim, q_rank=40, kv_rank=rank, window=window, experts=0)
                             for rot in (64, 32)], width=64, vocab=50)
    tensors, tokens = M.weights(cfg, seed=14), tokens_of(cfg, 230, seed=6)
    want, _ = M.oracle_model(cfg, tensors).run(tokens)
    worst = {}
    for kernel in (0, 2):   # the wide kernels, then the general one
        abi.load().nerva_hip_test_set_tuning(b"latent_attention_wide", kernel)
        s = M.session(cfg, tensors, 256)
        for sizes in ([230], [100, 3, 1, 1, 45, 1], [17, 2, 1], [1]):
            s.release_sequence()
            worst[kernel, str(sizes)] = M.errors(M.feed(s, tokens, sizes), want).max()
        s.destroy()
    abi.load().nerva_hip_test_set_tuning(None, 0)
    assert max(worst.values()) < HALF, worst


def test_wide_layers_take_the_streaming_kernels():
    """Widths that the streaming and matrix-core kernels take (whole prompt blocks and the remainders between them)."""
    cfg = M.parallel_config([M.latent(heads=16, dim=128, rot_dim=64, vdim=128, q_rank=512, kv_rank=512, window=200, experts=12, top=3, ff=256,
                                      limit=1.5, shared=512), M.latent(heads=16, dim=32, rot_dim=64, vdim=128, q_rank=1024, kv_rank=128,
                                                                       window=300, experts=5, top=2, ff=1024, shared=0)], width=2048, vocab=256)
    tensors = M.clear_routes(cfg, M.weights(cfg, seed=15))
    tokens = tokens_of(cfg, 700, seed=7)
    oracle = M.oracle_model(cfg, tensors)
    oracle.w = {k: v.astype(np.float32) for k, v in oracle.w.items()}
    want, _ = oracle.run(tokens)
    s = M.session(cfg, tensors, 720)
    for sizes in ([700], [300, 130, 64, 2, 1, 1, 1, 20]):
        s.release_sequence()
        got = M.feed(s, tokens, sizes)
        assert M.errors(got, want).max() < HALF, sizes
    s.destroy()


@pytest.mark.parametrize("sizes", [[700], [400, 90, 80, 2, 1, 127]], ids=str)
def test_experts_with_many_tokens(sizes):
    """Blocks in which an expert has enough tokens for the large tiles: whole steps, rows past the last tile, uneven experts."""
    cfg = M.parallel_config([M.latent(experts=2, top=1, ff=192, limit=1.1, shared=128), M.latent(experts=3, top=2, ff=136, shared=320, shared_limit=0.9),
                             M.latent(experts=1, top=1, ff=64, shared=0)], width=128)
    check(cfg, weights(cfg, 24, 0), tokens_of(cfg, 700, seed=9), sizes, 0)


def test_greedy_generation_through_the_session_loop():
    """start / advance / run: every token is the plain statement's choice, or within rounding of it."""
    cfg = M.parallel_config(EVERYTHING)
    prompt = tokens_of(cfg, 37, seed=8)
    for precision, slack in ((1, 1e-4), (0, 0.15)):
        tensors = weights(cfg, 16, precision)
        s = M.session(cfg, tensors, 128, precision)
        rc, res = s.start(prompt)
        assert rc == 0 and res.kv_tokens == 37
        rc, res, first = s.advance(24)
        assert rc == 0 and res.observed_tokens == 24 and res.graph_replays == 23 and res.hot_path_allocations == 0
        rc, res, more = s.advance(10)
        assert rc == 0 and len(more) == 10
        stream = np.concatenate([first, more])
        want, _ = M.oracle_model(cfg, tensors).run(np.concatenate([prompt, stream[:-1]]))
        for i, token in enumerate(stream):
            row = want[36 + i]
            assert row[token] >= row.max() - slack * max(1.0, want.std()), (precision, i)
        rc, res, again = s.run(prompt, 34)
        assert rc == 0
        if precision:
            assert again.tolist() == stream.tolist()
        rc, _ = s.start(prompt, eos=int(stream[3]))
        rc, res, out = s.advance(20)
        assert rc == 0 and out.tolist() == stream[:list(stream).index(stream[3]) + 1].tolist()
        s.release_sequence()
        rc, _, _, _ = s.extend(prompt[:20])
        rc, _, _, _ = s.extend(prompt[20:])
        rc, _, out = s.advance(8)
        assert rc == 0 and (not precision or out.tolist() == stream[:8].tolist())
        s.destroy()


def test_sampled_generation_follows_the_samplers_rule():
    from nerva_amd import abi, sample, DeviceBuffer
    cfg = M.parallel_config([M.latent(), M.latent(experts=0)])
    tensors, prompt = M.weights(cfg, seed=17), tokens_of(cfg, 12)
    s = M.session(cfg, tensors, 64)
    for top_k, top_p in ((0, 1.0), (5, 0.9)):
        sampler = abi.NervaHipHfDecodeSamplerConfig()
        sampler.temperature, sampler.top_k, sampler.top_p, sampler.seed = 0.8, top_k, top_p, 99
        rc, _ = s.start(prompt, sampler=sampler)
        assert rc == 0
        rc, _, _ = s.advance(5)
        assert rc == 0
        rc, _, last = s.advance(1)
        token = sample(DeviceBuffer.from_numpy(s.logits()), cfg["vocab"], 0.8, top_p, top_k, 99, 12 + 4)
        assert token == int(last[0])
    s.destroy()


def test_batch_steps_of_unequal_sequences():
    from nerva_amd import DecodeSession
    cfg = M.parallel_config(EVERYTHING)
    root = M.session(cfg, M.weights(cfg, seed=18), 128, 1)
    group = [root] + [root.fork_shared_weights() for _ in range(3)]
    prompts = [tokens_of(cfg, n, seed=40 + n) for n in (1, 5, 33, 90)]
    streams = []
    for s, prompt in zip(group, prompts):
        rc, _ = s.start(prompt)
        rc, _, out = s.advance(1)
        assert rc == 0
        streams.append(out.tolist())
    for _ in range(6):
        rc, res, out = DecodeSession.batch_advance_one(group, 4, 2)
        assert rc == 0 and res.block_tokens == 4
        for stream, token in zip(streams, out):
            stream.append(int(token))
    solo = root.fork_shared_weights()
    for prompt, stream in zip(prompts, streams):
        rc, _ = solo.start(prompt)
        rc, _, out = solo.advance(7)
        assert rc == 0 and out.tolist() == stream
    for s in group + [solo]:
        s.destroy()


def test_replayed_steps_are_the_eager_ones():
    """A captured decode step, replayed, against the same tokens through prompt blocks of one session after the other."""
    cfg = M.parallel_config(EVERYTHING)
    tensors, prompt = weights(cfg, 22, 0), tokens_of(cfg, 20)
    s = M.session(cfg, tensors, 64)
    rc, _ = s.start(prompt)
    rc, res, tokens = s.advance(12)
    assert rc == 0 and res.graph_replays == 11
    last = s.logits()
    s.release_sequence()
    got = M.feed(s, np.concatenate([prompt, tokens[:-1]]).astype(np.uint32), [31])
    assert M.errors(last[None], got[-1:].astype(np.float64)).max() < HALF
    s.destroy()


def other_stack(layers, arrangement, seed):
    """A stack put together by hand, no architecture's: (StackConfig, tensors)."""
    from nerva_amd import stacks
    stack = stacks.StackConfig(40, 53, 1e-5, layers, arrangement, 2.0, 0.5 if arrangement == stacks.PARALLEL else 1.0)
    rng = np.random.default_rng(seed)
    tensors = {}
    for name, shape in stack.manifest():
        a = rng.normal(0, 1.0 / np.sqrt(shape[-1]), shape) if len(shape) == 2 else rng.normal(0.0 if name.endswith(".b") else 1.0, 0.2, shape)
        tensors[name] = M.bf16(a * (np.sqrt(40) if name == "embed" else 1.0))
    return stack, tensors


@PRECISIONS
def test_mechanisms_in_other_arrangements(precision):
    """Latent attention between two layer norms, and grouped attention, minGRU and a dense feed-forward in parallel layers."""
    from nerva_amd import DecodeSession, WeightPlan, stacks
    latent = stacks.LatentAttention(3, 8, 4, 6, 12, 16, 4, 100.0, 0.3, 9)
    grouped = stacks.Attention(4, 2, 12, 10, 6, 200.0, 0.3, 13)
    for arrangement, layers in ((stacks.SANDWICH, [(latent, stacks.XieluFeedForward(24)), (stacks.MinGru(20), None)]),
                                (stacks.PARALLEL, [(grouped, stacks.XieluFeedForward(24)), (stacks.MinGru(20), stacks.ExpertFeedForward(3, 3, 8, 1.0)),
                                                   (latent, None)])):
        stack, tensors = other_stack(layers, arrangement, 23)
        w = {k: M.value(v).astype(np.float64) for k, v in tensors.items()}
        tokens = tokens_of(dict(vocab=53), 40)
        part = lambda prefix: {k[len(prefix):]: v for k, v in w.items() if k.startswith(prefix)}
        x = w["embed"][tokens] * 2.0
        for i, (mixer, ff) in enumerate(layers):
            name = "l%d." % i
            sandwich = arrangement == stacks.SANDWICH
            norm = (lambda v, key: O.layer_norm(v, w[name + key], w[name + key + ".b"], 1e-5)) if sandwich else \
                (lambda v, key: O.rms_norm(v, w[name + key], 1e-5))
            h, mix = norm(x, "norm1"), part(name + "mix.")
            if mixer is latent:
                y = O.latent_attention_mixer(h, dict(heads=3, dim=8, rot_dim=4, vdim=6, kv_rank=16, rot=dict(dims=4, base=100.0),
                                                     mask=dict(size=9), scale=0.3), mix, dict(c=[], r=[]), 0, 1e-5)
            elif mixer is grouped:
                y = O.attention_mixer(h, dict(heads=4, kv_heads=2, dim=12, vdim=10, rot=dict(dims=6, base=200.0), mask=dict(size=13), scale=0.3),
                                      mix, dict(k=[], v=[]), 0)
            else:
                y, _ = O.mingru_mixer(h, mix, np.zeros(20))
            forward = (lambda v: O.feed_forward(v, part(name + "mlp."))) if isinstance(ff, stacks.XieluFeedForward) else \
                (lambda v: O.expert_feed_forward(v, dict(router=dict(top=3), expert=dict(limit=1.0)), part(name + "mlp.")))
            if sandwich:
                x = x + norm(y, "norm1b")
                if ff is not None:
                    x = x + norm(forward(norm(x, "norm2")), "norm2b")
            else:
                x = x + y + (forward(norm(x, "norm2")) if ff is not None else 0.0)
        want = O.layer_norm(x, w["final.norm"], w["final.norm.b"], 1e-5) @ w["embed"].T if arrangement == stacks.SANDWICH else \
            O.rms_norm(x, w["final.norm"], 1e-5) @ w["head"].T * 0.5
        s = DecodeSession.create_stack(stack, WeightPlan.from_weights(stacks.StackWeights(stack, tensors)), 48, precision)
        for sizes in ([40], [1], [7, 1, 2]):
            s.release_sequence()
            assert M.errors(M.feed(s, tokens, sizes), want).max() < (EXACT if precision else HALF)
        s.destroy()


def test_requests_that_do_not_fit_are_refused():
    cfg = M.parallel_config([M.latent(), M.latent()])
    s = M.session(cfg, M.weights(cfg), 20)
    assert s.extend([1] * 21)[0] == -1 and s.extend([cfg["vocab"]])[0] == -1
    assert s.extend([1, 2, 3], [3])[0] == -1 and s.extend([1, 2, 3], [1, 1])[0] == -1
    assert s.extend([1] * 20)[0] == 0 and s.extend([1])[0] == -1
    s.destroy()
    from nerva_amd import DecodeSession, WeightPlan, stacks
    for change in (dict(rotary_dims=3), dict(rotary_dims=8), dict(kv_rank=0), dict(kv_rank=5000), dict(heads=0), dict(score_scale=float("nan"))):
        stack = stacks.READERS["Kavuvik"](cfg)
        for k, v in change.items():
            setattr(stack.layers[1][0], k, v)
        with pytest.raises(RuntimeError):
            DecodeSession.create_stack_synthetic(stack, 16)
    for change in (dict(top=0), dict(top=6), dict(experts=2000), dict(ff=0), dict(limit=-1.0)):
        stack = stacks.READERS["Kavuvik"](cfg)
        for k, v in change.items():
            setattr(stack.layers[0][1], k, v)
        with pytest.raises(RuntimeError):
            DecodeSession.create_stack_synthetic(stack, 16)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_replay_from_a_folder(tmp_path, dtype):
    """bin/trace_run over a folder: two requests alive at once, portions, single tokens, places in any order."""
    cfg = M.parallel_config(EVERYTHING)
    tensors = weights(cfg, 19, dtype == "float32")
    M.write_folder(str(tmp_path / "model"), cfg, tensors)
    a, b = tokens_of(cfg, 40, seed=50), tokens_of(cfg, 25, seed=51)
    steps = [([("a", a[:30], [29, 0, 7])], []), ([("b", b[:2], [])], []), ([("a", a[30:31], [0])], []), ([("b", b[2:], [22, 4])], ["b"]),
             ([("a", a[31:], [8])], ["a"]), ([("c", b, [24])], ["c"])]
    text = "".join(json.dumps(dict(step=i, entries=[dict(id=n, tokens=t.tolist(), want=w) for n, t, w in entries], end=end)) + "\n"
                   for i, (entries, end) in enumerate(steps))
    out = tmp_path / "out"
    out.mkdir()
    run = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path / "model"), "--dtype", dtype,
                          "--out", str(out), "--max-tokens", "65"], input=text, capture_output=True, text=True, timeout=100)
    assert run.returncode == 0, run.stderr[-2000:]
    want = {"a": M.oracle_model(cfg, tensors).run(a)[0], "b": M.oracle_model(cfg, tensors).run(b)[0]}
    want["c"] = want["b"]
    at = {}
    for i, (entries, _) in enumerate(steps):
        for name, t, places in entries:
            first = at.get(name, 0)
            at[name] = first + len(t)
            path = out / ("%d.f32" % i)
            assert path.exists() == bool(places)
            if places:
                got = np.fromfile(path, "<f4").reshape(len(places), cfg["vocab"])
                assert M.errors(got, want[name][[first + w for w in places]]).max() < (EXACT if dtype == "float32" else HALF)


def test_generation_from_a_folder(tmp_path):
    """bin/generate over a folder gives the tokens of a session over the same weights in memory."""
    cfg = M.parallel_config([M.latent(), M.latent(window=4)])
    tensors, prompt = M.weights(cfg, seed=21), tokens_of(cfg, 9)
    M.write_folder(str(tmp_path), cfg, tensors)
    s = M.session(cfg, tensors, 32, 1)
    rc, _ = s.start(prompt)
    rc, _, tokens = s.advance(12)
    s.destroy()
    run = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "generate"), "--model", str(tmp_path), "--dtype", "float32", "--steps", "12",
                          "--prompt", ",".join(str(t) for t in prompt)], capture_output=True, text=True, timeout=100)
    assert run.returncode == 0, run.stderr[-2000:]
    assert run.stdout.strip() == ",".join(str(t) for t in tokens)
