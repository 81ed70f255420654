"""Sessions over mixed layer stacks on the GPU against the plain statement of oracle/mixed_stack.py: every mechanism
alone, whole prompts, portions, decoding, chunk edges, reused sessions, sizes that take the wide kernels, generation."""
import os
import subprocess
import sys

import json

import numpy as np
import pytest

import stack_models as M

pytestmark = pytest.mark.gpu

EXACT, HALF = 3e-5, 0.05        # 32-bit and 16-bit sessions, relative to the logits' spread
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
EVERYTHING = [M.attention(), M.mingru(), M.attention(kv_from=0, chunk=29, ff=0), M.attention(heads=6, kv_heads=1, dim=10, vdim=7, rot=6, chunk=8),
              M.mingru(width=33, ff=0), M.attention(kv_from=0, chunk=13), M.mingru(width=64, ff=72)]


def tokens_of(cfg, n, seed=1):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).astype(np.uint32)


def check(cfg, tensors, tokens, sizes, precision, limit=None, max_context=None):
    s = M.session(cfg, tensors, max_context or len(tokens), precision)
    got = M.feed(s, tokens, sizes)
    want, _ = M.oracle_model(cfg, tensors).run(tokens)
    s.destroy()
    worst = M.errors(got, want)
    limit = limit or (EXACT if precision else HALF)
    assert worst.max() < limit, "position %d: %.2e" % (int(worst.argmax()), worst.max())


ALONE = {
    "feed-forward": [M.mingru(width=1)],
    "mingru": [M.mingru(ff=0)],
    "mingru narrow": [M.mingru(width=3, ff=0)],
    "attention": [M.attention(ff=0)],
    "one head": [M.attention(heads=1, kv_heads=1, dim=8, vdim=8, rot=8, ff=0)],
    "own kv head each": [M.attention(heads=3, kv_heads=3, dim=12, vdim=5, rot=2, ff=0)],
    "no rotation": [M.attention(rot=0, ff=0)],
    "full rotation": [M.attention(rot=16, base=20.0, ff=0)],
    "chunk of one": [M.attention(chunk=1, ff=0)],
    "chunk of two": [M.attention(chunk=2, ff=0)],
    "chunk of a block": [M.attention(chunk=16, ff=0)],
    "no chunk reached": [M.attention(chunk=1000, ff=0)],
    "negative scale": [M.attention(scale=-0.7, ff=0)],
    "borrowed keys": [M.attention(chunk=7, ff=0), M.attention(chunk=19, kv_from=0, ff=0)],
    "everything": EVERYTHING,
}


@pytest.mark.parametrize("precision", [1, 0], ids=["f32", "bf16"])
@pytest.mark.parametrize("name", ALONE)
def test_mechanism(name, precision):
    cfg = M.config(ALONE[name])
    check(cfg, M.weights(cfg, seed=3), tokens_of(cfg, 45), [45], precision)


@pytest.mark.parametrize("precision", [1, 0], ids=["f32", "bf16"])
def test_residual_rows_after_every_layer(precision):
    cfg = M.config(EVERYTHING)
    tensors, tokens = M.weights(cfg, seed=4), tokens_of(cfg, 30)
    s = M.session(cfg, tensors, 64, precision)
    rc, _, logits, rows = s.extend(tokens, [29], residual_layers=len(EVERYTHING))
    assert rc == 0
    want, trail = M.oracle_model(cfg, tensors).run(tokens)
    spread = np.sqrt((trail ** 2).mean())
    for l in range(len(EVERYTHING)):
        assert np.sqrt(((rows[l] - trail[l]) ** 2).mean()) / spread < (1e-5 if precision else 0.02), l
    assert M.errors(logits, want[29:]).max() < (EXACT if precision else HALF)
    # reading the rows back changes nothing that comes after
    rc, _, after, _ = s.extend(tokens[:1], [0])
    want, _ = M.oracle_model(cfg, tensors).run(np.append(tokens, tokens[0]))
    assert rc == 0 and M.errors(after, want[30:]).max() < (EXACT if precision else HALF)
    s.destroy()


@pytest.mark.parametrize("precision", [1, 0], ids=["f32", "bf16"])
@pytest.mark.parametrize("sizes", [[1], [2], [3, 1, 7, 2], [16], [40, 1, 1, 1], [13, 13, 29], [1, 60]], ids=str)
def test_portions(sizes, precision):
    cfg = M.config(EVERYTHING)
    check(cfg, M.weights(cfg, seed=5), tokens_of(cfg, 80, seed=2), sizes, precision)


@pytest.mark.parametrize("eps", [1e-12, 0.3])
def test_norm_constant(eps):
    cfg = M.config([M.mingru(), M.attention()], eps=eps)
    check(cfg, M.weights(cfg, seed=6), tokens_of(cfg, 20), [20], 1)


@pytest.mark.parametrize("width", [1, 3, 8, 50, 136, 520, 1024, 1030])
def test_model_widths(width):
    cfg = M.config([M.attention(ff=24), M.mingru(width=40, ff=9)], width=width, vocab=33)
    if width == 1:   # a row of one value is all mean: every norm gives its bias
        cfg["norm"]["eps"] = 0.5
    tensors, tokens = M.weights(cfg, seed=7), tokens_of(cfg, 21)
    check(cfg, tensors, tokens, [11, 1, 9], 1)
    check(cfg, tensors, tokens, [11, 1, 9], 0)


def needle_model(chunk, dim, heads, kv_heads, width=64, vocab=40, readers=1):
    """Token 1 asks, token 0 answers: where token 0 is visible its key outscores everything, and its value is large."""
    layers = [M.attention(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, rot=dim // 2, chunk=chunk, ff=0)]
    layers += [M.attention(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, rot=dim // 2, chunk=chunk + 5, kv_from=0, ff=0)
               for _ in range(readers - 1)]
    cfg = M.config(layers, width=width, vocab=vocab)
    tensors = M.weights(cfg, seed=8)
    rng = np.random.default_rng(9)
    embed = M.value(tensors["embed"]) * 0.3
    asks, answers = np.zeros(width), np.zeros(width)
    asks[0], answers[1] = 1.0, 1.0
    embed[:, :2] = 0.0
    embed[1], embed[0] = embed[1] + 6 * asks, embed[0] + 6 * answers
    tensors["embed"] = M.bf16(embed)
    for l in range(readers):
        name = "l%d." % l
        tensors[name + "norm1"] = M.bf16(np.ones(width))
        tensors[name + "norm1.b"] = M.bf16(np.zeros(width))
        q = rng.normal(0, 0.05, (heads, dim, width))
        q[:, dim - 1] += 1.5 * asks               # a dimension that is not rotated
        tensors[name + "mix.q"] = M.bf16(q.reshape(heads * dim, width))
        tensors[name + "mix.sink"] = M.bf16(np.full(heads, -2.0))
        tensors[name + "mix.talk"] = M.bf16(np.eye(heads) + rng.normal(0, 0.05, (heads, heads)))
    k = rng.normal(0, 0.05, (kv_heads, dim, width))
    k[:, dim - 1] += 1.5 * np.sqrt(dim) * answers
    tensors["l0.mix.k"] = M.bf16(k.reshape(kv_heads * dim, width))
    v = M.value(tensors["l0.mix.v"]).copy()
    v[:, 1] = rng.normal(0, 3.0, kv_heads * dim)
    tensors["l0.mix.v"] = M.bf16(v)
    return cfg, tensors


@pytest.mark.parametrize("shape", [(16, 4, 2), (128, 16, 4), (128, 32, 8)], ids=["general", "wide 16", "wide 32"])
@pytest.mark.parametrize("chunk", [16, 37, 48])
def test_one_key_at_a_chunk_edge(chunk, shape):
    """A key that decides the answer, at the first and last position of a chunk and just across its edge, asked for from a
    prompt and from a decoded token; and the plain statement itself must tell the cases apart."""
    dim, heads, kv_heads = shape
    cfg, tensors = needle_model(chunk, dim, heads, kv_heads)
    oracle = M.oracle_model(cfg, tensors)
    s = M.session(cfg, tensors, 4 * chunk + 8)
    fill = np.random.default_rng(3).integers(2, cfg["vocab"], 4 * chunk + 8)
    seen = {}
    for needle, ask in ((0, chunk - 1), (0, chunk), (chunk - 1, chunk), (chunk, chunk + 1), (chunk, 2 * chunk - 1), (chunk, 2 * chunk),
                        (2 * chunk, 3 * chunk - 1), (2 * chunk - 1, 3 * chunk - 1), (2 * chunk, 3 * chunk)):
        if needle == ask:
            continue
        tokens = fill[:ask + 1].copy()
        tokens[needle], tokens[ask] = 0, 1
        oracle.reset()
        want = oracle.run(tokens)[0][-1:]
        tokens[needle] = fill[needle]
        oracle.reset()
        without = oracle.run(tokens)[0][-1:]
        tokens[needle] = 0
        inside = needle // chunk == ask // chunk
        told = M.errors(without, want).max()
        assert told > 0.12 if inside else told < 1e-9
        for sizes in ([ask + 1], [ask, 1], [max(1, ask - 2), 3]):
            s.release_sequence()
            got = M.feed(s, tokens.astype(np.uint32), sizes)[-1:]
            assert M.errors(got, want).max() < 0.03, (needle, ask, sizes)
        seen[inside] = True
    assert len(seen) == 2
    s.destroy()


def test_borrowed_keys_with_a_wider_chunk_than_the_owner():
    cfg, tensors = needle_model(21, 16, 4, 2, readers=2)
    tokens = np.random.default_rng(5).integers(2, cfg["vocab"], 120)
    tokens[[3, 22, 25, 47, 77]] = 0
    tokens[[20, 23, 26, 51, 52, 90, 103]] = 1
    for sizes in ([120], [50, 1, 1, 9, 1], [1]):
        check(cfg, tensors, tokens.astype(np.uint32), sizes, 1)


def test_the_block_ring_wraps():
    """Contexts far longer than a layer's ring of cache blocks, prompts and decoding; a layer that borrows the keys with a
    chunk of its own sizes the ring for both."""
    cfg = M.config([M.attention(heads=2, kv_heads=1, dim=8, vdim=8, rot=4, chunk=24, ff=0), M.mingru(width=16, ff=0),
                    M.attention(heads=2, kv_heads=1, dim=8, vdim=8, rot=4, chunk=70, kv_from=0, ff=0)], width=24, vocab=31)
    tensors, tokens = M.weights(cfg, seed=11), tokens_of(cfg, 2300)
    s = M.session(cfg, tensors, 2400, 1)
    assert s.create_result.resident_kv_bytes < 2400 * 16 * 4 / 2
    want, _ = M.oracle_model(cfg, tensors).run(tokens)
    for sizes in ([2300], [700, 511, 513, 2, 512, 40, 1]):
        s.release_sequence()
        assert M.errors(M.feed(s, tokens, sizes), want).max() < EXACT
    s.destroy()


def test_sessions_are_reused_and_forked():
    """Sequences of unequal length on sessions of one set of weights, released and started again in between."""
    cfg = M.config(EVERYTHING)
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
    # a fork carries cache and recurrent state over, and both go on by themselves
    tokens = tokens_of(cfg, 50, seed=30)
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
    cfg = M.config([M.attention(chunk=50), M.mingru(), M.attention(kv_from=0, chunk=300), M.mingru()])
    check(cfg, M.weights(cfg, seed=13), tokens_of(cfg, 700), [20, 1], 1)
    check(cfg, M.weights(cfg, seed=13), tokens_of(cfg, 400), [20, 1], 0)


WIDE = {
    "16 heads": [M.attention(16, 8, 128, 128, rot=128, base=1e6, chunk=100, ff=256), M.mingru(128, ff=0)],
    "16 heads, 4 kv": [M.attention(16, 4, 128, 128, rot=32, chunk=333, ff=0), M.attention(16, 4, 128, 128, rot=32, chunk=41, kv_from=0, ff=0)],
    "32 heads": [M.attention(32, 8, 128, 128, rot=64, chunk=90, ff=0), M.mingru(64)],
    "32 heads, 4 kv": [M.attention(32, 4, 128, 128, rot=128, chunk=70, ff=0)],
    "16 heads, 2 kv": [M.attention(16, 2, 128, 128, rot=0, chunk=1000, ff=0)],
}


@pytest.mark.parametrize("name", WIDE)
def test_wide_attention(name):
    from nerva_amd import abi
    cfg = M.config(WIDE[name], width=64, vocab=50)
    tensors, tokens = M.weights(cfg, seed=14), tokens_of(cfg, 230, seed=6)
    want, _ = M.oracle_model(cfg, tensors).run(tokens)
    worst = {}
    for kernel in (0, 2):   # the wide kernels, then the general one
        abi.load().nerva_hip_test_set_tuning(b"mixed_attention_wide", kernel)
        s = M.session(cfg, tensors, 256)
        for sizes in ([230], [100, 3, 1, 1, 45, 1], [17, 2, 1], [1]):
            s.release_sequence()
            worst[kernel, str(sizes)] = M.errors(M.feed(s, tokens, sizes), want).max()
        s.destroy()
    assert max(worst.values()) < HALF, worst


def test_wide_layers_take_the_streaming_kernels():
    """Widths that the lean GEMVs and the multi-row matrix-core kernels take (512-, 256- and 128-token blocks and the
    remainders between them), against the plain statement."""
    cfg = M.config([M.mingru(2048, ff=2048), M.attention(16, 8, 128, 128, rot=128, chunk=200, ff=6144)], width=2048, vocab=256)
    tensors = M.weights(cfg, seed=15)
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


def test_greedy_generation_through_the_session_loop():
    """start / advance / run in a 32-bit session: every token is the plain statement's choice, or within rounding of it."""
    cfg = M.config(EVERYTHING)
    tensors, prompt = M.weights(cfg, seed=16), tokens_of(cfg, 37, seed=8)
    for precision, slack in ((1, 1e-4), (0, 0.15)):
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
            assert row[token] >= row.max() - slack, (precision, i)
        rc, res, again = s.run(prompt, 34)          # the prompt walked token by token
        assert rc == 0
        if precision:
            assert again.tolist() == stream.tolist()
        # a stop token ends the sequence; the session goes on with another one
        rc, _ = s.start(prompt, eos=int(stream[3]))
        rc, res, out = s.advance(20)
        assert rc == 0 and out.tolist() == stream[:list(stream).index(stream[3]) + 1].tolist()
        # go on from a running sequence with given tokens: as if all of it had been the prompt
        s.release_sequence()
        rc, _, _, _ = s.extend(prompt[:20])
        rc, _, _, _ = s.extend(prompt[20:])
        rc, _, out = s.advance(8)
        assert rc == 0 and (not precision or out.tolist() == stream[:8].tolist())
        s.destroy()


def test_sampled_generation_follows_the_samplers_rule():
    from nerva_amd import abi, sample, DeviceBuffer
    cfg = M.config([M.attention(), M.mingru()])
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
        logits = s.logits()
        token = sample(DeviceBuffer.from_numpy(logits), cfg["vocab"], 0.8, top_p, top_k, 99, 12 + 4)
        assert token == int(last[0])
    s.destroy()


def test_batch_steps_of_unequal_sequences():
    cfg = M.config(EVERYTHING)
    tensors = M.weights(cfg, seed=18)
    from nerva_amd import DecodeSession
    root = M.session(cfg, tensors, 128, 1)
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


def test_requests_that_do_not_fit_are_refused():
    cfg = M.config([M.attention(), M.mingru()])
    s = M.session(cfg, M.weights(cfg), 20)
    assert s.extend([1] * 21)[0] == -1 and s.extend([cfg["vocab"]])[0] == -1
    assert s.extend([1, 2, 3], [3])[0] == -1 and s.extend([1, 2, 3], [1, 1])[0] == -1
    assert s.extend([1] * 20)[0] == 0 and s.extend([1])[0] == -1
    assert s.profile_step(1)[0] == -1 and s.lib.nerva_hip_session_step_trace_bytes(s.handle) == 0
    s.destroy()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_replay_from_a_folder(tmp_path, dtype):
    """bin/trace_run over a folder: two requests alive at once, portions, single tokens, places in any order."""
    cfg = M.config(EVERYTHING)
    tensors = M.weights(cfg, seed=19)
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
    assert [l for l in run.stdout.splitlines() if l.startswith("done")] == ["done %d" % i for i in range(len(steps))]
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
    cfg = M.config([M.attention(), M.mingru()])
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
