"""Mixed layer stacks without a GPU: reading a config.json, the arena's tensor order, file-backed plans, refusals, and
the plain statement (oracle/mixed_stack.py) held to what its mechanisms must do."""
import copy
import json

import numpy as np
import pytest

import stack_models as M
from nerva_amd import WeightPlan, checkpoint, stacks
from oracle import mixed_stack as O

CFG = M.config([M.attention(), M.mingru(), M.attention(kv_from=0, chunk=29, ff=0), M.mingru(width=20, ff=0)])


def test_the_reader_takes_every_size_and_constant_from_the_config():
    stack = checkpoint.parse_config(CFG)["stack"]
    layers = stack.c_layers()
    first, last = CFG["layers"][0]["mixer"], CFG["layers"][2]["mixer"]
    assert (layers[0].heads, layers[0].kv_heads, layers[0].key_dim, layers[0].value_dim, layers[0].chunk_tokens) == (
        first["heads"], first["kv_heads"], first["dim"], first["vdim"], first["mask"]["size"])
    assert layers[0].rotary_dims == first["rot"]["dims"] and layers[0].rotary_base == first["rot"]["base"]
    assert abs(layers[0].score_scale - first["scale"]) < 1e-7
    assert layers[0].kv_layer == stacks.OWN_KEYS and layers[2].kv_layer == 0 and layers[2].chunk_tokens == last["mask"]["size"]
    assert (layers[1].width, layers[1].ff, layers[3].width, layers[3].ff) == (56, 40, 20, 0)
    assert (stack.hidden, stack.vocab, stack.eps) == (CFG["width"], CFG["vocab"], CFG["norm"]["eps"])
    assert (stack.arrangement, stack.embedding_scale, stack.logit_scale) == (stacks.SANDWICH, 1.0, 1.0)


PARALLEL = M.parallel_config([M.latent(), M.latent(heads=5, dim=6, rot_dim=8, rot=4, vdim=3, q_rank=9, kv_rank=14, window=70, experts=0),
                              M.latent(experts=7, top=3, ff=11, limit=0.25, shared=0)])


def test_parallel_layers_are_read_likewise():
    stack = checkpoint.parse_config(PARALLEL)["stack"]
    a, b, c = stack.c_layers()
    m = PARALLEL["layers"][1]["mixer"]
    assert (b.mixer, b.heads, b.key_dim, b.rotary_key_dim, b.value_dim, b.q_rank, b.kv_rank, b.window_tokens) == (
        stacks.LatentAttention.kind, m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["q_rank"], m["kv_rank"], m["mask"]["size"])
    assert (b.rotary_dims, b.rotary_base, b.experts, b.shared_ff) == (4, m["rot"]["base"], 0, 0) and abs(b.score_scale - m["scale"]) < 1e-7
    assert (a.experts, a.experts_per_token, a.expert_ff, a.shared_ff, a.ff) == (5, 2, 24, 20, 0)
    assert abs(a.expert_limit - 0.8) < 1e-6 and abs(a.shared_limit - 1.3) < 1e-6
    assert (c.experts, c.experts_per_token, c.expert_ff, c.shared_ff, c.expert_limit) == (7, 3, 11, 0, 0.25)
    assert (stack.arrangement, stack.embedding_scale, stack.logit_scale) == (
        stacks.PARALLEL, PARALLEL["embedding"]["scale"], PARALLEL["logit_scale"])
    shapes = dict(stack.manifest())
    assert len(shapes) == len(stack.manifest()) and list(shapes)[0] == "embed" and list(shapes)[-2:] == ["final.norm", "head"]
    assert shapes["l1.mix.uq"] == [5 * 14, 9] and shapes["l1.mix.dkv"] == [22, 44] and shapes["l2.mlp.e6.down"] == [44, 11]
    assert "l1.norm2" not in shapes and "l0.norm2" in shapes and "l0.mlp.shared.up" in shapes and "l2.mlp.shared.up" not in shapes
    without = copy.deepcopy(PARALLEL)
    without["layers"][0]["mixer"]["mask"] = None
    assert checkpoint.parse_config(without)["stack"].c_layers()[0].window_tokens == 0


def test_manifest_names_each_tensor_once():
    names = [n for n, _ in checkpoint.tensor_manifest(checkpoint.parse_config(CFG))]
    assert len(names) == len(set(names))
    assert names[0] == "embed" and names[-2:] == ["final.norm", "final.norm.b"]
    assert "l0.mix.k" in names and "l2.mix.k" not in names and "l2.mix.v" not in names
    assert "l2.norm2" not in names and "l2.mlp.up" not in names and "l1.mix.z.b" in names


def test_plan_points_at_the_tensors_bytes(tmp_path):
    tensors = M.weights(CFG)
    M.write_folder(str(tmp_path), CFG, tensors)
    plan = checkpoint.plan_checkpoint(str(tmp_path))
    offset = 0
    with open(tmp_path / "model.safetensors", "rb") as f:
        for (name, _, begin, size), block in zip(plan.entries, plan.blocks):
            f.seek(begin)
            assert f.read(size) == tensors[name].tobytes()
            assert (block.offset_bytes, block.bytes) == (offset, size)
            offset += size
    stack = plan.cfg["stack"]
    memory = WeightPlan.from_weights(stacks.StackWeights(stack, tensors))
    assert memory.descriptor_hash == plan.descriptor_hash


def broken(change):
    cfg = copy.deepcopy(CFG)
    change(cfg)
    return cfg


@pytest.mark.parametrize("change", [
    lambda c: c.pop("width"), lambda c: c.update(vocab=0), lambda c: c.update(layers=[]), lambda c: c["norm"].pop("eps"),
    lambda c: c["layers"][0].update(type="other"), lambda c: c["layers"][0]["mixer"].update(heads=3),
    lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7), lambda c: c["layers"][0]["mixer"]["rot"].update(dims=18),
    lambda c: c["layers"][0]["mixer"].pop("mask"), lambda c: c["layers"][2]["mixer"].update(kv_from=1),
    lambda c: c["layers"][2]["mixer"].update(kv_from=2), lambda c: c["layers"][2]["mixer"].update(vdim=8),
    lambda c: c["layers"][0].update(mlp=dict(kind="sparse", ff=4)), lambda c: c["layers"][1]["mixer"].update(width=1.5),
], ids=range(14))
def test_configs_that_do_not_describe_a_model_are_refused(change):
    with pytest.raises(stacks.CheckpointError):
        checkpoint.parse_config(broken(change))


@pytest.mark.parametrize("change", [
    lambda c: c.pop("logit_scale"), lambda c: c["embedding"].pop("scale"), lambda c: c["norm"].update(eps=-1.0), lambda c: c.update(vocab=1.5),
    lambda c: c["layers"][0].update(type="attention"), lambda c: c["layers"][0]["mixer"].pop("q_rank"),
    lambda c: c["layers"][0]["mixer"]["rot"].update(dims=5), lambda c: c["layers"][0]["mixer"]["rot"].update(dims=8),
    lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), lambda c: c["layers"][0]["mixer"].update(scale=float("nan")),
    lambda c: c["layers"][0]["mlp"].update(kind="dense"), lambda c: c["layers"][0]["mlp"]["router"].update(top=6),
    lambda c: c["layers"][0]["mlp"]["router"].pop("experts"), lambda c: c["layers"][0]["mlp"]["expert"].pop("limit"),
    lambda c: c["layers"][0]["mlp"]["shared"].update(ff=0), lambda c: c["layers"][0]["mlp"]["shared"].update(limit=-1.0),
], ids=range(16))
def test_parallel_configs_that_do_not_describe_a_model_are_refused(change):
    cfg = copy.deepcopy(PARALLEL)
    change(cfg)
    with pytest.raises(stacks.CheckpointError):
        checkpoint.parse_config(cfg)


def test_parallel_plan_points_at_the_tensors_bytes(tmp_path):
    tensors = M.weights(PARALLEL)
    M.write_folder(str(tmp_path), PARALLEL, tensors)
    plan = checkpoint.plan_checkpoint(str(tmp_path))
    with open(tmp_path / "model.safetensors", "rb") as f:
        for name, _, begin, size in plan.entries:
            f.seek(begin)
            assert f.read(size) == tensors[name].tobytes()
    memory = WeightPlan.from_weights(stacks.StackWeights(plan.cfg["stack"], tensors))
    assert memory.descriptor_hash == plan.descriptor_hash


def test_folders_that_do_not_hold_the_model_are_refused(tmp_path):
    tensors = M.weights(CFG)
    for i, change in enumerate((lambda t: t.pop("l1.mix.x.b"), lambda t: t.update({"l0.mix.talk": t["l0.mix.talk"][:2]}))):
        some = dict(tensors)
        change(some)
        M.write_folder(str(tmp_path / str(i)), CFG, some)
        with pytest.raises(stacks.CheckpointError):
            checkpoint.plan_checkpoint(str(tmp_path / str(i)))


def test_unknown_architectures_stay_with_the_dense_reader():
    with pytest.raises(stacks.CheckpointError):
        checkpoint.parse_config(dict(CFG, architecture="Unheard"))
    assert json.loads(json.dumps(CFG)) == CFG


# ---- the plain statement ----------------------------------------------------------------------

def test_oracle_portions_are_the_whole():
    tensors, tokens = M.weights(CFG, seed=2), np.random.default_rng(0).integers(0, CFG["vocab"], 50)
    m = M.oracle_model(CFG, tensors)
    whole, _ = m.run(tokens)
    m.reset()
    parts = np.concatenate([m.run(t)[0] for t in np.split(tokens, [1, 3, 20, 21, 47])])
    assert np.abs(parts - whole).max() < 1e-9


def test_oracle_chunks_end_what_a_token_sees():
    cfg = M.config([M.attention(chunk=10, ff=0)])
    m = M.oracle_model(cfg, M.weights(cfg))
    tokens = np.arange(30) % cfg["vocab"]
    base, _ = m.run(tokens)
    changed = tokens.copy()
    changed[[9, 12]] = 77
    m.reset()
    other, _ = m.run(changed)
    moved = np.abs(other - base).max(-1) > 1e-9
    assert moved.tolist() == [i == 9 or 12 <= i < 20 for i in range(30)]


def test_oracle_mechanisms():
    rng = np.random.default_rng(1)
    x = rng.normal(3.0, 2.0, (5, 64))
    n = O.layer_norm(x, np.ones(64), np.zeros(64), 0.0)
    assert np.abs(n.mean(-1)).max() < 1e-12 and np.abs((n * n).mean(-1) - 1).max() < 1e-12
    # a rotation keeps lengths and, between two positions, depends on their distance only
    q, k = rng.normal(size=(1, 12)), rng.normal(size=(1, 12))
    near = (O.rotate(q, 7, 8, 100.0) * O.rotate(k, 5, 8, 100.0)).sum()
    far = (O.rotate(q, 107, 8, 100.0) * O.rotate(k, 105, 8, 100.0)).sum()
    assert abs(near - far) < 1e-9 and abs(np.linalg.norm(O.rotate(q, 9, 8, 100.0)) - np.linalg.norm(q)) < 1e-12
    # the sink takes weight and gives nothing; far below the scores it does nothing
    s = rng.normal(size=(2, 6))
    w = O.softmax_with_sink(s, np.array([1.0, -80.0]))
    assert w[0].sum() < 1 and abs(w[1].sum() - 1) < 1e-12
    assert abs(w[0, 0] - np.exp(s[0, 0]) / (np.exp(s[0]).sum() + np.exp(1.0))) < 1e-12
    # continuous at zero, slope one half there
    z = np.array([-1e-4, 0.0, 1e-4])
    y = O.xielu(z, 0.3, -0.2)
    assert y[1] == 0 and abs((y[2] - y[0]) / 2e-4 - 0.5) < 1e-3
    # a closed gate keeps the state, an open one replaces it
    w = dict(z=np.zeros((2, 3)), x=np.zeros((2, 3)), g=np.zeros((2, 3)), o=np.zeros((3, 2)))
    w["z.b"], w["x.b"] = np.array([-60.0, 60.0]), np.array([0.25, -1.0])
    _, state = O.mingru_mixer(np.ones((1, 3)), w, np.array([5.0, 5.0]))
    assert abs(state[0] - 5.0) < 1e-12 and abs(state[1] - 1 / (1 + np.exp(1.0))) < 1e-12


def test_oracle_parallel_portions_are_the_whole():
    tensors, tokens = M.weights(PARALLEL, seed=2), np.random.default_rng(0).integers(0, PARALLEL["vocab"], 50)
    m = M.oracle_model(PARALLEL, tensors)
    whole, _ = m.run(tokens)
    m.reset()
    parts = np.concatenate([m.run(t)[0] for t in np.split(tokens, [1, 3, 20, 21, 47])])
    assert np.abs(parts - whole).max() < 1e-9


def test_oracle_windows_end_what_a_token_sees():
    cfg = M.parallel_config([M.latent(window=10, experts=0)])
    m = M.oracle_model(cfg, M.weights(cfg))
    tokens = np.arange(30) % cfg["vocab"]
    base, _ = m.run(tokens)
    changed = tokens.copy()
    changed[7] = 77
    m.reset()
    other, _ = m.run(changed)
    assert (np.abs(other - base).max(-1) > 1e-9).tolist() == [7 <= i < 17 for i in range(30)]


def test_oracle_latent_attention_is_attention_with_expanded_keys():
    """Against the grouped-query function on keys and values written out: [unrotated, rotated] per head, every head its own."""
    rng = np.random.default_rng(3)
    H, d, rd, dv, rank, width = 3, 4, 2, 5, 6, 8
    w = {k: rng.normal(size=s) for k, s in dict(dq=(7, width), uq=(H * (d + rd), 7), dkv=(rank + rd, width), uk=(H * d, rank), uv=(H * dv, rank),
                                                g=(H * dv, width), o=(width, H * dv)).items()}
    w["dq.norm"], w["dkv.norm"] = rng.normal(1, 0.2, 7), rng.normal(1, 0.2, rank)
    h = rng.normal(size=(9, width))
    mixer = dict(heads=H, dim=d, rot_dim=rd, vdim=dv, kv_rank=rank, rot=dict(dims=rd, base=10.0), mask=dict(size=4), scale=0.4)
    got = O.latent_attention_mixer(h, mixer, w, dict(c=[], r=[]), 0, 1e-5)
    c = O.rms_norm(h @ w["dkv"][:rank].T, w["dkv.norm"], 1e-5)
    q = (O.rms_norm(h @ w["dq"].T, w["dq.norm"], 1e-5) @ w["uq"].T).reshape(9, H, d + rd)
    keys = np.concatenate([(c @ w["uk"].T).reshape(9, H, d),
                           np.stack([np.repeat(O.rotate((h[t] @ w["dkv"][rank:].T)[None], t, rd, 10.0), H, 0) for t in range(9)])], -1)
    values = (c @ w["uv"].T).reshape(9, H, dv)
    for t in range(9):
        qt = q[t].copy()
        qt[:, d:] = O.rotate(qt[:, d:], t, rd, 10.0)
        lo = O.window_start(t, 4)
        a = O.attend(qt, keys[lo:t + 1], values[lo:t + 1], 0.4, np.eye(H), np.full(H, -1e9))
        assert np.abs(w["o"] @ (a.reshape(-1) * O.sigmoid(w["g"] @ h[t])) - got[t]).max() < 1e-9


def test_oracle_expert_mechanisms():
    # bounds: the gate from above only, the linear part on both sides, which moves up by one
    assert O.clamped_glu(np.array(9.0), np.array(-9.0), 2.0) == O.clamped_glu(np.array(2.0), np.array(-2.0), 2.0)
    assert O.clamped_glu(np.array(-9.0), np.array(0.5), 2.0) != O.clamped_glu(np.array(-2.0), np.array(0.5), 2.0)
    assert O.clamped_glu(np.array(1.0), np.array(-1.0), 2.0) == 0.0
    # the largest scores, in order, the lower index first among equals; weights are the scores' own shares
    chosen, weights = O.choose_experts(np.array([0.1, 2.0, -1.0, 2.0, 0.3]), 3)
    assert chosen.tolist() == [1, 3, 4] and abs(weights.sum() - 1) < 1e-12
    assert abs(weights[2] / weights[0] - O.sigmoid(0.3) / O.sigmoid(2.0)) < 1e-12
    # the root mean square, not the deviation: a constant row keeps its sign and gets length one
    assert np.abs(O.rms_norm(np.full((1, 5), -3.0), np.ones(5), 0.0) + 1).max() < 1e-12
