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
