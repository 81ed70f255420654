"""Small random models of mixed layer stacks for the tests: configurations, weights, checkpoint folders, error measures."""
import json
import os

import numpy as np

from oracle import mixed_stack


def attention(heads=4, kv_heads=2, dim=16, vdim=24, rot=8, base=500.0, chunk=13, scale=None, kv_from=None, ff=40):
    mixer = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, rot=dict(dims=rot, base=base), mask=dict(size=chunk),
                 scale=dim ** -0.5 if scale is None else scale)
    if kv_from is not None:
        mixer["kv_from"] = kv_from
    return dict(type="attention", mixer=mixer, mlp=dict(kind="dense", ff=ff) if ff else None)


def mingru(width=56, ff=40):
    return dict(type="mingru", mixer=dict(width=width), mlp=dict(kind="dense", ff=ff) if ff else None)


def latent(heads=3, dim=10, rot_dim=6, vdim=7, q_rank=18, kv_rank=20, rot=None, base=300.0, window=11, scale=None, experts=5, top=2, ff=24,
           limit=0.8, shared=20, shared_limit=1.3):
    """Latent attention beside experts (experts=0: no feed-forward; shared=0: no shared expert)."""
    mixer = dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, q_rank=q_rank, kv_rank=kv_rank, mask=dict(size=window),
                 rot=dict(dims=rot_dim if rot is None else rot, base=base), scale=(dim + rot_dim) ** -0.5 if scale is None else scale)
    mlp = dict(kind="moe", router=dict(experts=experts, top=top), expert=dict(ff=ff, limit=limit))
    if shared:
        mlp["shared"] = dict(ff=shared, limit=shared_limit)
    return dict(type="latent_attention", mixer=mixer, mlp=mlp if experts else None)


def parallel_config(layers, width=44, vocab=93, eps=1e-5, embedding_scale=3.0, logit_scale=0.7):
    return dict(architecture="Kavuvik", width=width, vocab=vocab, norm=dict(eps=eps), layers=list(layers),
                embedding=dict(scale=embedding_scale), logit_scale=logit_scale)


def config(layers, width=48, vocab=97, eps=1e-5):
    return dict(architecture="Retorax", width=width, vocab=vocab, norm=dict(eps=eps), layers=list(layers))


def bf16(a):
    """Nearest 16-bit value, as its bits."""
    bits = np.ascontiguousarray(a, np.float32).view(np.uint32).astype(np.uint64)
    return ((bits + 0x7FFF + ((bits >> 16) & 1)) >> 16).astype(np.uint16)


def value(bits):
    return (np.asarray(bits, np.uint16).astype(np.uint32) << 16).view(np.float32)


def weights(cfg, seed=0, **changes):
    """Random 16-bit tensors by name; `changes`: name (dots as __) -> array put in place of the random one."""
    from nerva_amd import stacks
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in stacks.READERS[cfg["architecture"]](cfg).manifest():
        if name == "embed":
            a = rng.normal(0, 1.0, shape)
        elif name.endswith(".act"):
            a = rng.normal(0, 0.7, shape)
        elif name.endswith(".sink"):
            a = rng.normal(1.0, 1.0, shape)
        elif name.endswith(".talk"):
            a = np.eye(shape[0]) + rng.normal(0, 0.4, shape)
        elif name.endswith(".b"):
            a = rng.normal(0, 0.3, shape)
        elif len(shape) == 1:
            a = rng.normal(1.0, 0.3, shape)
        else:
            gain = 2.0 if name.endswith((".q", ".k", ".uq", ".uk")) else 1.0
            a = rng.normal(0, gain / np.sqrt(shape[1]), shape)
        out[name] = bf16(a)
    for key, a in changes.items():
        name = key.replace("__", ".")
        assert out[name].shape == np.shape(a), name
        out[name] = bf16(a)
    return out


FEATURES = 8


def clear_routes(cfg, tensors, seed=0):
    """The same model with routing that rounding cannot turn: the first FEATURES columns of the residual are a token's own
    and no layer writes them, and every router tells the tokens' features apart by a wide margin."""
    rng = np.random.default_rng(seed)
    out = dict(tensors)
    signs = rng.choice([-2.0, 2.0], (cfg["vocab"], FEATURES))
    embed = value(out["embed"]).copy()
    embed[:, :FEATURES] = signs
    out["embed"] = bf16(embed)
    for i, layer in enumerate(cfg["layers"]):
        if layer["mlp"] is None:
            continue
        name = "l%d." % i
        for key in list(out):
            if key.startswith(name) and key.endswith((".o", ".down")):
                a = value(out[key]).copy()
                a[:FEATURES] = 0.0
                out[key] = bf16(a)
        norm = value(out[name + "norm2"]).copy()
        norm[:FEATURES] = 1.0
        out[name + "norm2"] = bf16(norm)
        experts, top = layer["mlp"]["router"]["experts"], layer["mlp"]["router"]["top"]
        best, gap = None, -1.0
        for _ in range(400 if top < experts else 1):
            r = rng.normal(0, 0.5, (experts, FEATURES))
            z = np.sort(signs @ r.T, -1)
            g = (z[:, experts - top] - z[:, experts - top - 1]).min() if top < experts else 1.0
            if g > gap:
                best, gap = r, g
        assert gap > 0.02
        router = rng.normal(0, 0.0005, (experts, cfg["width"]))
        router[:, :FEATURES] = best
        out[name + "mlp.router"] = bf16(router)
    return out


def oracle_model(cfg, tensors):
    return mixed_stack.Model(cfg, {k: value(v) for k, v in tensors.items()})


def write_folder(path, cfg, tensors):
    """config.json and model.safetensors, the tensors in another order than the arena's."""
    from checkpoint_files import write_safetensors
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    write_safetensors(os.path.join(path, "model.safetensors"), sorted(tensors.items(), reverse=True), "BF16")


def session(cfg, tensors, max_context, precision=0):
    from nerva_amd import DecodeSession, WeightPlan, stacks
    stack = stacks.READERS[cfg["architecture"]](cfg)
    return DecodeSession.create_stack(stack, WeightPlan.from_weights(stacks.StackWeights(stack, tensors)), max_context, precision)


def errors(got, want):
    """Per row: root mean square of the difference with its mean taken off, over that of the wanted logits."""
    d = np.asarray(got, np.float64) - want
    d -= d.mean(-1, keepdims=True)
    w = want - want.mean(-1, keepdims=True)
    return np.sqrt((d * d).mean(-1)) / np.sqrt((w * w).mean())


def feed(s, tokens, sizes):
    """Logits of all tokens, fed in portions of the given sizes (the last one repeats)."""
    out, at, i = [], 0, 0
    while at < len(tokens):
        n = min(sizes[min(i, len(sizes) - 1)], len(tokens) - at)
        rc, res, logits, _ = s.extend(tokens[at:at + n], range(n))
        assert rc == 0, "extend failed: hip_error=%d" % res.hip_error
        out.append(logits)
        at, i = at + n, i + 1
    return np.concatenate(out)
