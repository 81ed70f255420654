"""Mixed layer stacks: models whose layers are described one by one (include/nerva_hip_api.h, NervaHipStackLayer).

`READERS` is the registry: the `architecture` a config.json names -> the function that reads it into a StackConfig. A
StackConfig knows the session's layer descriptions and, in the order of the weight arena, the names and shapes of its
tensors; checkpoint.py turns that into file-backed descriptors like any other model's.
"""
import ctypes as C
import math

import numpy as np

from . import abi

PRECISION_16, PRECISION_32 = abi.NERVA_HIP_PRECISION_16, abi.NERVA_HIP_PRECISION_32
OWN_KEYS = 0xFFFFFFFF


class CheckpointError(ValueError):
    pass


class Attention:
    """Grouped-query attention with mixed heads, sinks, an output gate and chunked visibility."""
    kind = abi.NERVA_HIP_MIXER_ATTENTION

    def __init__(self, heads, kv_heads, key_dim, value_dim, rotary_dims, rotary_base, score_scale, chunk_tokens,
                 kv_layer=None):
        self.heads, self.kv_heads, self.key_dim, self.value_dim = heads, kv_heads, key_dim, value_dim
        self.rotary_dims, self.rotary_base, self.score_scale = rotary_dims, rotary_base, score_scale
        self.chunk_tokens, self.kv_layer = chunk_tokens, kv_layer

    def tensors(self, hidden):
        out = [("q", [self.heads * self.key_dim, hidden])]
        if self.kv_layer is None:
            out += [("k", [self.kv_heads * self.key_dim, hidden]), ("v", [self.kv_heads * self.value_dim, hidden])]
        return out + [("g", [self.heads * self.value_dim, hidden]), ("talk", [self.heads, self.heads]),
                      ("sink", [self.heads]), ("o", [hidden, self.heads * self.value_dim])]

    def fill(self, layer):
        layer.heads, layer.kv_heads, layer.key_dim, layer.value_dim = self.heads, self.kv_heads, self.key_dim, self.value_dim
        layer.rotary_dims, layer.rotary_base, layer.score_scale = self.rotary_dims, self.rotary_base, self.score_scale
        layer.chunk_tokens = self.chunk_tokens
        layer.kv_layer = OWN_KEYS if self.kv_layer is None else self.kv_layer


class MinGru:
    """Gated recurrence of `width` channels whose gates read the current token only."""
    kind = abi.NERVA_HIP_MIXER_MINGRU

    def __init__(self, width):
        self.width = width

    def tensors(self, hidden):
        w = self.width
        return [("z", [w, hidden]), ("x", [w, hidden]), ("g", [w, hidden]), ("z.b", [w]), ("x.b", [w]), ("o", [hidden, w])]

    def fill(self, layer):
        layer.width = self.width


class LatentAttention:
    """Attention whose keys and values are projections of one normalised latent per token, with a rotated key part shared
    by the heads, an output gate and a sliding window (0: none)."""
    kind = abi.NERVA_HIP_MIXER_LATENT

    def __init__(self, heads, key_dim, rotary_key_dim, value_dim, q_rank, kv_rank, rotary_dims, rotary_base, score_scale,
                 window_tokens):
        self.heads, self.key_dim, self.rotary_key_dim, self.value_dim = heads, key_dim, rotary_key_dim, value_dim
        self.q_rank, self.kv_rank, self.window_tokens = q_rank, kv_rank, window_tokens
        self.rotary_dims, self.rotary_base, self.score_scale = rotary_dims, rotary_base, score_scale

    def tensors(self, hidden):
        values = self.heads * self.value_dim
        return [("dq", [self.q_rank, hidden]), ("dkv", [self.kv_rank + self.rotary_key_dim, hidden]), ("g", [values, hidden]),
                ("dq.norm", [self.q_rank]), ("dkv.norm", [self.kv_rank]),
                ("uq", [self.heads * (self.key_dim + self.rotary_key_dim), self.q_rank]),
                ("uk", [self.heads * self.key_dim, self.kv_rank]), ("uv", [values, self.kv_rank]), ("o", [hidden, values])]

    def fill(self, layer):
        layer.heads, layer.key_dim, layer.value_dim, layer.rotary_key_dim = self.heads, self.key_dim, self.value_dim, self.rotary_key_dim
        layer.q_rank, layer.kv_rank, layer.window_tokens = self.q_rank, self.kv_rank, self.window_tokens
        layer.rotary_dims, layer.rotary_base, layer.score_scale = self.rotary_dims, self.rotary_base, self.score_scale


class XieluFeedForward:
    """Dense: up, xIELU, down."""

    def __init__(self, ff):
        self.ff = ff

    def tensors(self, hidden):
        return [("up", [self.ff, hidden]), ("down", [hidden, self.ff]), ("act", [2])]

    def fill(self, layer):
        layer.ff = self.ff


class ExpertFeedForward:
    """Routed experts with bounded gates; an expert that takes every token besides, where shared_ff != 0."""

    def __init__(self, experts, top, ff, limit, shared_ff=0, shared_limit=0.0):
        self.experts, self.top, self.ff, self.limit = experts, top, ff, limit
        self.shared_ff, self.shared_limit = shared_ff, shared_limit

    def tensors(self, hidden):
        out = [("router", [self.experts, hidden])]
        names = [("e%d" % e, self.ff) for e in range(self.experts)] + ([("shared", self.shared_ff)] if self.shared_ff else [])
        for name, ff in names:
            out += [(name + ".gate", [ff, hidden]), (name + ".up", [ff, hidden]), (name + ".down", [hidden, ff])]
        return out

    def fill(self, layer):
        layer.experts, layer.experts_per_token, layer.expert_ff, layer.expert_limit = self.experts, self.top, self.ff, self.limit
        layer.shared_ff, layer.shared_limit = self.shared_ff, self.shared_limit


SANDWICH, PARALLEL = abi.NERVA_HIP_STACK_SANDWICH, abi.NERVA_HIP_STACK_PARALLEL


class StackConfig:
    """hidden, vocab, eps and the layers: (mixer, feed-forward or None). `arrangement`: one sublayer after the other, each
    between two layer norms, the embedding as the head (SANDWICH); or both on the same row, each behind an RMS norm, and a
    head of its own (PARALLEL)."""

    def __init__(self, hidden, vocab, eps, layers, arrangement=SANDWICH, embedding_scale=1.0, logit_scale=1.0):
        self.hidden, self.vocab, self.eps, self.layers = hidden, vocab, eps, list(layers)
        self.arrangement, self.embedding_scale, self.logit_scale = arrangement, embedding_scale, logit_scale

    def c_layers(self):
        out = (abi.NervaHipStackLayer * len(self.layers))()
        for c, (mixer, ff) in zip(out, self.layers):
            c.mixer, c.kv_layer = mixer.kind, OWN_KEYS
            mixer.fill(c)
            if ff is not None:
                ff.fill(c)
        return out

    def _norm(self, name):
        return [(name, [self.hidden])] + ([(name + ".b", [self.hidden])] if self.arrangement == SANDWICH else [])

    def manifest(self):
        """(name, shape) of every tensor in the order of the weight arena."""
        h = self.hidden
        out = [("embed", [self.vocab, h])]
        for i, (mixer, ff) in enumerate(self.layers):
            name = "l%d." % i
            norms = ("norm1", "norm1b", "norm2", "norm2b") if self.arrangement == SANDWICH else ("norm1", "norm2")
            for norm in norms if ff is not None else norms[:len(norms) // 2]:
                out += self._norm(name + norm)
            out += [(name + "mix." + t, shape) for t, shape in mixer.tensors(h)]
            if ff is not None:
                out += [(name + "mlp." + t, shape) for t, shape in ff.tensors(h)]
        return out + self._norm("final.norm") + ([("head", [self.vocab, h])] if self.arrangement == PARALLEL else [])


class StackWeights:
    """Host weights (16-bit arrays by tensor name) of a StackConfig, for sessions that are not read from files."""

    def __init__(self, config, tensors):
        self.config = config
        self.tensors = {}
        for name, shape in config.manifest():
            array = np.ascontiguousarray(tensors[name], np.uint16)
            if list(array.shape) != shape:
                raise CheckpointError("tensor %s shape %r does not match expected %r" % (name, list(array.shape), shape))
            self.tensors[name] = array

    def arena_tensors(self):
        return [self.tensors[name] for name, _ in self.config.manifest()]


def _number(value, what, integer=True, least=1):
    ok = isinstance(value, (int,) if integer else (int, float)) and not isinstance(value, bool) and math.isfinite(value)
    if not ok or value < least:
        raise CheckpointError("config.json: %s missing or out of range (%r)" % (what, value))
    return int(value) if integer else float(value)


def _part(parent, key, what):
    value = parent.get(key)
    if not isinstance(value, dict):
        raise CheckpointError("config.json: %s has no %s" % (what, key))
    return value


def read_retorax(config):
    """Retorax: layers of chunked attention with mixed heads or of minGRU, each with a dense xIELU feed-forward or none."""
    hidden, vocab = _number(config.get("width"), "width"), _number(config.get("vocab"), "vocab")
    eps = _number(_part(config, "norm", "the model").get("eps"), "norm.eps", integer=False, least=0.0)
    entries = config.get("layers")
    if not isinstance(entries, list) or not entries:
        raise CheckpointError("config.json: no layers")
    layers = []
    for i, entry in enumerate(entries):
        what = "layer %d" % i
        kind, m = entry.get("type"), _part(entry, "mixer", what)
        if kind == "attention":
            rot, mask = _part(m, "rot", what), _part(m, "mask", what)
            mixer = Attention(_number(m.get("heads"), what + " heads"), _number(m.get("kv_heads"), what + " kv_heads"),
                              _number(m.get("dim"), what + " dim"), _number(m.get("vdim"), what + " vdim"),
                              _number(rot.get("dims"), what + " rot.dims", least=0),
                              _number(rot.get("base"), what + " rot.base", integer=False, least=0.0),
                              _number(m.get("scale"), what + " scale", integer=False, least=-math.inf),
                              _number(mask.get("size"), what + " mask.size"), m.get("kv_from"))
            if mixer.heads % mixer.kv_heads != 0 or mixer.rotary_dims % 2 != 0 or mixer.rotary_dims > mixer.key_dim:
                raise CheckpointError("config.json: %s has sizes that do not go together" % what)
            if mixer.kv_layer is not None:
                source = layers[mixer.kv_layer][0] if isinstance(mixer.kv_layer, int) and 0 <= mixer.kv_layer < i else None
                if not isinstance(source, Attention) or source.kv_layer is not None or \
                        (source.kv_heads, source.key_dim, source.value_dim) != (mixer.kv_heads, mixer.key_dim, mixer.value_dim):
                    raise CheckpointError("config.json: %s takes keys from layer %r, which has none for it" % (what, mixer.kv_layer))
        elif kind == "mingru":
            mixer = MinGru(_number(m.get("width"), what + " width"))
        else:
            raise CheckpointError("config.json: %s has type %r" % (what, kind))
        mlp, ff = entry.get("mlp"), None
        if mlp is not None:
            if not isinstance(mlp, dict) or mlp.get("kind") != "dense":
                raise CheckpointError("config.json: %s has a feed-forward of kind %r" % (what, mlp))
            ff = XieluFeedForward(_number(mlp.get("ff"), what + " ff"))
        layers.append((mixer, ff))
    return StackConfig(hidden, vocab, eps, layers)


def read_kavuvik(config):
    """Kavuvik: layers of latent attention through sliding windows beside routed experts (or none), both on the same row."""
    hidden, vocab = _number(config.get("width"), "width"), _number(config.get("vocab"), "vocab")
    eps = _number(_part(config, "norm", "the model").get("eps"), "norm.eps", integer=False, least=0.0)
    embedding_scale = _number(_part(config, "embedding", "the model").get("scale"), "embedding.scale", integer=False, least=-math.inf)
    logit_scale = _number(config.get("logit_scale"), "logit_scale", integer=False, least=-math.inf)
    entries = config.get("layers")
    if not isinstance(entries, list) or not entries:
        raise CheckpointError("config.json: no layers")
    layers = []
    for i, entry in enumerate(entries):
        what = "layer %d" % i
        if entry.get("type") != "latent_attention":
            raise CheckpointError("config.json: %s has type %r" % (what, entry.get("type")))
        m = _part(entry, "mixer", what)
        rot = _part(m, "rot", what)
        window = 0 if m.get("mask") is None else _number(_part(m, "mask", what).get("size"), what + " mask.size")
        sizes = {k: _number(m.get(k), "%s %s" % (what, k)) for k in ("heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank")}
        mixer = LatentAttention(sizes["heads"], sizes["dim"], sizes["rot_dim"], sizes["vdim"], sizes["q_rank"], sizes["kv_rank"],
                                _number(rot.get("dims"), what + " rot.dims", least=0),
                                _number(rot.get("base"), what + " rot.base", integer=False, least=0.0),
                                _number(m.get("scale"), what + " scale", integer=False, least=-math.inf), window)
        if mixer.rotary_dims % 2 != 0 or mixer.rotary_dims > mixer.rotary_key_dim:
            raise CheckpointError("config.json: %s has sizes that do not go together" % what)
        mlp, ff = entry.get("mlp"), None
        if mlp is not None:
            if not isinstance(mlp, dict) or mlp.get("kind") != "moe":
                raise CheckpointError("config.json: %s has a feed-forward of kind %r" % (what, mlp))
            router, expert = _part(mlp, "router", what), _part(mlp, "expert", what)
            ff = ExpertFeedForward(_number(router.get("experts"), what + " experts"), _number(router.get("top"), what + " top"),
                                   _number(expert.get("ff"), what + " expert ff"),
                                   _number(expert.get("limit"), what + " expert limit", integer=False, least=0.0))
            if mlp.get("shared") is not None:
                shared = _part(mlp, "shared", what)
                ff.shared_ff = _number(shared.get("ff"), what + " shared ff")
                ff.shared_limit = _number(shared.get("limit"), what + " shared limit", integer=False, least=0.0)
            if ff.top > ff.experts:
                raise CheckpointError("config.json: %s takes %d of %d experts" % (what, ff.top, ff.experts))
        layers.append((mixer, ff))
    return StackConfig(hidden, vocab, eps, layers, PARALLEL, embedding_scale, logit_scale)


READERS = {"Kavuvik": read_kavuvik, "Retorax": read_retorax}
