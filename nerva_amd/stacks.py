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


class StackConfig:
    """hidden, vocab, eps and the layers: (mixer, feed-forward width or 0)."""

    def __init__(self, hidden, vocab, eps, layers):
        self.hidden, self.vocab, self.eps, self.layers = hidden, vocab, eps, list(layers)

    def c_layers(self):
        out = (abi.NervaHipStackLayer * len(self.layers))()
        for c, (mixer, ff) in zip(out, self.layers):
            c.mixer, c.ff, c.kv_layer = mixer.kind, ff, OWN_KEYS
            mixer.fill(c)
        return out

    def manifest(self):
        """(name, shape) of every tensor in the order of the weight arena."""
        h = self.hidden
        out = [("embed", [self.vocab, h])]
        for i, (mixer, ff) in enumerate(self.layers):
            name = "l%d." % i
            for norm in ("norm1", "norm1b") + (("norm2", "norm2b") if ff else ()):
                out += [(name + norm, [h]), (name + norm + ".b", [h])]
            out += [(name + "mix." + t, shape) for t, shape in mixer.tensors(h)]
            if ff:
                out += [(name + "mlp.up", [ff, h]), (name + "mlp.down", [h, ff]), (name + "mlp.act", [2])]
        return out + [("final.norm", [h]), ("final.norm.b", [h])]


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
        mlp, ff = entry.get("mlp"), 0
        if mlp is not None:
            if not isinstance(mlp, dict) or mlp.get("kind") != "dense":
                raise CheckpointError("config.json: %s has a feed-forward of kind %r" % (what, mlp))
            ff = _number(mlp.get("ff"), what + " ff")
        layers.append((mixer, ff))
    return StackConfig(hidden, vocab, eps, layers)


READERS = {"Retorax": read_retorax}
