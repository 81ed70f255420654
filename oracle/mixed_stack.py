"""Plain statement of a mixed layer stack (test infrastructure; the product never imports it).

One function per mechanism, numpy in double precision unless told otherwise, a loop over tokens wherever the
product has a kernel that does many at once. A model is a configuration (the dictionary of its config.json) and a
dictionary of named float arrays; `forward` returns the logits of every position and the residual stream after
every layer. Nothing here is fast, and nothing is shared with nerva_amd.
"""
import numpy as np


def sigmoid(z):
    return 0.5 * (1.0 + np.tanh(0.5 * z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def layer_norm(x, weight, bias, eps):
    """Centre, divide by the root of (mean squared deviation + eps), scale, shift - row by row."""
    centred = x - x.mean(-1, keepdims=True)
    spread = (centred * centred).mean(-1, keepdims=True)
    return centred / np.sqrt(spread + eps) * weight + bias


def xielu(z, p, q):
    """Above zero: a quadratic with curvature softplus(p) on the line z / 2. At and below: the exponential's
    remainder after its first two terms, scaled by softplus(q) + 1/2, on the same line."""
    below = np.minimum(z, 0.0)
    return np.where(z > 0.0, softplus(p) * z * z, (softplus(q) + 0.5) * (np.expm1(below) - below)) + 0.5 * z


def rotate(heads, position, dims, base):
    """heads [n, dim] turned pair by pair; element i goes with element i + dims/2, elements from `dims` on stay."""
    out, half = np.array(heads), dims // 2
    if half:
        angle = position * base ** (-2.0 * np.arange(half) / dims)
        u, v = heads[:, :half], heads[:, half:dims]
        out[:, :half] = u * np.cos(angle) - v * np.sin(angle)
        out[:, half:dims] = v * np.cos(angle) + u * np.sin(angle)
    return out


def first_visible(position, chunk):
    """Oldest position a query may look at: the start of its own chunk (chunk 0: no chunks)."""
    return position // chunk * chunk if chunk else 0


def mix_heads(scores, talk):
    """scores [heads, keys] -> every head's scores as a combination of all heads' scores."""
    return talk @ scores


def softmax_with_sink(scores, sink):
    """Rows of weights whose denominator also counts exp(sink) for a key that has no value."""
    top = np.maximum(scores.max(-1), sink)
    e = np.exp(scores - top[:, None])
    return e / (e.sum(-1) + np.exp(sink - top))[:, None]


def attend(q, keys, values, scale, talk, sink):
    """One token's heads q [H, d] over keys [n, G, d] and values [n, G, dv] it may see -> [H, dv]."""
    H, G = q.shape[0], keys.shape[1]
    scores = np.stack([keys[:, h // (H // G)] @ q[h] for h in range(H)]) * scale
    weights = softmax_with_sink(mix_heads(scores, talk), sink)
    return np.stack([weights[h] @ values[:, h // (H // G)] for h in range(H)])


def attention_mixer(h, mixer, w, cache, first):
    """Rows h [n, width] at positions first.. ; `cache` is {"k": [...], "v": [...]}: rows of this layer, appended to
    here, or of the layer whose keys and values it uses, which hold these positions already."""
    H, G, d, dv = mixer["heads"], mixer["kv_heads"], mixer["dim"], mixer["vdim"]
    rot = mixer["rot"]
    out = []
    for t, row in enumerate(h):
        p = first + t
        q = rotate((w["q"] @ row).reshape(H, d), p, rot["dims"], rot["base"])
        if "k" in w:
            cache["k"].append(rotate((w["k"] @ row).reshape(G, d), p, rot["dims"], rot["base"]))
            cache["v"].append((w["v"] @ row).reshape(G, dv))
        lo = first_visible(p, mixer["mask"]["size"])
        o = attend(q, np.stack(cache["k"][lo:p + 1]), np.stack(cache["v"][lo:p + 1]), mixer["scale"], w["talk"], w["sink"])
        out.append(w["o"] @ (o.reshape(-1) * sigmoid(w["g"] @ row)))
    return np.stack(out)


def mingru_mixer(h, w, state):
    """The gate z and the candidate come from the current token alone; returns the rows and the last state."""
    out = []
    for row in h:
        z = sigmoid(w["z"] @ row + w["z.b"])
        u = w["x"] @ row + w["x.b"]
        candidate = np.where(u >= 0.0, u + 0.5, sigmoid(u))
        state = state + z * (candidate - state)
        out.append(w["o"] @ (state * silu(w["g"] @ row)))
    return np.stack(out), state


def feed_forward(h, w):
    p, q = w["act"]
    return xielu(h @ w["up"].T, p, q) @ w["down"].T


class Model:
    """A configuration, its weights, and the cache and state of one sequence."""

    def __init__(self, config, weights, dtype=np.float64):
        self.config = config
        self.w = {k: np.asarray(v, dtype) for k, v in weights.items()}
        self.dtype = dtype
        self.reset()

    def reset(self):
        self.position = 0
        self.cache = [{"k": [], "v": []} for _ in self.config["layers"]]
        self.state = [np.zeros(l["mixer"].get("width", 0), self.dtype) for l in self.config["layers"]]

    def part(self, prefix):
        return {k[len(prefix):]: v for k, v in self.w.items() if k.startswith(prefix)}

    def norm(self, x, name):
        return layer_norm(x, self.w[name], self.w[name + ".b"], self.config["norm"]["eps"])

    def run(self, tokens):
        """The next tokens of the sequence -> (logits [n, vocab], residual after each layer [layers, n, width])."""
        x = self.w["embed"][np.asarray(tokens, int)]
        trail = []
        for i, layer in enumerate(self.config["layers"]):
            name = "l%d." % i
            mixer, w = layer["mixer"], self.part(name + "mix.")
            h = self.norm(x, name + "norm1")
            if layer["type"] == "attention":
                y = attention_mixer(h, mixer, w, self.cache[mixer.get("kv_from", i)], self.position)
            else:
                y, self.state[i] = mingru_mixer(h, w, self.state[i])
            x = x + self.norm(y, name + "norm1b")
            if layer["mlp"] is not None:
                x = x + self.norm(feed_forward(self.norm(x, name + "norm2"), self.part(name + "mlp.")), name + "norm2b")
            trail.append(x)
        self.position += len(tokens)
        return self.norm(x, "final.norm") @ self.w["embed"].T, np.stack(trail)
