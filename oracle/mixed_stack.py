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


def rms_norm(x, weight, eps):
    """Divide by the root of (mean square + eps), scale - row by row."""
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps) * weight


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


def window_start(position, window):
    """Oldest position a query may look at through a window of that many tokens, itself included (0: no window)."""
    return max(0, position - window + 1) if window else 0


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


def softmax(scores):
    e = np.exp(scores - scores.max(-1, keepdims=True))
    return e / e.sum(-1, keepdims=True)


def latent_attention_mixer(h, mixer, w, cache, first, eps):
    """Keys and values are projections of one normalised latent per token, expanded here for every query anew; one
    rotated key part serves all heads. `cache` is {"c": [...], "r": [...]}: latents and rotated parts, appended to."""
    H, d, rd, dv, rank = mixer["heads"], mixer["dim"], mixer["rot_dim"], mixer["vdim"], mixer["kv_rank"]
    rot, window = mixer["rot"], (mixer.get("mask") or {}).get("size", 0)
    out = []
    for t, row in enumerate(h):
        p = first + t
        q = (w["uq"] @ rms_norm(w["dq"] @ row, w["dq.norm"], eps)).reshape(H, d + rd)
        q_rotated = rotate(q[:, d:], p, rot["dims"], rot["base"])
        down = w["dkv"] @ row
        cache["c"].append(rms_norm(down[:rank], w["dkv.norm"], eps))
        cache["r"].append(rotate(down[None, rank:], p, rot["dims"], rot["base"])[0])
        lo = window_start(p, window)
        latents, parts = np.stack(cache["c"][lo:p + 1]), np.stack(cache["r"][lo:p + 1])
        keys = (latents @ w["uk"].T).reshape(-1, H, d)
        values = (latents @ w["uv"].T).reshape(-1, H, dv)
        scores = np.stack([keys[:, i] @ q[i, :d] + parts @ q_rotated[i] for i in range(H)]) * mixer["scale"]
        weights = softmax(scores)
        o = np.stack([weights[i] @ values[:, i] for i in range(H)])
        out.append(w["o"] @ (o.reshape(-1) * sigmoid(w["g"] @ row)))
    return np.stack(out)


def clamped_glu(g, u, limit):
    """The gate bounded above, the linear part on both sides and moved up by one."""
    g, u = np.minimum(g, limit), np.clip(u, -limit, limit)
    return g * sigmoid(1.702 * g) * (u + 1.0)


def expert(row, w, name, limit):
    return w[name + ".down"] @ clamped_glu(w[name + ".gate"] @ row, w[name + ".up"] @ row, limit)


def choose_experts(z, top):
    """Indices of the `top` largest scores and the weights of their outputs."""
    s = sigmoid(z)
    chosen = np.argsort(-s, kind="stable")[:top]
    return chosen, s[chosen] / (s[chosen].sum() + 1e-20)


def expert_feed_forward(h, mlp, w):
    out = []
    for row in h:
        chosen, weights = choose_experts(w["router"] @ row, mlp["router"]["top"])
        y = sum(a * expert(row, w, "e%d" % e, mlp["expert"]["limit"]) for e, a in zip(chosen, weights))
        if mlp.get("shared"):
            y = y + expert(row, w, "shared", mlp["shared"]["limit"])
        out.append(y)
    return np.stack(out)


class Model:
    """A configuration, its weights, and the cache and state of one sequence."""

    def __init__(self, config, weights, dtype=np.float64):
        self.config = config
        self.w = {k: np.asarray(v, dtype) for k, v in weights.items()}
        self.dtype = dtype
        self.reset()

    def reset(self):
        self.position = 0
        self.cache = [{"k": [], "v": [], "c": [], "r": []} for _ in self.config["layers"]]
        self.state = [np.zeros(l["mixer"].get("width", 0), self.dtype) for l in self.config["layers"]]

    def part(self, prefix):
        return {k[len(prefix):]: v for k, v in self.w.items() if k.startswith(prefix)}

    def norm(self, x, name):
        return layer_norm(x, self.w[name], self.w[name + ".b"], self.config["norm"]["eps"])

    def mix(self, i, h):
        layer, w = self.config["layers"][i], self.part("l%d.mix." % i)
        mixer = layer["mixer"]
        if layer["type"] == "latent_attention":
            return latent_attention_mixer(h, mixer, w, self.cache[i], self.position, self.config["norm"]["eps"])
        if layer["type"] == "attention":
            return attention_mixer(h, mixer, w, self.cache[mixer.get("kv_from", i)], self.position)
        y, self.state[i] = mingru_mixer(h, w, self.state[i])
        return y

    def run(self, tokens):
        """The next tokens of the sequence -> (logits [n, vocab], residual after each layer [layers, n, width])."""
        run = self.run_parallel if self.config["architecture"] == "Kavuvik" else self.run_sandwich
        out = run(self.w["embed"][np.asarray(tokens, int)])
        self.position += len(tokens)
        return out

    def run_sandwich(self, x):
        """A norm before and after every sublayer; the head is the embedding."""
        trail = []
        for i, layer in enumerate(self.config["layers"]):
            name = "l%d." % i
            x = x + self.norm(self.mix(i, self.norm(x, name + "norm1")), name + "norm1b")
            if layer["mlp"] is not None:
                x = x + self.norm(feed_forward(self.norm(x, name + "norm2"), self.part(name + "mlp.")), name + "norm2b")
            trail.append(x)
        return self.norm(x, "final.norm") @ self.w["embed"].T, np.stack(trail)

    def run_parallel(self, x):
        """Both sublayers read the same row, each through a norm of its own; a head of its own, scaled."""
        x = x * self.config["embedding"]["scale"]
        eps, trail = self.config["norm"]["eps"], []
        for i, layer in enumerate(self.config["layers"]):
            name = "l%d." % i
            y = self.mix(i, rms_norm(x, self.w[name + "norm1"], eps))
            if layer["mlp"] is not None:
                y = y + expert_feed_forward(rms_norm(x, self.w[name + "norm2"], eps), layer["mlp"], self.part(name + "mlp."))
            x = x + y
            trail.append(x)
        return rms_norm(x, self.w["final.norm"], eps) @ self.w["head"].T * self.config["logit_scale"], np.stack(trail)
