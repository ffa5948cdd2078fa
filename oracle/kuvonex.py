"""Plain float64 NumPy implementation of the Kuvonex decoder: one function per mechanism, a loop wherever a loop is
the shortest way to say it.  Test infrastructure only: it shares no code with the product path and reads its weights
from a dict of float arrays under the checkpoint's tensor names.

Conventions: tokens are rows, a linear weight is [out, in] and is applied as x @ W.T.
"""

import numpy as np


def rms_norm(x, w, eps):
    """w * x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def rotate_interleaved(v, positions, base):
    """Rotate neighbouring pairs (2i, 2i + 1) of the last axis of v [T, ..., D] by the angle position * base^(-2i / D)."""
    D = v.shape[-1]
    out = np.array(v, dtype=np.float64)
    for t, p in enumerate(positions):
        for i in range(D // 2):
            a = p * float(base) ** (-2.0 * i / D)
            x, y = v[t, ..., 2 * i], v[t, ..., 2 * i + 1]
            out[t, ..., 2 * i] = x * np.cos(a) - y * np.sin(a)
            out[t, ..., 2 * i + 1] = y * np.cos(a) + x * np.sin(a)
    return out


def latent_rows(h, w_dkv, norm_w, kv_rank, eps, positions, base):
    """What a layer caches per token: the normed latent [T, kv_rank] and the shared rotated key part [T, rot_dim]."""
    z = h @ w_dkv.T
    return rms_norm(z[:, :kv_rank], norm_w, eps), rotate_interleaved(z[:, kv_rank:], positions, base)


def sink_softmax(scores, sink):
    """Softmax of a score row whose denominator also counts exp(sink) once."""
    m = max(scores.max(), sink)
    e = np.exp(scores - m)
    return e / (e.sum() + np.exp(sink - m))


def latent_attention(q, c, k_rot, w_uk, w_uv, sinks, heads, dim, vdim, rot_dim, scale, positions, base):
    """Causal attention of the query rows q [T, heads * (dim + rot_dim)] (not yet rotated) at `positions` over the
    cached rows 0 .. max(positions): [T, heads * vdim]."""
    T = q.shape[0]
    q = q.reshape(T, heads, dim + rot_dim)
    qu, qr = q[..., :dim], rotate_interleaved(q[..., dim:], positions, base)
    k = (c @ w_uk.T).reshape(-1, heads, dim)
    v = (c @ w_uv.T).reshape(-1, heads, vdim)
    out = np.zeros((T, heads, vdim))
    for t, p in enumerate(positions):
        for h in range(heads):
            s = (k[:p + 1, h] @ qu[t, h] + k_rot[:p + 1] @ qr[t, h]) * scale
            out[t, h] = sink_softmax(s, sinks[h]) @ v[:p + 1, h]
    return out.reshape(T, heads * vdim)


def route(h, w_router, correction, top, groups, keep):
    """Grouped sigmoid router for one token h [width]: (expert ids, weights), ids in descending order of choice."""
    s = sigmoid(h @ w_router.T)
    choice = s + correction
    E = choice.shape[0]
    size = E // groups
    group_score = [np.sort(choice[g * size:(g + 1) * size])[::-1][:2].sum() for g in range(groups)]
    kept = sorted(range(groups), key=lambda g: (-group_score[g], g))[:keep]
    allowed = [e for e in range(E) if e // size in kept]
    ids = sorted(allowed, key=lambda e: (-choice[e], e))[:top]
    return ids, s[ids]


def expert(h, w_gate, w_up, w_down):
    return (silu(h @ w_gate.T) * (h @ w_up.T)) @ w_down.T


def mixture(h, w, prefix, mlp):
    r = mlp["router"]
    g = r.get("groups") or {"count": 1, "keep": 1}
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        ids, wt = route(h[t], w[prefix + "router"], w[prefix + "correction"], r["top"], g["count"], g["keep"])
        for e, a in zip(ids, wt):
            out[t] += a * expert(h[t], *(w[f"{prefix}e{e}.{n}"] for n in ("gate", "up", "down")))
    return out


class Model:
    """Runs portions of one sequence; keeps (latent, rotated key) rows per layer that has a cache."""

    def __init__(self, config, weights):
        self.c = config
        self.w = {k: np.asarray(v, dtype=np.float64) for k, v in weights.items()}
        self.reset()

    def reset(self):
        self.cache = {}
        self.pos = 0

    def mixer(self, i, h, positions):
        m, w, p = self.c["layers"][i]["mixer"], self.w, f"l{i}.mix."
        base = m["rot"]["base"]
        src = m.get("kv_from")
        if src is None:
            src = i
            new = latent_rows(h, w[p + "dkv"], w[p + "dkv.norm"], m["kv_rank"], self.c["norm"]["eps"], positions, base)
            old = self.cache.get(i)
            self.cache[i] = new if old is None else tuple(np.concatenate([a, b]) for a, b in zip(old, new))
        c, k_rot = self.cache[src]
        o = latent_attention(h @ w[p + "q"].T, c, k_rot, w[p + "uk"], w[p + "uv"], w[p + "sink"], m["heads"], m["dim"], m["vdim"],
                             m["rot_dim"], m["scale"], positions, base)
        return (o * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T

    def step(self, tokens):
        """Logits of every token of the portion [T, vocab]; the residual after every layer is left in self.layers."""
        w, eps = self.w, self.c["norm"]["eps"]
        positions = range(self.pos, self.pos + len(tokens))
        x = w["embed"][np.asarray(tokens)] * self.c["embedding"]["scale"]
        self.layers = []
        for i, layer in enumerate(self.c["layers"]):
            x = x + rms_norm(self.mixer(i, x, positions), w[f"l{i}.norm1"], eps)
            if layer.get("mlp") is not None:
                x = x + rms_norm(mixture(x, w, f"l{i}.mlp.", layer["mlp"]), w[f"l{i}.norm2"], eps)
            self.layers.append(x)
        self.pos += len(tokens)
        return rms_norm(x, w["final.norm"], eps) @ w["head"].T
