"""Plain float64 NumPy implementation of the Sitirax decoder: one function per mechanism, a loop wherever a loop is the
shortest way to say it.  Test infrastructure only: it shares no code with the product path and reads its weights from a
dict of float arrays under the checkpoint's tensor names.

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


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def softplus(z):
    return np.logaddexp(0.0, z)


def softmax(s):
    e = np.exp(s - s.max())
    return e / e.sum()


def window_attention(q, k, v, positions, scale, window):
    """q [T, H, D] at `positions` over k [N, G, D] and v [N, G, V] at positions 0 .. N - 1: the query at position i sees the
    `window` positions up to and with i.  Query head h reads key / value head h // (H / G)."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = np.zeros((T, H, v.shape[2]))
    for t, i in enumerate(positions):
        lo = max(0, i - window + 1)
        for h in range(H):
            g = h // (H // G)
            out[t, h] = softmax(k[lo:i + 1, g] @ q[t, h] * scale) @ v[lo:i + 1, g]
    return out


def lightning(q, k, v, decay, state):
    """q, k [T, H, D], v [T, H, V], one decay per head: S = decay S + k v^T, o = S^T q.  `state` [H, D, V] is brought forward."""
    out = np.zeros(v.shape)
    for t in range(q.shape[0]):
        for h in range(q.shape[1]):
            state[h] = decay[h] * state[h] + np.outer(k[t, h], v[t, h])
            out[t, h] = state[h].T @ q[t, h]
    return out


def short_convolution(x, w, history):
    """x [T, C], one filter of w [C, taps] per channel whose last tap meets the current row; `history` [taps - 1, C] are the
    rows in front.  Returns (result, new history)."""
    taps = w.shape[1]
    rows = np.concatenate([history, x])
    out = np.zeros(x.shape)
    for t in range(x.shape[0]):
        for j in range(taps):
            out[t] += w[:, j] * rows[t + j]
    return out, rows[rows.shape[0] - (taps - 1):]


def unit(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + 1e-6)


def channel_decay(z, a_log, dt_bias):
    """z [T, H, D] -> one factor per head and key channel."""
    return np.exp(-np.exp(a_log)[:, None] * softplus(z + dt_bias.reshape(z.shape[1:])))


def delta_rule(q, k, v, beta, g, state):
    """q, k [T, Hk, D], v [T, H, V], beta [T, H], g [T, H, D]; head h uses q / k head h // (H / Hk).  `state` [H, D, V]."""
    T, H, _ = v.shape
    r = H // q.shape[1]
    out = np.zeros(v.shape)
    for t in range(T):
        for h in range(H):
            s = g[t, h][:, None] * state[h]
            u = beta[t, h] * (v[t, h] - s.T @ k[t, h // r])
            state[h] = s + np.outer(k[t, h // r], u)
            out[t, h] = state[h].T @ q[t, h // r]
    return out


class Model:
    """Runs portions of one sequence; keeps what every layer carries from token to token."""

    def __init__(self, config, weights):
        self.c = config
        self.w = {k: np.asarray(v, dtype=np.float64) for k, v in weights.items()}
        self.reset()

    def reset(self):
        self.state = {}
        self.pos = 0

    def own(self, i):
        """Layer whose tensors layer i uses."""
        while self.c["layers"][i].get("weights_of") is not None:
            i = self.c["layers"][i]["weights_of"]
        return i

    def parallel(self, i, h, positions):
        m, w, p, eps, T = self.c["layers"][i]["mixer"], self.w, f"l{self.own(i)}.mix.", self.c["norm"]["eps"], h.shape[0]
        a, b = m["left"], m["right"]
        H, G = a["heads"], a["kv_heads"]
        q = rms_norm((h @ w[p + "left.q"].T).reshape(T, H, a["dim"]), w[p + "left.q.norm"], eps)
        k = rms_norm((h @ w[p + "left.k"].T).reshape(T, G, a["dim"]), w[p + "left.k.norm"], eps)
        v = (h @ w[p + "left.v"].T).reshape(T, G, a["vdim"])
        st = self.state.setdefault(i, {"k": k[:0], "v": v[:0], "s": np.zeros((b["heads"], b["dim"], b["vdim"]))})
        st["k"], st["v"] = np.concatenate([st["k"], k]), np.concatenate([st["v"], v])
        left = window_attention(q, st["k"], st["v"], positions, a["scale"], a["mask"]["size"]).reshape(T, -1) @ w[p + "left.o"].T
        q, k, v = (silu(h @ w[p + "right." + n].T).reshape(T, b["heads"], -1) for n in "qkv")
        o = lightning(q, k, v, b["decay"], st["s"]).reshape(T, -1)
        o = rms_norm(o, w[p + "right.norm"], eps) * sigmoid(h @ w[p + "right.g"].T)
        return m["left_scale"] * left + m["right_scale"] * (o @ w[p + "right.o"].T)

    def channel_delta(self, i, h, positions):
        m, w, p, eps, T = self.c["layers"][i]["mixer"], self.w, f"l{self.own(i)}.mix.", self.c["norm"]["eps"], h.shape[0]
        H, D = m["heads"], m["dim"]
        st = self.state.setdefault(i, {"s": np.zeros((H, D, m["vdim"])), **{n: np.zeros((m["conv"] - 1, w[p + n].shape[0])) for n in "qkv"}})
        x = {}
        for n in "qkv":
            x[n], st[n] = short_convolution(h @ w[p + n].T, w[p + n + ".conv"], st[n])
            x[n] = silu(x[n]).reshape(T, H if n == "v" else m["kv_heads"], -1)
        q, k = unit(x["q"]) * D ** -0.5, unit(x["k"])
        g = channel_decay((h @ w[p + "a1"].T @ w[p + "a2"].T).reshape(T, H, D), w[p + "A_log"], w[p + "dt_bias"])
        o = delta_rule(q, k, x["v"], sigmoid(h @ w[p + "b"].T), g, st["s"])
        gate = sigmoid(h @ w[p + "g1"].T @ w[p + "g2"].T).reshape(o.shape)
        return (rms_norm(o, w[p + "norm"], eps) * gate).reshape(T, -1) @ w[p + "o"].T

    def step(self, tokens):
        """Logits of every token of the portion [T, vocab]; the residual after every layer is left in self.layers."""
        w, eps = self.w, self.c["norm"]["eps"]
        positions = range(self.pos, self.pos + len(tokens))
        x = w["embed"][np.asarray(tokens)]
        self.layers = []
        for i, layer in enumerate(self.c["layers"]):
            p = f"l{self.own(i)}."
            x = x + getattr(self, layer["type"])(i, rms_norm(x, w[p + "norm1"], eps), positions)
            if layer.get("mlp") is not None:
                h = rms_norm(x, w[p + "norm2"], eps)
                x = x + (gelu_tanh(h @ w[p + "mlp.gate"].T) * (h @ w[p + "mlp.up"].T)) @ w[p + "mlp.down"].T
            self.layers.append(x)
        self.pos += len(tokens)
        return rms_norm(x, w["final.norm"], eps) @ w["embed"].T * self.c["logit_scale"]
