"""Sitirax: a decoder with norms on the sublayers' inputs whose layers mix either by windowed softmax attention and lightning
attention side by side ('parallel') or by a gated delta rule with a decay per key channel ('channel_delta'), followed (where the
layer has one) by a GELU-gated feed-forward.  A layer may use another layer's weights with a state of its own; the head is the
embedding.

Two passes over the same weights and caches (dense.py has the ops; the residual is fp32 throughout):

  one token      seven launches a layer.  parallel: residual + norm + all projections (silu included) | query / key norm, cache append
                 and lightning state step | attention over the keys of the window | merge, norm and gate | one product for both outputs
                 channel_delta: residual + norm + all projections | convolution, decay and gate products | state step | norm and gate |
                 output product
                 feed-forward: residual + norm + gate / up with the activation | down
  many tokens    the same steps as products over all rows; the recurrences in chunks of 64 tokens
"""

import dataclasses
import math
from typing import List, Optional, Tuple, Union

import torch

from . import dense
from .dense_model import DenseModel, SequenceCache, place

# Up to this many tokens a portion attends with its keys split over workgroups, like a single token.
SPLIT_MAX_TOKENS = 16
UNIT_EPS = 1e-6      # in the length of a query or key of the delta rule


@dataclasses.dataclass(frozen=True)
class WindowMixer:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: int


@dataclasses.dataclass(frozen=True)
class LightningMixer:
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]


@dataclasses.dataclass(frozen=True)
class ParallelMixer:
    left: WindowMixer
    right: LightningMixer
    left_scale: float
    right_scale: float


@dataclasses.dataclass(frozen=True)
class DeltaMixer:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    taps: int


@dataclasses.dataclass(frozen=True)
class LayerConfig:
    mixer: Union[ParallelMixer, DeltaMixer]
    ff: Optional[int]
    weights_of: Optional[int] = None    # a layer with weights of its own


def _grouped(what, m):
    heads, groups = int(m["heads"]), int(m["kv_heads"])
    if heads <= 0 or groups <= 0 or heads % groups:
        raise ValueError(f"{what}: {heads} heads over {groups} key / value heads")
    return heads, groups


def _parallel(what, m):
    a, b = m["left"], m["right"]
    heads, groups = _grouped(what, a)
    left = WindowMixer(heads, groups, int(a["dim"]), int(a["vdim"]), float(a["scale"]), int(a["mask"]["size"]))
    right = LightningMixer(int(b["heads"]), int(b["dim"]), int(b["vdim"]), tuple(float(x) for x in b["decay"]))
    if left.window <= 0 or left.scale == 0.0:
        raise ValueError(f"{what}: the window must be positive and the score scale not zero")
    if len(right.decay) != right.heads or min(right.decay) < 0.0:
        raise ValueError(f"{what}: {right.heads} heads need as many decays, none of them negative")
    return ParallelMixer(left, right, float(m["left_scale"]), float(m["right_scale"]))


def _delta(what, m):
    heads, groups = _grouped(what, m)
    out = DeltaMixer(heads, groups, int(m["dim"]), int(m["vdim"]), int(m["conv"]))
    if out.taps <= 0:
        raise ValueError(f"{what}: a convolution of {out.taps} taps")
    return out


MIXERS = {"parallel": _parallel, "channel_delta": _delta}


@dataclasses.dataclass(frozen=True)
class SitiraxConfig:
    vocab: int
    width: int
    eps: float
    logit_scale: float
    layers: List[LayerConfig]

    @classmethod
    def from_json(cls, c):
        layers = []
        for i, l in enumerate(c["layers"]):
            what = f"layer {i}"
            if l["type"] not in MIXERS:
                raise ValueError(f"{what}: unknown mixer '{l['type']}'")
            mixer, ff = MIXERS[l["type"]](what, l["mixer"]), None
            if l.get("mlp") is not None:
                if l["mlp"].get("kind", "dense") != "dense":
                    raise ValueError(f"{what}: unknown feed-forward '{l['mlp']['kind']}'")
                ff = int(l["mlp"]["ff"])
            of = l.get("weights_of")
            if of is not None:
                of = int(of)
                if not 0 <= of < len(c["layers"]) or of == i:
                    raise ValueError(f"{what}: weights_of must name another layer")
            layers.append(LayerConfig(mixer, ff, of))
        config = cls(vocab=int(c["vocab"]), width=int(c["width"]), eps=float(c["norm"]["eps"]), logit_scale=float(c["logit_scale"]), layers=layers)
        for i, l in enumerate(layers):
            j = config.owner(i)
            if (l.mixer, l.ff) != (layers[j].mixer, layers[j].ff):
                raise ValueError(f"layer {i}: differs from layer {j}, whose weights it uses")
        return config

    def owner(self, i):
        """The layer whose tensors layer i uses."""
        seen = set()
        while self.layers[i].weights_of is not None:
            if i in seen:
                raise ValueError(f"layer {i}: weights_of goes round in a circle")
            seen.add(i)
            i = self.layers[i].weights_of
        return i


def tensor_shapes(config):
    """Name -> shape of every tensor of a checkpoint; None is a length that the tensor itself decides (ranks)."""
    W = config.width
    out = {"embed": (config.vocab, W), "final.norm": (W,)}
    for i, l in enumerate(config.layers):
        if l.weights_of is not None:
            continue
        p, m = f"l{i}.", l.mixer
        out[p + "norm1"] = (W,)
        if isinstance(m, ParallelMixer):
            a, b, p2 = m.left, m.right, p + "mix."
            out.update({p2 + "left.q": (a.heads * a.dim, W), p2 + "left.k": (a.kv_heads * a.dim, W), p2 + "left.v": (a.kv_heads * a.vdim, W),
                        p2 + "left.q.norm": (a.dim,), p2 + "left.k.norm": (a.dim,), p2 + "left.o": (W, a.heads * a.vdim),
                        p2 + "right.q": (b.heads * b.dim, W), p2 + "right.k": (b.heads * b.dim, W), p2 + "right.v": (b.heads * b.vdim, W),
                        p2 + "right.g": (b.heads * b.vdim, W), p2 + "right.o": (W, b.heads * b.vdim), p2 + "right.norm": (b.heads * b.vdim,)})
        else:
            p2 = p + "mix."
            sizes = {"q": m.kv_heads * m.dim, "k": m.kv_heads * m.dim, "v": m.heads * m.vdim}
            for n, c in sizes.items():
                out.update({p2 + n: (c, W), p2 + n + ".conv": (c, m.taps)})
            out.update({p2 + "b": (m.heads, W), p2 + "A_log": (m.heads,), p2 + "norm": (m.vdim,), p2 + "a1": (None, W), p2 + "a2": (m.heads * m.dim, None),
                        p2 + "dt_bias": (m.heads * m.dim,), p2 + "g1": (None, W), p2 + "g2": (m.heads * m.vdim, None), p2 + "o": (W, m.heads * m.vdim)})
        if l.ff is not None:
            out.update({p + "norm2": (W,), p + "mlp.gate": (l.ff, W), p + "mlp.up": (l.ff, W), p + "mlp.down": (W, l.ff)})
    return out


class _Tensors:
    """Checkpoint tensors of one layer in the kernels' form: padded with zeros, head by head."""

    def __init__(self, config, i, tensor, dtype, device):
        self.p, self.tensor, self.dtype, self.device = f"l{i}.", tensor, dtype, device
        self.W, self.WP = config.width, dense.pad_to(config.width, dense.KP)

    def get(self, name, *shape):
        return self.tensor(self.p + name, shape).to(device=self.device, dtype=self.dtype)

    def f32(self, name, *shape):
        return self.tensor(self.p + name, shape).to(device=self.device, dtype=torch.float32)

    def vec(self, name, n, padded):
        return place(self.f32(name, n), (padded,)).contiguous()

    def heads_in(self, name, heads, dim, dim_p):
        """[heads * dim, W] -> [heads * dim_p, WP]"""
        return place(self.get(name, heads * dim, self.W).reshape(heads, dim, self.W), (heads, dim_p, self.WP)).reshape(-1, self.WP)

    def heads_out(self, name, heads, dim, dim_p):
        """[W, heads * dim] -> [WP, heads * dim_p]"""
        return place(self.get(name, self.W, heads * dim).reshape(self.W, heads, dim), (self.WP, heads, dim_p)).reshape(self.WP, -1)

    def heads_of(self, name, heads, dim, dim_p):
        """fp32 [heads * dim] -> [heads * dim_p]"""
        return place(self.f32(name, heads * dim).reshape(heads, dim), (heads, dim_p)).reshape(-1).contiguous()


def _check_state(spec):
    if not spec.supported():
        raise ValueError(f"no recurrence kernel for queries and keys of {spec.dim}")


def _output_width(columns):
    return dense.pad_to(columns, dense.KP)


class ParallelLayer:
    """Windowed attention and lightning attention on the same input.  The scales of the two results are folded into what is in front
    of their output products, which are one: out = [attention | read-outs], W = [W_o left | W_o right]."""

    def __init__(self, t, m, eps):
        a, b = m.left, m.right
        self.eps = eps
        sign = 1.0 if a.scale > 0 else -1.0
        self.attn = dense.HeadSpec(a.heads, a.kv_heads, a.dim, a.vdim, a.window, abs(a.scale), m.left_scale)
        self.state = s = dense.StateSpec(b.heads, b.heads, b.dim, b.vdim)
        A = self.attn
        parts = [t.heads_in("mix.left.q", a.heads, a.dim, A.dim_p), t.heads_in("mix.left.k", a.kv_heads, a.dim, A.dim_p),
                 t.heads_in("mix.left.v", a.kv_heads, a.vdim, A.vdim_p), t.heads_in("mix.right.q", b.heads, b.dim, s.dim_p),
                 t.heads_in("mix.right.k", b.heads, b.dim, s.dim_p), t.heads_in("mix.right.v", b.heads, b.vdim, s.vdim_p),
                 t.heads_in("mix.right.g", b.heads, b.vdim, s.vdim_p)]
        self.q_off = A.proj_width
        self.offsets = (self.q_off, self.q_off + s.qk_width, self.q_off + 2 * s.qk_width)
        self.gate_off = self.q_off + s.channels
        self.silu = (self.q_off, self.gate_off)
        self.w_in = torch.cat(parts).contiguous()
        self.q_norm = t.vec("mix.left.q.norm", a.dim, A.dim_p) * sign
        self.k_norm = t.vec("mix.left.k.norm", a.dim, A.dim_p)
        self.norm = t.heads_of("mix.right.norm", b.heads, b.vdim, s.vdim_p) * m.right_scale
        self.true_cols = b.heads * b.vdim
        self.log2_decay = torch.tensor([max(math.log2(x), -1.0e6) if x > 0 else -1.0e6 for x in b.decay], dtype=torch.float32, device=t.device)
        o = torch.cat([t.heads_out("mix.left.o", a.heads, a.vdim, A.vdim_p), t.heads_out("mix.right.o", b.heads, b.vdim, s.vdim_p)], dim=1)
        self.out_columns = o.shape[1]
        self.w_o = place(o, (t.WP, _output_width(o.shape[1]))).contiguous()

    def check(self, dtype):
        if not (self.attn.decode_supported(dtype) or self.attn.prefill_supported(dtype)):
            raise ValueError("no attention kernel for these head sizes")
        _check_state(self.state)

    def captured(self, dtype):
        return self.attn.decode_supported(dtype)

    def new_cache(self, model, capacity):
        A = self.attn
        ring = A.ring(capacity, model.max_portion)
        return {"rows": torch.empty((A.kv_heads, ring, A.dim_p + A.vdim_p), dtype=model.dtype, device=model.device),
                "state": self.state.new_state(model.device)}

    def mix(self, proj, cache, pos, out, pos_dev, capacity):
        M, A = proj.shape[0], self.attn
        few = A.decode_supported(proj.dtype) and (M <= SPLIT_MAX_TOKENS or not A.prefill_supported(proj.dtype))
        if pos_dev is not None and not few:
            raise ValueError("these head sizes cannot run with the position on the device")
        nsplit = dense.head_splits(A, 1, capacity) if pos_dev is not None else None
        if few and M == 1:
            dense.attention_and_state(A, self.state, proj, 0, self.q_norm, self.k_norm, self.eps, cache["rows"], self.offsets, cache["state"],
                                      self.log2_decay, pos, self.norm, self.true_cols, self.gate_off, out, pos_dev, nsplit)
            return
        dense.head_attention(A, proj, 0, self.q_norm, self.k_norm, self.eps, cache["rows"], pos, out, pos_dev=pos_dev, nsplit=nsplit, rows_form=not few)
        o = dense.recurrence(self.state, proj, self.offsets, cache["state"], pos, log2_decay=self.log2_decay, pos_dev=pos_dev)
        dense.gated_norm(o, self.norm, self.eps, 1, self.true_cols, proj[:, self.gate_off:], out[:, A.heads * A.vdim_p:])


class DeltaLayer:
    """Gated delta rule with a decay per key channel behind a short convolution."""

    silu = None

    def __init__(self, t, m, eps):
        self.eps, self.heads = eps, m.heads
        self.state = s = dense.StateSpec(m.heads, m.kv_heads, m.dim, m.vdim)
        self.q_scale = m.dim ** -0.5
        low = {n: t.get(f"mix.{n}", None, t.W) for n in ("a1", "g1")}
        rank = {n: dense.pad_to(x.shape[0], dense.KP) for n, x in low.items()}
        parts = [t.heads_in("mix.q", m.kv_heads, m.dim, s.dim_p), t.heads_in("mix.k", m.kv_heads, m.dim, s.dim_p),
                 t.heads_in("mix.v", m.heads, m.vdim, s.vdim_p), *(place(low[n], (rank[n], t.WP)) for n in ("a1", "g1")),
                 place(t.get("mix.b", m.heads, t.W), (dense.pad_to(m.heads, dense.ROW_PAD), t.WP))]
        self.a_off = s.channels
        self.g_off = self.a_off + rank["a1"]
        self.b_off = self.g_off + rank["g1"]
        self.w_in = torch.cat(parts).contiguous()
        a2, g2 = t.get("mix.a2", m.heads * m.dim, low["a1"].shape[0]), t.get("mix.g2", m.heads * m.vdim, low["g1"].shape[0])
        self.w_a2 = place(a2.reshape(m.heads, m.dim, -1), (m.heads, s.dim_p, rank["a1"])).reshape(-1, rank["a1"]).contiguous()
        self.w_g2 = place(g2.reshape(m.heads, m.vdim, -1), (m.heads, s.vdim_p, rank["g1"])).reshape(-1, rank["g1"]).contiguous()
        conv = []
        for n, heads, dim, dim_p in (("q", m.kv_heads, m.dim, s.dim_p), ("k", m.kv_heads, m.dim, s.dim_p), ("v", m.heads, m.vdim, s.vdim_p)):
            conv.append(place(t.f32(f"mix.{n}.conv", heads * dim, m.taps).reshape(heads, dim, m.taps), (heads, dim_p, m.taps)).reshape(-1, m.taps))
        self.conv = torch.cat(conv).t().contiguous()
        self.a_log = t.f32("mix.A_log", m.heads).contiguous()
        self.dt_bias = t.heads_of("mix.dt_bias", m.heads, m.dim, s.dim_p)
        self.norm = t.vec("mix.norm", m.vdim, s.vdim_p)
        self.out_columns = s.v_width
        self.w_o = place(t.heads_out("mix.o", m.heads, m.vdim, s.vdim_p), (t.WP, _output_width(s.v_width))).contiguous()

    def check(self, dtype):
        _check_state(self.state)

    def captured(self, dtype):
        return True

    def new_cache(self, model, capacity):
        return {"history": torch.zeros((self.conv.shape[0], self.state.channels), dtype=model.dtype, device=model.device),
                "state": self.state.new_state(model.device)}

    def mix(self, proj, cache, pos, out, pos_dev, capacity):
        s = self.state
        conv = (s, proj, 0, self.conv, cache["history"], pos, self.q_scale, UNIT_EPS)
        low_a, low_g = proj[:, self.a_off:self.g_off], proj[:, self.g_off:self.b_off]
        if proj.shape[0] == 1:
            act, factors, z, gate = dense.conv_products(*conv, low_a, self.w_a2, low_g, self.w_g2, pos_dev)
        else:
            act, factors = dense.short_conv(*conv, pos_dev)
            z, gate = dense.gemm(low_a, self.w_a2, out_f32=True), dense.gemm(low_g, self.w_g2)
        o = dense.recurrence(s, act, (0, s.qk_width, 2 * s.qk_width), cache["state"], pos, z=z, a_log=self.a_log, dt_bias=self.dt_bias, factors=factors,
                             beta=proj[:, self.b_off:], pos_dev=pos_dev)
        dense.gated_norm(o, self.norm, self.eps, s.heads, s.vdim, gate, out)


class SitiraxLayer:
    """Device tensors of one layer in the form the kernels read."""

    def __init__(self, config, i, tensor, dtype, device):
        l, t = config.layers[i], _Tensors(config, i, tensor, dtype, device)
        self.mixer = (ParallelLayer if isinstance(l.mixer, ParallelMixer) else DeltaLayer)(t, l.mixer, config.eps)
        try:
            self.mixer.check(dtype)
        except ValueError as e:
            raise ValueError(f"layer {i}: {e}") from None
        self.norm1 = t.vec("norm1", t.W, t.WP)
        self.norm2 = self.w_gate_up = self.w_down = None
        if l.ff is not None:
            FP = dense.pad_to(l.ff, dense.KP)
            self.norm2 = t.vec("norm2", t.W, t.WP)
            gu = [place(t.get(f"mlp.{n}", l.ff, t.W), (FP, t.WP)).reshape(FP // 16, 16, t.WP) for n in ("gate", "up")]
            self.w_gate_up = torch.stack(gu, dim=1).reshape(2 * FP, t.WP).contiguous()   # 16 gate rows, 16 up rows, ...
            self.w_down = place(t.get("mlp.down", t.W, l.ff), (t.WP, FP)).contiguous()


class SitiraxCache(SequenceCache):
    """One sequence: per layer a ring of key / value rows as long as the window and a portion, and fp32 states (with the last inputs
    of the convolution).  Nothing is cleared between sequences: what lies in front of position 0 is never read."""

    def __init__(self, model, capacity):
        super().__init__(model, capacity)
        self.layers = [l.mixer.new_cache(model, capacity) for l in model.layers]


class SitiraxModel(DenseModel):
    config_class = SitiraxConfig
    max_portion = 8192

    def __init__(self, config, tensor, dtype=torch.bfloat16, device="cuda", max_portion=None):
        """`tensor(name, shape)` gives the checkpoint's tensors (any device).  max_portion: most tokens that go through the layers
        at once, which bounds the activations and the key / value rows kept beside the window."""
        dense.dtype_code(dtype)
        self.config, self.dtype, self.device, self.vocab = config, dtype, torch.device(device), config.vocab
        if max_portion is not None:
            self.max_portion = max_portion
        W, self.width = config.width, dense.pad_to(config.width, dense.KP)
        t = tensor("embed", (config.vocab, W)).to(device=device, dtype=dtype)
        self.embed = self.head = place(t, (dense.pad_to(config.vocab, dense.ROW_PAD), self.width)).contiguous()
        final = tensor("final.norm", (W,)).to(device=device, dtype=torch.float32) * config.logit_scale   # (the logits are linear in it)
        self.final_norm = place(final, (self.width,)).contiguous()
        own = {i: SitiraxLayer(config, i, tensor, dtype, device) for i in range(len(config.layers)) if config.layers[i].weights_of is None}
        self.layers = [own[config.owner(i)] for i in range(len(config.layers))]

    def new_cache(self, max_tokens):
        return SitiraxCache(self, max_tokens)

    def _captured_decode(self):
        return all(l.mixer.captured(self.dtype) for l in self.layers)

    def _mix(self, i, proj, cache, pos, pos_dev=None):
        m, M = self.layers[i].mixer, proj.shape[0]
        exact = m.out_columns == m.w_o.shape[1]
        out = (torch.empty if exact else torch.zeros)((M, m.w_o.shape[1]), dtype=self.dtype, device=self.device)
        m.mix(proj, cache.layers[i], pos, out, pos_dev, cache.capacity)
        return out

    def _one_token(self, cache, token, pos, pos_dev=None):
        """One token (device int32 [1]) through every layer; returns the Sum in front of the final norm."""
        c = self.config
        s = dense.Sum(token=token, embed=self.embed)
        for i, l in enumerate(self.layers):
            proj, res = dense.gemv_normed(s, l.norm1, c.eps, c.width, l.mixer.w_in, silu=l.mixer.silu)
            out = self._mix(i, proj.reshape(1, -1), cache, pos, pos_dev)
            s = dense.Sum(res, dense.gemv(out.reshape(-1), l.mixer.w_o, out_f32=True))
            if l.norm2 is not None:
                h, res = dense.gemv_normed(s, l.norm2, c.eps, c.width, l.w_gate_up, gate=dense.GATE_GELU)
                s = dense.Sum(res, dense.gemv(h, l.w_down, out_f32=True))
        return s

    def _rows(self, cache, tokens, pos, trace=None):
        """M tokens (device int32 [M]) through every layer; returns the fp32 residual [M, width].  `trace`: a list that
        receives a copy of the residual after every layer."""
        c, M = self.config, tokens.numel()
        res = torch.empty((M, self.width), dtype=torch.float32, device=self.device)
        y, embedding = None, dict(tokens=tokens, embed=self.embed)
        for i, l in enumerate(self.layers):
            h = dense.add_norm_rows(res, y, l.norm1, c.eps, c.width, self.dtype, **embedding)
            embedding = {}
            out = self._mix(i, dense.gemm(h, l.mixer.w_in, silu=l.mixer.silu), cache, pos)
            y = dense.gemm(out, l.mixer.w_o, out_f32=True)
            if l.norm2 is not None:
                h = dense.add_norm_rows(res, y, l.norm2, c.eps, c.width, self.dtype)
                y = dense.gemm(dense.gemm(h, l.w_gate_up, gate=dense.GATE_GELU), l.w_down, out_f32=True)
            if trace is not None:
                trace.append(res + y)
        dense.add_norm_rows(res, y, None, c.eps, c.width, self.dtype, **embedding)
        return res

    def _pending(self, res):
        return dense.Sum(res)

    def _head(self, s, keys=None):
        c = self.config
        return dense.gemv_normed(s, self.final_norm, c.eps, c.width, self.head, out_f32=True, keys=keys, n_valid=self.vocab, keep=False)[0]

    def _head_rows(self, res, rows):
        c = self.config
        return dense.gemm(dense.norm_rows(res, self.final_norm, c.eps, c.width, self.dtype, rows), self.head, out_f32=True)
