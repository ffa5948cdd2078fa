"""Kuvonex: a decoder whose layers are latent attention with a sink and an output gate, followed (where the layer has one)
by a mixture of experts behind a grouped sigmoid router.  The norms sit on the sublayers' outputs, the residual stream
is fp32 and is what the sublayers read; a layer may attend over the cache of an earlier layer instead of its own.

Two paths over the same weights and caches (dense.py has the ops):

  one token      per layer eight launches: residual + norm + Q | latent | gate product; cache append + key projection of the
                 queries; attention over the latents; merge + value projection + gate; O product; residual + norm + router
                 product; gate / up of the chosen experts (choosing included); their weighted down products.  The tail is
                 one product with both norms in its intake, and the argmax.
  many tokens    the same steps as products over all rows.  Long portions expand keys and values per head, short ones
                 attend over the latents like a single token; the experts run grouped over entries sorted by expert.
"""

import dataclasses
from typing import List, Optional

import numpy as np
import torch

from . import dense
from .dense_model import DenseModel, SequenceCache, place as _place

# Up to this many tokens a portion attends over the latents: expanding keys and values of the whole cache costs
# rank * (dim + vdim) per cached token and head whatever the portion's length, the latent form (2 rank + rot) instead
# of (dim + rot + vdim) per pair of query and key.
ABSORB_MAX_TOKENS = 64


@dataclasses.dataclass(frozen=True)
class LatentMixer:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    rot_base: float
    kv_from: Optional[int] = None


@dataclasses.dataclass(frozen=True)
class Mixture:
    experts: int
    top: int
    groups: int
    keep: int
    ff: int


@dataclasses.dataclass(frozen=True)
class LayerConfig:
    mixer: LatentMixer
    mlp: Optional[Mixture]


@dataclasses.dataclass(frozen=True)
class KuvonexConfig:
    vocab: int
    width: int
    eps: float
    embed_scale: float
    layers: List[LayerConfig]

    @classmethod
    def from_json(cls, c):
        layers = []
        for i, l in enumerate(c["layers"]):
            if l["type"] != "latent_attention":
                raise ValueError(f"layer {i}: unknown mixer '{l['type']}'")
            m = l["mixer"]
            src = m.get("kv_from")
            mixer = LatentMixer(heads=int(m["heads"]), dim=int(m["dim"]), rot_dim=int(m["rot_dim"]), vdim=int(m["vdim"]), kv_rank=int(m["kv_rank"]),
                                scale=float(m["scale"]), rot_base=float(m["rot"]["base"]), kv_from=None if src is None else int(src))
            if mixer.rot_dim <= 0 or mixer.rot_dim % 2 or int(m["rot"].get("dims", mixer.rot_dim)) != mixer.rot_dim:
                raise ValueError(f"layer {i}: rot_dim must be even, positive and the same in rot.dims")
            if not mixer.scale > 0:
                raise ValueError(f"layer {i}: the score scale must be positive")
            if src is not None:
                if not 0 <= mixer.kv_from < i or layers[mixer.kv_from].mixer.kv_from is not None:
                    raise ValueError(f"layer {i}: kv_from must name an earlier layer with a latent of its own")
                s = layers[mixer.kv_from].mixer
                if (s.kv_rank, s.rot_dim, s.rot_base) != (mixer.kv_rank, mixer.rot_dim, mixer.rot_base):
                    raise ValueError(f"layer {i}: latent size and rotation differ from layer {mixer.kv_from}'s")
            mlp = None
            if l.get("mlp") is not None:
                f = l["mlp"]
                if f.get("kind", "moe") != "moe":
                    raise ValueError(f"layer {i}: unknown feed-forward '{f['kind']}'")
                r = f["router"]
                g = r.get("groups") or {"count": 1, "keep": 1}
                mlp = Mixture(experts=int(r["experts"]), top=int(r["top"]), groups=int(g["count"]), keep=int(g["keep"]), ff=int(f["expert"]["ff"]))
                if mlp.groups <= 0 or mlp.experts % mlp.groups or not 0 < mlp.keep <= mlp.groups or mlp.top > mlp.keep * (mlp.experts // mlp.groups):
                    raise ValueError(f"layer {i}: {mlp.experts} experts in {mlp.groups} groups, {mlp.keep} kept, do not give {mlp.top}")
            layers.append(LayerConfig(mixer, mlp))
        return cls(vocab=int(c["vocab"]), width=int(c["width"]), eps=float(c["norm"]["eps"]), embed_scale=float(c["embedding"]["scale"]), layers=layers)


def tensor_shapes(config):
    """Name -> shape of every tensor of a checkpoint."""
    W = config.width
    out = {"embed": (config.vocab, W), "final.norm": (W,), "head": (config.vocab, W)}
    for i, l in enumerate(config.layers):
        m, p = l.mixer, f"l{i}."
        out.update({p + "norm1": (W,), p + "mix.q": (m.heads * (m.dim + m.rot_dim), W), p + "mix.uk": (m.heads * m.dim, m.kv_rank),
                    p + "mix.uv": (m.heads * m.vdim, m.kv_rank), p + "mix.sink": (m.heads,), p + "mix.g": (m.heads * m.vdim, W),
                    p + "mix.o": (W, m.heads * m.vdim)})
        if m.kv_from is None:
            out.update({p + "mix.dkv": (m.kv_rank + m.rot_dim, W), p + "mix.dkv.norm": (m.kv_rank,)})
        if l.mlp is not None:
            f = l.mlp
            out.update({p + "norm2": (W,), p + "mlp.router": (f.experts, W), p + "mlp.correction": (f.experts,)})
            for e in range(f.experts):
                out.update({f"{p}mlp.e{e}.gate": (f.ff, W), f"{p}mlp.e{e}.up": (f.ff, W), f"{p}mlp.e{e}.down": (W, f.ff)})
    return out


@dataclasses.dataclass
class KuvonexLayer:
    """Device tensors of one layer in the form the kernels read (padded with zeros, see dense.py)."""

    spec: dense.LatentSpec
    source: int              # layer whose cache is attended over (its own index with a latent of its own)
    rot_base: float
    w_in: torch.Tensor       # Q per head [dim | rot], then latent | key part (own latent only), then the gate
    kv_off: int              # columns of that product: latent (-1: none) ...
    gate_off: int            # ... and gate
    kv_norm: Optional[torch.Tensor]
    w_ukv: torch.Tensor      # key projections of all heads, then value projections
    sink: torch.Tensor
    w_o: torch.Tensor
    norm1: torch.Tensor
    norm2: Optional[torch.Tensor] = None
    router: Optional[dense.RouterSpec] = None
    w_router: Optional[torch.Tensor] = None
    w_gate_up: Optional[torch.Tensor] = None
    w_down: Optional[torch.Tensor] = None


def prepare_layer(config, i, tensor, dtype=torch.bfloat16, device="cuda"):
    """Layer i from `tensor(name, shape)` (checkpoint orientation [out, in]) in the kernels' form."""
    l, p = config.layers[i], f"l{i}."
    m, W = l.mixer, config.width
    spec = dense.LatentSpec(m.heads, m.dim, m.rot_dim, m.vdim, m.kv_rank, m.scale)
    WP = dense.pad_to(W, dense.KP)

    def get(name, *shape):
        return tensor(p + name, shape).to(device=device, dtype=dtype)

    def vec(name, n, padded):
        return _place(tensor(p + name, (n,)).to(device=device, dtype=torch.float32), (padded,)).contiguous()

    H, R = m.heads, m.kv_rank
    q = get("mix.q", H * (m.dim + m.rot_dim), W).reshape(H, m.dim + m.rot_dim, W)
    parts = [torch.cat([_place(q[:, :m.dim], (H, spec.dim_p, WP)), _place(q[:, m.dim:], (H, spec.rot_p, WP))], dim=1).reshape(-1, WP)]
    kv_off, kv_norm = -1, None
    if m.kv_from is None:
        kv_off = parts[0].shape[0]
        dkv = get("mix.dkv", R + m.rot_dim, W)
        parts += [_place(dkv[:R], (spec.rank_p, WP)), _place(dkv[R:], (spec.rot_p, WP))]
        kv_norm = vec("mix.dkv.norm", R, spec.rank_p)
    gate_off = sum(x.shape[0] for x in parts)
    parts.append(_place(get("mix.g", H * m.vdim, W).reshape(H, m.vdim, W), (H, spec.vdim_p, WP)).reshape(-1, WP))
    uk = _place(get("mix.uk", H * m.dim, R).reshape(H, m.dim, R), (H, spec.dim_p, spec.rank_p)).reshape(-1, spec.rank_p)
    uv = _place(get("mix.uv", H * m.vdim, R).reshape(H, m.vdim, R), (H, spec.vdim_p, spec.rank_p)).reshape(-1, spec.rank_p)
    o = _place(get("mix.o", W, H * m.vdim).reshape(W, H, m.vdim), (WP, H, spec.vdim_p)).reshape(WP, -1)
    out = KuvonexLayer(spec=spec, source=i if m.kv_from is None else m.kv_from, rot_base=m.rot_base, w_in=torch.cat(parts).contiguous(), kv_off=kv_off,
                       gate_off=gate_off, kv_norm=kv_norm, w_ukv=torch.cat([uk, uv]).contiguous(), sink=vec("mix.sink", H, H),
                       w_o=_place(o, (WP, spec.out_width)).contiguous(), norm1=vec("norm1", W, WP))
    if l.mlp is not None:
        f = l.mlp
        FP = dense.pad_to(f.ff, dense.KP)
        out.norm2 = vec("norm2", W, WP)
        out.w_router = _place(get("mlp.router", f.experts, W), (dense.pad_to(f.experts, dense.ROW_PAD), WP)).contiguous()
        out.router = dense.RouterSpec(vec("mlp.correction", f.experts, f.experts), f.experts, f.top, f.groups, f.keep)
        out.w_gate_up = torch.empty((f.experts, 2 * FP, WP), dtype=dtype, device=device)
        out.w_down = torch.empty((f.experts, WP, FP), dtype=dtype, device=device)
        for e in range(f.experts):
            gu = torch.stack([_place(get(f"mlp.e{e}.{n}", f.ff, W), (FP, WP)).reshape(FP // 16, 16, WP) for n in ("gate", "up")], dim=1)
            out.w_gate_up[e] = gu.reshape(2 * FP, WP)   # 16 gate rows, 16 up rows, ...
            out.w_down[e] = _place(get(f"mlp.e{e}.down", W, f.ff), (WP, FP))
    return out


def rotation_table(base, dims, n, device):
    """fp32 [n, dims / 2, 2]: cos and sin of position * base^(-2 i / dims), evaluated in float64."""
    f = float(base) ** (-np.arange(0, dims, 2, dtype=np.float64) / dims)
    a = np.outer(np.arange(n, dtype=np.float64), f)
    return torch.from_numpy(np.stack([np.cos(a), np.sin(a)], axis=-1).astype(np.float32)).to(device)


class LatentCache(SequenceCache):
    """Latent rows of one sequence: one matrix [capacity, rank + rot] per layer that has a latent of its own (layers that
    share one have no entry)."""

    def __init__(self, model, capacity):
        super().__init__(model, capacity)
        dev = model.device
        self.rows = {i: torch.empty((capacity, l.spec.cache_width), dtype=model.dtype, device=dev) for i, l in enumerate(model.layers) if l.source == i}
        self.tables = {(l.rot_base, l.spec.rot): model.rotation(l.rot_base, l.spec.rot, capacity) for l in model.layers}


class KuvonexModel(DenseModel):
    config_class = KuvonexConfig

    def __init__(self, config, tensor, dtype=torch.bfloat16, device="cuda"):
        """`tensor(name, shape)` gives the checkpoint's tensors (any device)."""
        dense.dtype_code(dtype)
        self.config, self.dtype, self.device, self.vocab = config, dtype, torch.device(device), config.vocab
        W, WP = config.width, dense.pad_to(config.width, dense.KP)
        self.width = WP

        def matrix(name):
            t = tensor(name, (config.vocab, W)).to(device=device, dtype=dtype)
            return _place(t, (dense.pad_to(config.vocab, dense.ROW_PAD), WP)).contiguous()

        self.embed, self.head = matrix("embed"), matrix("head")
        self.final_norm = _place(tensor("final.norm", (W,)).to(device=device, dtype=torch.float32), (WP,)).contiguous()
        self.layers = [prepare_layer(config, i, tensor, dtype, device) for i in range(len(config.layers))]
        for i, l in enumerate(self.layers):
            if not (l.spec.decode_supported(dtype) or l.spec.prefill_supported(dtype)):
                raise ValueError(f"layer {i}: no attention kernel for these head and latent sizes")
        self._tables = {}

    def new_cache(self, max_tokens):
        return LatentCache(self, max_tokens)

    def rotation(self, base, dims, n):
        """Rotation table of at least n positions, shared by the caches (which keep the one they were made with)."""
        table = self._tables.get((base, dims))
        if table is None or table.shape[0] < n:
            table = self._tables[(base, dims)] = rotation_table(base, dims, n, self.device)
        return table

    # -- pieces --------------------------------------------------------------------------
    def _attend(self, l, proj, cache, pos, pos_dev=None, nsplit=None):
        M = 1 if proj.dim() == 1 else proj.shape[0]
        args = (l.spec, proj, l.kv_off, l.gate_off, cache.tables[(l.rot_base, l.spec.rot)], l.kv_norm, self.config.eps, cache.rows[l.source], pos,
                l.w_ukv, l.sink)
        if l.spec.decode_supported(self.dtype) and (M <= ABSORB_MAX_TOKENS or not l.spec.prefill_supported(self.dtype)):
            return dense.latent_attention_absorbed(*args, pos_dev=pos_dev, nsplit=nsplit)
        if pos_dev is not None:
            raise ValueError("this head or latent size cannot run with the position on the device")
        return dense.latent_attention_rows(l.spec, proj.reshape(M, -1), *args[2:])

    def _one_token(self, cache, token, pos, pos_dev=None):
        """One token (device int32 [1]) through every layer; returns the Residual in front of the final norm."""
        c = self.config
        r = None
        for l in self.layers:
            if r is None:
                proj, res, _ = dense.gemv_embed(token, self.embed, c.embed_scale, l.w_in)
            else:
                proj, res, _ = dense.gemv_residual(r, l.w_in)
            nsplit = None if pos_dev is None else dense.latent_splits(l.spec, 1, cache.capacity)
            attn = self._attend(l, proj, cache, pos, pos_dev, nsplit)
            y = dense.gemv(attn.reshape(-1), l.w_o, out_f32=True)
            r = dense.Residual(res, y, l.norm1, c.eps, c.width)
            if l.router is not None:
                logits, res, h = dense.gemv_residual(r, l.w_router, out_f32=True, want_h=True)
                y = dense.moe_gemv(h, logits, l.router, l.w_gate_up, l.w_down)
                r = dense.Residual(res, y, l.norm2, c.eps, c.width)
        return r

    def _rows(self, cache, tokens, pos, trace=None):
        """M tokens (device int32 [M]) through every layer; returns the fp32 residual [M, width].  `trace`: a list that
        receives a copy of the residual after every layer."""
        c = self.config
        res, h = dense.embed_rows(tokens, self.embed, c.embed_scale)
        for l in self.layers:
            attn = self._attend(l, dense.gemm(h, l.w_in), cache, pos)
            y = dense.gemm(attn, l.w_o, out_f32=True)
            h = dense.residual_norm_rows(res, y, l.norm1, c.eps, c.width, self.dtype)
            if l.router is not None:
                logits = dense.gemm(h, l.w_router, out_f32=True)
                y, wts = dense.moe_rows(h, logits, l.router, l.w_gate_up, l.w_down)
                h = dense.residual_norm_rows(res, y, l.norm2, c.eps, c.width, self.dtype, weights=wts)
            if trace is not None:
                trace.append(res.clone())
        return res

    def _pending(self, res):
        return dense.Residual(res, None, None, self.config.eps, self.config.width)

    def _head(self, r, keys=None):
        return dense.gemv_final(r, self.final_norm, self.head, keys, self.vocab)

    def _head_rows(self, res, rows):
        c = self.config
        return dense.gemm(dense.norm_rows(res, self.final_norm, c.eps, c.width, self.dtype, rows), self.head, out_f32=True)

    def _captured_decode(self):
        return all(l.spec.decode_supported(self.dtype) for l in self.layers)
