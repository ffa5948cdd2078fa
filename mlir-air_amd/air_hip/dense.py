"""Operator-level wrappers over the dense-weight C ABI (include/dense_lm.h) for torch (ROCm) tensors.

As in ops.py, torch is used for device memory and streams only, every function launches on the current torch stream and
returns without synchronising, and there is no CPU path.  Weights and activations are bf16 or float32 throughout a call;
the residual stream, norm weights, sinks and router logits are float32.  Sizes are padded with zeros by whoever prepares
the weights (`pad_to`, KP / HEAD_PAD / ROW_PAD below).
"""

import ctypes

import torch

from . import _lib
from .ops import _need_cuda, _ptr, _stream

KP = 64          # input lengths of products, the latent's rank
HEAD_PAD = 32    # parts of a head
ROW_PAD = 16     # output lengths

PLAIN, RESIDUAL, EMBED, FINAL = 0, 1, 2, 3
NORMED = 4
OUT_ELEM, OUT_F32, OUT_SWIGLU, OUT_GEGLU = 0, 1, 2, 3
GATE_NONE, GATE_SILU, GATE_GELU = 0, 1, 2
STATE_PAD = 64   # a recurrence's query / key size ...
STATE_MAX = 512  # ... and the largest there is a kernel for


def pad_to(n, k):
    return (n + k - 1) // k * k


def dtype_code(t):
    """0 / 1 of a bf16 / float32 tensor (or torch dtype)."""
    dt = t if isinstance(t, torch.dtype) else t.dtype
    if dt == torch.bfloat16:
        return 0
    if dt == torch.float32:
        return 1
    raise TypeError(f"the dense-weight kernels take bfloat16 or float32, got {dt}")


def _need_f32(*tensors):
    for t in tensors:
        if t is not None and t.dtype != torch.float32:
            raise TypeError(f"expected a float32 tensor, got {t.dtype}")


def _opt(t):
    return None if t is None else t.data_ptr()


def _same(what, a, *others):
    for t in others:
        if t is not None and t.dtype != a.dtype:
            raise TypeError(f"{what}: mixed element types {a.dtype} and {t.dtype}")


class Residual:
    """The residual stream of one token between two sublayers: fp32 `res`, and the previous sublayer's output `y`, whose
    norm (weight `norm_w`) is still to be added.  The next product adds it on its way in."""

    __slots__ = ("res", "y", "norm_w", "eps", "width")

    def __init__(self, res, y, norm_w, eps, width):
        self.res, self.y, self.norm_w, self.eps, self.width = res, y, norm_w, eps, width


def _gemv(w, intake, out_f32, keys, n_valid, device):
    lib = _lib.load_dense_library()
    N, K = w.shape
    out = torch.empty((N,), dtype=torch.float32 if out_f32 else w.dtype, device=device)
    _lib.check_dense(lib.dlm_gemv(dtype_code(w), _ptr(w), ctypes.byref(intake), None if out_f32 else _ptr(out), _ptr(out) if out_f32 else None,
                                  _opt(keys), n_valid, K, N, _stream()))
    return out


def gemv(x, w, out_f32=False, keys=None, n_valid=0):
    """y[N] = W[N, K] x[K] (in the element type, or fp32)."""
    _need_cuda(x, w)
    _same("gemv", w, x)
    if x.numel() != w.shape[1]:
        raise ValueError(f"x has {x.numel()} elements but the matrix has {w.shape[1]} columns")
    return _gemv(w, _lib.Intake(mode=PLAIN, x=_ptr(x)), out_f32, keys, n_valid, w.device)


def gemv_embed(token, embed, scale, w, want_h=False):
    """The embedding row of token[0] times `scale` into a one-token product.  Returns (y, residual fp32 [K], h or None)."""
    _need_cuda(token, embed, w)
    _same("gemv_embed", w, embed)
    K = w.shape[1]
    if embed.shape[1] != K or token.dtype != torch.int32:
        raise ValueError("gemv_embed: embed must be [vocab, K] and token int32")
    res = torch.empty((K,), dtype=torch.float32, device=w.device)
    h = torch.empty((K,), dtype=w.dtype, device=w.device) if want_h else None
    intake = _lib.Intake(mode=EMBED, width=K, scale=scale, embed=_ptr(embed), token=_ptr(token), res_out=_ptr(res), h_out=_opt(h))
    return _gemv(w, intake, False, None, 0, w.device), res, h


def gemv_residual(r, w, out_f32=False, want_h=False):
    """The Residual `r` brought up to date into a one-token product.  Returns (y, new residual fp32 [K], h or None)."""
    _need_cuda(r.res, r.y, r.norm_w, w)
    _need_f32(r.res, r.y, r.norm_w)
    K = w.shape[1]
    if r.res.numel() != K or r.y.numel() != K or r.norm_w.numel() != K:
        raise ValueError(f"gemv_residual: residual, output and norm weight must have {K} elements")
    res = torch.empty((K,), dtype=torch.float32, device=w.device)
    h = torch.empty((K,), dtype=w.dtype, device=w.device) if want_h else None
    intake = _lib.Intake(mode=RESIDUAL, width=r.width, eps=r.eps, res=_ptr(r.res), y=_ptr(r.y), norm_w=_ptr(r.norm_w), res_out=_ptr(res),
                         h_out=_opt(h))
    return _gemv(w, intake, out_f32, None, 0, w.device), res, h


def gemv_final(r, final_w, w, keys=None, n_valid=0):
    """fp32 logits [N] of the Residual `r`: brought up to date, normed with final_w, times W."""
    _need_cuda(r.res, final_w, w)
    _need_f32(r.res, r.y, r.norm_w, final_w)
    K = w.shape[1]
    if r.res.numel() != K or final_w.numel() != K:
        raise ValueError(f"gemv_final: residual and norm weight must have {K} elements")
    intake = _lib.Intake(mode=FINAL, width=r.width, eps=r.eps, res=_ptr(r.res), y=_opt(r.y), norm_w=_opt(r.norm_w), final_w=_ptr(final_w))
    return _gemv(w, intake, True, keys, n_valid, w.device)


class Sum:
    """The residual stream of one token in front of a sublayer that norms its input: fp32 `res`, and the previous sublayer's output
    `y` (or None), still to be added; or, in front of the first layer, the embedding row of a token."""

    __slots__ = ("res", "y", "token", "embed", "scale")

    def __init__(self, res=None, y=None, token=None, embed=None, scale=1.0):
        self.res, self.y, self.token, self.embed, self.scale = res, y, token, embed, scale


def gemv_normed(s, norm_w, eps, width, w, silu=None, gate=GATE_NONE, out_f32=False, keys=None, n_valid=0, keep=True):
    """The Sum `s` brought up to date, normed with norm_w, times W.  `silu`: a range of rows that silu is applied to; `gate`: W holds
    interleaved gate and up rows (16 each) and the result is their gated half.  Returns (y, the sum fp32 [K] with `keep`)."""
    lib = _lib.load_dense_library()
    _need_cuda(norm_w, w)
    _need_f32(s.res, s.y, norm_w)
    N, K = w.shape
    if norm_w.numel() != K or any(t is not None and t.numel() != K for t in (s.res, s.y)) or (s.embed is not None and s.embed.shape[1] != K):
        raise ValueError(f"gemv_normed: the stream and the norm weight must have {K} elements")
    _same("gemv_normed", w, s.embed)
    if s.token is not None and s.token.dtype != torch.int32:
        raise TypeError("gemv_normed takes an int32 token")
    res = torch.empty((K,), dtype=torch.float32, device=w.device) if keep else None
    intake = _lib.Intake(mode=NORMED, width=width, eps=eps, scale=s.scale, res=_opt(s.res), y=_opt(s.y), final_w=_ptr(norm_w), res_out=_opt(res),
                         embed=_opt(s.embed), token=_opt(s.token))
    if gate == GATE_NONE and silu is None:
        return _gemv(w, intake, out_f32, keys, n_valid, w.device), res
    if out_f32 or keys is not None:
        raise ValueError("gemv_normed: activations come in the element type and without keys")
    out = torch.empty((N // 2 if gate else N,), dtype=w.dtype, device=w.device)
    begin, end = silu or (0, 0)
    ro = _lib.RowOutput(silu_begin=begin, silu_end=end, gate=gate)
    _lib.check_dense(lib.dlm_gemv_act(dtype_code(w), _ptr(w), ctypes.byref(intake), ctypes.byref(ro), _ptr(out), K, N, _stream()))
    return out, res


def new_keys(w):
    """Argmax keys of a one-token product with W."""
    n = _lib.load_dense_library().dlm_gemv_keys(w.shape[1], w.shape[0])
    return torch.empty((n,), dtype=torch.int64, device=w.device)


def argmax(keys, token=None, position=None, history=None):
    """Greedy choice from the keys of a product: token[0] = the row; position[0] += 1; history[position[0]] = the row."""
    for t in (token, position, history):
        if t is not None and (t.dtype != torch.int32 or not t.is_cuda):
            raise TypeError("argmax: token, position and history are int32 GPU tensors")
    lib = _lib.load_dense_library()
    _lib.check_dense(lib.dlm_argmax(_ptr(keys), keys.numel(), _opt(token), _opt(position), _opt(history), _stream()))


def gemm(a, w, out_f32=False, lda=None, rows=None, out=None, silu=None, gate=GATE_NONE):
    """out[M, N] = A[M, K] W[N, K]^T; a: [M, >= K] with row stride `lda` (default: its width).  `silu`, `gate` as in gemv_normed."""
    lib = _lib.load_dense_library()
    _need_cuda(w)
    _same("gemm", w, a)
    N, K = w.shape
    M = a.shape[0] if rows is None else rows
    lda = a.stride(0) if lda is None else lda
    if not a.is_cuda or a.stride(-1) != 1 or a.shape[1] < K or M > a.shape[0]:
        raise ValueError(f"gemm: A must be a GPU matrix with at least {K} columns and {M} rows")
    width = N // 2 if gate else N
    if out is None:
        out = torch.empty((M, width), dtype=torch.float32 if out_f32 else w.dtype, device=w.device)
    begin, end = silu or (0, 0)
    epilogue = OUT_F32 if out_f32 else {GATE_NONE: OUT_ELEM, GATE_SILU: OUT_SWIGLU, GATE_GELU: OUT_GEGLU}[gate]
    g = _lib.GemmArgs(a=a.data_ptr(), w=_ptr(w), out=_ptr(out), lda=lda, ldo=width, M=M, N=N, K=K, epilogue=epilogue, silu_begin=begin, silu_end=end,
                      tile_rows=lib.dlm_gemm_tile_rows(dtype_code(w), M, N, 1))
    _lib.check_dense(lib.dlm_gemm(dtype_code(w), ctypes.byref(g), _stream()))
    return out


def embed_rows(tokens, embed, scale):
    """(residual fp32 [M, K], the same in the element type) of int32 tokens [M]."""
    lib = _lib.load_dense_library()
    _need_cuda(tokens, embed)
    if tokens.dtype != torch.int32:
        raise TypeError("embed_rows takes int32 tokens")
    M, K = tokens.numel(), embed.shape[1]
    res = torch.empty((M, K), dtype=torch.float32, device=embed.device)
    h = torch.empty((M, K), dtype=embed.dtype, device=embed.device)
    _lib.check_dense(lib.dlm_embed_rows(dtype_code(embed), _ptr(tokens), _ptr(embed), scale, _ptr(res), _ptr(h), M, K, _stream()))
    return res, h


def residual_norm_rows(res, y, norm_w, eps, width, dtype, weights=None):
    """res += norm(y) in place; returns res in the element type.  With router weights [M, top], y [M * top, K] holds the
    chosen experts' outputs in the element type; otherwise y is fp32 [M, K]."""
    lib = _lib.load_dense_library()
    _need_cuda(res, y, norm_w)
    _need_f32(res, norm_w, weights)
    M, K = res.shape
    top = 0 if weights is None else weights.shape[1]
    if tuple(y.shape) != (M * max(top, 1), K) or norm_w.numel() != K or y.dtype != (dtype if top else torch.float32):
        raise ValueError("residual_norm_rows: shapes or types of y and the norm weight do not match")
    h = torch.empty((M, K), dtype=dtype, device=res.device)
    _lib.check_dense(lib.dlm_residual_norm_rows(dtype_code(dtype), _ptr(res), _ptr(y), _opt(weights), top, _ptr(norm_w), eps, width, _ptr(h), M, K,
                                                _stream()))
    return h


def add_norm_rows(res, y, norm_w, eps, width, dtype, tokens=None, embed=None, scale=1.0):
    """The residual rows brought up to date in place - res + y (y fp32 [M, K] or None), or with `tokens` the embedding rows times
    `scale` - and their norm in the element type (None without norm_w)."""
    lib = _lib.load_dense_library()
    _need_cuda(res)
    _need_f32(res, y, norm_w)
    M, K = res.shape
    if (y is not None and tuple(y.shape) != (M, K)) or (norm_w is not None and norm_w.numel() != K):
        raise ValueError("add_norm_rows: shapes of the residual, y and the norm weight do not match")
    if tokens is not None and (tokens.dtype != torch.int32 or tokens.numel() != M or embed.shape[1] != K or embed.dtype != dtype or y is not None):
        raise ValueError("add_norm_rows: int32 tokens, one per row, and an embedding of the rows' width")
    h = None if norm_w is None else torch.empty((M, K), dtype=dtype, device=res.device)
    _lib.check_dense(lib.dlm_add_norm_rows(dtype_code(dtype), _ptr(res), _opt(y), _opt(tokens), _opt(embed), scale, _opt(norm_w), eps, width, _opt(h), M, K,
                                           _stream()))
    return h


def norm_rows(res, norm_w, eps, width, dtype, rows=None):
    """norm(res[rows]) in the element type; rows: int32 indices (every row without them)."""
    lib = _lib.load_dense_library()
    _need_cuda(res, norm_w)
    _need_f32(res, norm_w)
    n = res.shape[0] if rows is None else rows.numel()
    if rows is not None and (rows.dtype != torch.int32 or not rows.is_cuda):
        raise TypeError("norm_rows takes int32 GPU row indices")
    out = torch.empty((n, res.shape[1]), dtype=dtype, device=res.device)
    _lib.check_dense(lib.dlm_norm_rows(dtype_code(dtype), _ptr(res), _opt(rows), _ptr(norm_w), eps, width, _ptr(out), n, res.shape[1], _stream()))
    return out


class RouterSpec:
    """Grouped sigmoid router: sizes and the choice correction (fp32 [experts])."""

    __slots__ = ("correction", "experts", "top", "groups", "keep")

    def __init__(self, correction, experts, top, groups=1, keep=1):
        self.correction, self.experts, self.top, self.groups, self.keep = correction, experts, top, groups, keep

    def bind(self, logits):
        _need_cuda(logits, self.correction)
        _need_f32(logits, self.correction)
        return _lib.Router(logits=_ptr(logits), correction=_ptr(self.correction), ld=logits.shape[-1], experts=self.experts, top=self.top,
                           groups=self.groups, keep=self.keep)


def moe_gemv(x, logits, router, w_gate_up, w_down):
    """Mixture output fp32 [N] of one token (two launches).  w_gate_up [experts, 2 ff, K] interleaved by 16 rows,
    w_down [experts, N, ff]."""
    lib = _lib.load_dense_library()
    _need_cuda(x, w_gate_up, w_down)
    _same("moe_gemv", w_gate_up, x, w_down)
    E, ff2, K = w_gate_up.shape
    ff, N, top = ff2 // 2, w_down.shape[1], router.top
    if x.numel() != K or tuple(w_down.shape) != (E, N, ff) or E != router.experts:
        raise ValueError("moe_gemv: shapes of x and the experts do not match")
    dev = x.device
    h = torch.empty((top, ff), dtype=x.dtype, device=dev)
    ids = torch.empty((top,), dtype=torch.int32, device=dev)
    wts = torch.empty((top,), dtype=torch.float32, device=dev)
    y = torch.empty((N,), dtype=torch.float32, device=dev)
    r = router.bind(logits)
    dt = dtype_code(x)
    _lib.check_dense(lib.dlm_moe_gate_up_gemv(dt, ctypes.byref(r), _ptr(x), _ptr(w_gate_up), _ptr(h), _ptr(ids), _ptr(wts), K, ff, _stream()))
    _lib.check_dense(lib.dlm_moe_down_gemv(dt, _ptr(h), _ptr(w_down), _ptr(ids), _ptr(wts), _ptr(y), top, E, ff, N, _stream()))
    return y


def moe_select(logits, router):
    """(ids int32 [M, top], weights fp32 [M, top]) for router logits [M, ld]."""
    lib = _lib.load_dense_library()
    M = logits.shape[0]
    ids = torch.empty((M, router.top), dtype=torch.int32, device=logits.device)
    wts = torch.empty((M, router.top), dtype=torch.float32, device=logits.device)
    r = router.bind(logits)
    _lib.check_dense(lib.dlm_moe_select(ctypes.byref(r), M, _ptr(ids), _ptr(wts), _stream()))
    return ids, wts


def moe_rows(h, logits, router, w_gate_up, w_down):
    """Chosen experts' outputs in the element type [M * top, N] (row token * top + slot) and the router weights [M, top]."""
    lib = _lib.load_dense_library()
    _need_cuda(h, w_gate_up, w_down)
    _same("moe_rows", w_gate_up, h, w_down)
    E, ff2, K = w_gate_up.shape
    ff, N, top = ff2 // 2, w_down.shape[1], router.top
    if h.shape[1] != K or tuple(w_down.shape) != (E, N, ff) or E != router.experts or logits.shape[0] != h.shape[0]:
        raise ValueError("moe_rows: shapes of the rows and the experts do not match")
    M, dev, dt = h.shape[0], h.device, dtype_code(h)
    ids, wts = moe_select(logits, router)
    entries = M * top
    tile_rows = lib.dlm_gemm_tile_rows(dt, entries // E, max(ff2, N), E)
    n_tiles = lib.dlm_moe_max_tiles(entries, E, tile_rows)
    order = torch.empty((entries,), dtype=torch.int32, device=dev)
    tiles = torch.empty((n_tiles + 1, 4), dtype=torch.int32, device=dev)
    _lib.check_dense(lib.dlm_moe_plan(_ptr(ids), entries, E, tile_rows, _ptr(order), _ptr(tiles), _stream()))
    act = torch.empty((entries, ff), dtype=h.dtype, device=dev)
    out = torch.empty((entries, N), dtype=h.dtype, device=dev)
    common = dict(tiles=_ptr(tiles), order=_ptr(order), M=entries, n_tiles=n_tiles, tile_rows=tile_rows)
    g = _lib.GemmArgs(a=_ptr(h), w=_ptr(w_gate_up), out=_ptr(act), lda=K, ldo=ff, w_stride=ff2 * K, N=ff2, K=K, epilogue=OUT_SWIGLU, gather=top,
                      **common)
    _lib.check_dense(lib.dlm_gemm(dt, ctypes.byref(g), _stream()))
    g = _lib.GemmArgs(a=_ptr(act), w=_ptr(w_down), out=_ptr(out), lda=ff, ldo=N, w_stride=N * ff, N=N, K=ff, epilogue=OUT_ELEM, gather=0, **common)
    _lib.check_dense(lib.dlm_gemm(dt, ctypes.byref(g), _stream()))
    return out, wts


class LatentSpec:
    """Sizes of one latent attention: true and padded."""

    __slots__ = ("heads", "dim", "rot", "vdim", "rank", "scale", "dim_p", "rot_p", "vdim_p", "rank_p", "shape")

    def __init__(self, heads, dim, rot, vdim, rank, scale):
        self.heads, self.dim, self.rot, self.vdim, self.rank, self.scale = heads, dim, rot, vdim, rank, scale
        self.dim_p, self.rot_p, self.vdim_p = pad_to(dim, HEAD_PAD), pad_to(rot, HEAD_PAD), pad_to(vdim, HEAD_PAD)
        self.rank_p = pad_to(rank, KP)
        self.shape = _lib.LatentShape(heads=heads, dim=self.dim_p, rot=self.rot_p, vdim=self.vdim_p, rank=self.rank_p, rot_pairs=rot // 2,
                                      true_rank=rank, scale=scale)

    @property
    def cache_width(self):
        return self.rank_p + self.rot_p

    @property
    def out_width(self):
        """Columns of the attention output: the heads, up to a whole input length of the next product."""
        return pad_to(self.heads * self.vdim_p, KP)

    def decode_supported(self, dtype):
        return bool(_lib.load_dense_library().dlm_latent_decode_supported(dtype_code(dtype), ctypes.byref(self.shape)))

    def prefill_supported(self, dtype):
        return bool(_lib.load_dense_library().dlm_latent_prefill_supported(dtype_code(dtype), ctypes.byref(self.shape)))


def _latent_rows(spec, proj, kv_off, gate_off, lut, kv_norm, eps, cache, M, pos, pos_dev):
    _need_cuda(proj, lut, cache)
    _same("latent attention", cache, proj)
    _need_f32(lut, kv_norm)
    if cache.shape[1] != spec.cache_width or lut.shape[1:] != (spec.rot // 2, 2):
        raise ValueError("latent attention: the cache or the rotation table has another width")
    if pos_dev is None and (pos + M > cache.shape[0] or pos + M > lut.shape[0]):
        raise ValueError(f"latent attention: positions {pos} .. {pos + M - 1} do not fit a cache of {cache.shape[0]} rows")
    return _lib.LatentRows(proj=_ptr(proj), lut=_ptr(lut), kv_norm=_opt(kv_norm), cache=_ptr(cache), pos_dev=_opt(pos_dev), ld=proj.shape[-1],
                           kv_off=kv_off, gate_off=gate_off, M=M, pos=pos, eps=eps)


def _attn_out(spec, M, like):
    exact = spec.out_width == spec.heads * spec.vdim_p
    return (torch.empty if exact else torch.zeros)((M, spec.out_width), dtype=like.dtype, device=like.device)


def latent_attention_rows(spec, proj, kv_off, gate_off, lut, kv_norm, eps, cache, pos, w_ukv, sink):
    """Gated attention output [M, out_width] of a long portion at positions pos ..: queries rotated (in place in proj),
    cache rows appended, keys and values of all cached rows expanded, causal attention."""
    lib = _lib.load_dense_library()
    M, dt = proj.shape[0], dtype_code(proj)
    r = _latent_rows(spec, proj, kv_off, gate_off, lut, kv_norm, eps, cache, M, pos, None)
    _need_cuda(w_ukv, sink)
    if tuple(w_ukv.shape) != (spec.heads * (spec.dim_p + spec.vdim_p), spec.rank_p):
        raise ValueError("latent attention: the key / value projection has another shape")
    _lib.check_dense(lib.dlm_latent_prepare(dt, ctypes.byref(spec.shape), ctypes.byref(r), _stream()))
    kv = gemm(cache, w_ukv, rows=pos + M)
    out = _attn_out(spec, M, proj)
    _lib.check_dense(lib.dlm_latent_prefill(dt, ctypes.byref(spec.shape), ctypes.byref(r), _ptr(kv), kv.shape[1], _ptr(sink), _ptr(out), out.shape[1],
                                            _stream()))
    return out


def latent_splits(spec, M, total):
    """How many workgroups share the keys of 16 rows.  A workgroup's time grows with its blocks of 32 keys, the merge's with
    the splits and rows: the square root balances them (constant measured at 16, 32 and 128 heads, 2k to 128k keys)."""
    rows, blocks = M * spec.heads, (total + 31) // 32
    return max(1, min(256, 512 // ((rows + 15) // 16), blocks, round((512 * blocks / rows) ** 0.5)))


def latent_attention_absorbed(spec, proj, kv_off, gate_off, lut, kv_norm, eps, cache, pos, w_ukv, sink, pos_dev=None, nsplit=None):
    """The same for one token or a short portion, on the latents themselves (proj [M, ld] or [ld]).  pos_dev: the
    position lies on the device (nsplit then has to be given)."""
    lib = _lib.load_dense_library()
    M = 1 if proj.dim() == 1 else proj.shape[0]
    dt, dev = dtype_code(proj), proj.device
    r = _latent_rows(spec, proj, kv_off, gate_off, lut, kv_norm, eps, cache, M, pos, pos_dev)
    _need_cuda(w_ukv, sink)
    if tuple(w_ukv.shape) != (spec.heads * (spec.dim_p + spec.vdim_p), spec.rank_p):
        raise ValueError("latent attention: the key / value projection has another shape")
    w_uk, w_uv = w_ukv[:spec.heads * spec.dim_p], w_ukv[spec.heads * spec.dim_p:]
    if nsplit is None:
        nsplit = latent_splits(spec, M, pos + M)
    rows = M * spec.heads
    qa = torch.empty((rows, spec.cache_width), dtype=proj.dtype, device=dev)
    part_o = torch.empty((rows, nsplit, spec.rank_p), dtype=torch.float32, device=dev)
    part_ml = torch.empty((rows, nsplit, 2), dtype=torch.float32, device=dev)
    out = _attn_out(spec, M, proj)
    s, rr = ctypes.byref(spec.shape), ctypes.byref(r)
    _lib.check_dense(lib.dlm_latent_absorb(dt, s, rr, _ptr(w_uk), _ptr(qa), _stream()))
    _lib.check_dense(lib.dlm_latent_decode(dt, s, rr, _ptr(qa), nsplit, _ptr(part_o), _ptr(part_ml), _stream()))
    _lib.check_dense(lib.dlm_latent_combine(dt, s, rr, nsplit, _ptr(part_o), _ptr(part_ml), _ptr(sink), _ptr(w_uv), _ptr(out), out.shape[1],
                                            _stream()))
    return out


class HeadSpec:
    """Sizes of one windowed attention of grouped heads: true and padded."""

    __slots__ = ("heads", "kv_heads", "dim", "vdim", "window", "scale", "out_scale", "dim_p", "vdim_p")

    def __init__(self, heads, kv_heads, dim, vdim, window, scale, out_scale=1.0):
        self.heads, self.kv_heads, self.dim, self.vdim, self.window, self.scale, self.out_scale = heads, kv_heads, dim, vdim, window, scale, out_scale
        self.dim_p, self.vdim_p = pad_to(dim, HEAD_PAD), pad_to(vdim, HEAD_PAD)

    @property
    def proj_width(self):
        return (self.heads + self.kv_heads) * self.dim_p + self.kv_heads * self.vdim_p

    def ring(self, capacity, portion):
        """Cache rows for a sequence of `capacity` tokens that come in portions of at most `portion`."""
        rows = capacity if portion is None else min(capacity, self.window - 1 + portion)
        return pad_to(rows, 64)

    def shape(self, ring):
        return _lib.HeadShape(heads=self.heads, kv_heads=self.kv_heads, dim=self.dim_p, vdim=self.vdim_p, true_dim=self.dim,
                              window=min(self.window, 1 << 30), ring=ring, scale=self.scale, out_scale=self.out_scale)

    def decode_supported(self, dtype):
        return bool(_lib.load_dense_library().dlm_head_decode_supported(dtype_code(dtype), ctypes.byref(self.shape(64))))

    def prefill_supported(self, dtype):
        return bool(_lib.load_dense_library().dlm_head_prefill_supported(dtype_code(dtype), ctypes.byref(self.shape(64))))


def head_splits(spec, M, total):
    """How many workgroups share the keys of 16 query rows of a key / value head: enough of them to fill the GPU twice, as far as
    there are blocks of 32 keys."""
    tiles = spec.kv_heads * ((M * (spec.heads // spec.kv_heads) + 15) // 16)
    blocks = (min(total, spec.window + M - 1) + 31) // 32 + 1
    return max(1, min(256, 512 // tiles, blocks))


def head_attention(spec, proj, off, q_norm, k_norm, eps, cache, pos, out, pos_dev=None, nsplit=None, rows_form=False):
    """Windowed attention of the rows of proj [M, ld] (q, k, v from column `off` on) at positions pos .. into the first columns of
    out [M, ldo]; their keys and values are appended to cache [kv_heads, ring, dim + vdim].  rows_form: the kernel for many rows."""
    lib = _lib.load_dense_library()
    M, dt = proj.shape[0], dtype_code(proj)
    s, r, q = _head_args(spec, proj, off, q_norm, k_norm, eps, cache, pos, out, pos_dev)
    _lib.check_dense(lib.dlm_head_prepare(dt, s, r, _ptr(q), _stream()))
    if rows_form:
        _lib.check_dense(lib.dlm_head_prefill(dt, s, r, _ptr(q), out.data_ptr(), out.stride(0), _stream()))
        return
    nsplit, part_o, part_ml = _head_parts(spec, M, pos, nsplit, proj.device)
    _lib.check_dense(lib.dlm_head_decode(dt, s, r, _ptr(q), nsplit, _ptr(part_o), _ptr(part_ml), _stream()))
    _lib.check_dense(lib.dlm_head_merge(dt, s, r, nsplit, _ptr(part_o), _ptr(part_ml), out.data_ptr(), out.stride(0), _stream()))


def _head_args(spec, proj, off, q_norm, k_norm, eps, cache, pos, out, pos_dev):
    _need_cuda(cache, q_norm, k_norm)
    _same("head attention", cache, proj, out)
    _need_f32(q_norm, k_norm)
    M = proj.shape[0]
    if tuple(cache.shape[::2]) != (spec.kv_heads, spec.dim_p + spec.vdim_p) or out.shape[0] != M or proj.shape[1] < off + spec.proj_width:
        raise ValueError("head attention: the cache, the projections or the output have another shape")
    if q_norm.numel() != spec.dim_p or k_norm.numel() != spec.dim_p:
        raise ValueError(f"head attention: the norm weights must have {spec.dim_p} elements")
    s = spec.shape(cache.shape[1])
    r = _lib.HeadRows(proj=proj.data_ptr(), q_norm=_ptr(q_norm), k_norm=_ptr(k_norm), cache=_ptr(cache), pos_dev=_opt(pos_dev), ld=proj.stride(0), off=off, M=M,
                      pos=pos, eps=eps)
    q = torch.empty((M * spec.heads, spec.dim_p), dtype=proj.dtype, device=proj.device)
    return ctypes.byref(s), ctypes.byref(r), q


def _head_parts(spec, M, pos, nsplit, device):
    if nsplit is None:
        nsplit = head_splits(spec, M, pos + M)
    part_o = torch.empty((M * spec.heads, nsplit, spec.vdim_p), dtype=torch.float32, device=device)
    return nsplit, part_o, torch.empty((M * spec.heads, nsplit, 2), dtype=torch.float32, device=device)


class StateSpec:
    """Sizes of one linear recurrence over a matrix state per head: true and padded."""

    __slots__ = ("heads", "k_heads", "dim", "vdim", "dim_p", "vdim_p")

    def __init__(self, heads, k_heads, dim, vdim):
        self.heads, self.k_heads, self.dim, self.vdim = heads, k_heads, dim, vdim
        self.dim_p, self.vdim_p = pad_to(dim, STATE_PAD), pad_to(vdim, HEAD_PAD)

    def supported(self):
        return self.dim_p <= STATE_MAX

    @property
    def qk_width(self):
        return self.k_heads * self.dim_p

    @property
    def v_width(self):
        return self.heads * self.vdim_p

    @property
    def channels(self):
        return 2 * self.qk_width + self.v_width

    def new_state(self, device):
        return torch.zeros((self.heads, self.vdim_p, self.dim_p), dtype=torch.float32, device=device)


def short_conv(spec, proj, off, w, history, pos, q_scale, unit_eps, pos_dev=None):
    """(act [M, channels], factors [M, 2 k_heads]) of the channels of proj [M, ld] from column `off` on; w fp32 [taps, channels],
    history [taps, channels] is brought forward."""
    lib = _lib.load_dense_library()
    c, act, factors = _conv_args(spec, proj, off, w, history, pos, q_scale, unit_eps, pos_dev)
    _lib.check_dense(lib.dlm_short_conv(dtype_code(proj), c, _ptr(act), _stream()))
    return act, factors


def conv_products(spec, proj, off, w, history, pos, q_scale, unit_eps, low_a, w_a, low_b, w_b, pos_dev=None):
    """short_conv of one token, and in the same launch the products w_a low_a (fp32) and w_b low_b of short vectors.  Returns (act, factors,
    the two results [1, N])."""
    lib = _lib.load_dense_library()
    _need_cuda(w_a, w_b)
    _same("conv_products", proj, low_a, w_a, low_b, w_b)
    if low_a.numel() != w_a.shape[1] or low_b.numel() != w_b.shape[1]:
        raise ValueError("conv_products: shapes of the products do not match")
    c, act, factors = _conv_args(spec, proj, off, w, history, pos, q_scale, unit_eps, pos_dev)
    out_a = torch.empty((1, w_a.shape[0]), dtype=torch.float32, device=proj.device)
    out_b = torch.empty((1, w_b.shape[0]), dtype=proj.dtype, device=proj.device)
    a, b = (_lib.ShortProduct(w=_ptr(m), x=x.data_ptr(), out=_ptr(o), K=m.shape[1], N=m.shape[0]) for m, x, o in ((w_a, low_a, out_a), (w_b, low_b, out_b)))
    _lib.check_dense(lib.dlm_conv_products(dtype_code(proj), c, _ptr(act), ctypes.byref(a), ctypes.byref(b), _stream()))
    return act, factors, out_a, out_b


def _conv_args(spec, proj, off, w, history, pos, q_scale, unit_eps, pos_dev):
    _need_cuda(w, history)
    _need_f32(w)
    _same("short_conv", history, proj)
    M, C = proj.shape[0], spec.channels
    if w.shape[1] != C or history.shape != w.shape or proj.shape[1] < off + C:
        raise ValueError(f"short_conv: projections, filters and history must have {C} channels")
    act = torch.empty((M, C), dtype=proj.dtype, device=proj.device)
    factors = torch.empty((M, 2 * spec.k_heads), dtype=torch.float32, device=proj.device)
    c = _lib.ShortConvArgs(proj=proj.data_ptr(), w=_ptr(w), history=_ptr(history), factors=_ptr(factors), pos_dev=_opt(pos_dev), ld=proj.stride(0),
                           k_heads=spec.k_heads, heads=spec.heads, dim=spec.dim_p, vdim=spec.vdim_p, taps=w.shape[0], off=off, M=M, pos=pos, q_scale=q_scale,
                           unit_eps=unit_eps)
    return ctypes.byref(c), act, factors


# Up to this many tokens a portion goes through a recurrence token by token.
STEPS_MAX_TOKENS = 16


def recurrence(spec, qkv, offsets, state, pos, log2_decay=None, z=None, a_log=None, dt_bias=None, factors=None, beta=None, pos_dev=None, chunks=None):
    """Read-outs fp32 [M, heads * vdim_p] of the tokens of qkv [M, ld] (q, k, v at the column `offsets`); `state` is brought forward.
    log2_decay [heads]: a decay per head; z [M, heads * dim_p] with a_log, dt_bias, factors and beta [M, >= heads]: a decay per channel
    and the delta rule.  chunks: which form to run (default: by the number of tokens)."""
    lib = _lib.load_dense_library()
    a, o = _recurrence_args(spec, qkv, offsets, state, pos, log2_decay, z, a_log, dt_bias, factors, beta, pos_dev)
    nbytes = lib.dlm_recurrence_chunk_bytes(a)
    if chunks is None:
        chunks = qkv.shape[0] > STEPS_MAX_TOKENS and nbytes > 0
    if chunks:
        work = torch.empty((nbytes,), dtype=torch.uint8, device=qkv.device)
        _lib.check_dense(lib.dlm_recurrence_chunks(dtype_code(qkv), a, _ptr(work), _ptr(o), _stream()))
    else:
        _lib.check_dense(lib.dlm_recurrence_steps(dtype_code(qkv), a, _ptr(o), _stream()))
    return o


def _recurrence_args(spec, qkv, offsets, state, pos, log2_decay, z, a_log, dt_bias, factors, beta, pos_dev):
    _need_cuda(state)
    _need_f32(state, log2_decay, z, a_log, dt_bias, factors)
    M, H = qkv.shape[0], spec.heads
    if tuple(state.shape) != (H, spec.vdim_p, spec.dim_p) or qkv.stride(1) != 1:
        raise ValueError("recurrence: the state has another shape")
    if z is None:
        if log2_decay.numel() != H:
            raise ValueError(f"recurrence: {H} decays")
    elif tuple(z.shape) != (M, H * spec.dim_p) or a_log.numel() != H or dt_bias.numel() != H * spec.dim_p or tuple(factors.shape) != (M, 2 * spec.k_heads) \
            or beta.shape[0] != M or beta.shape[1] < H or beta.dtype != qkv.dtype:
        raise ValueError("recurrence: shapes of the decay, the factors or beta do not match")
    a = _lib.RecurrenceArgs(qkv=qkv.data_ptr(), log2_decay=_opt(log2_decay), z=_opt(z), a_log=_opt(a_log), dt_bias=_opt(dt_bias), factors=_opt(factors),
                            beta=_opt(beta), state=_ptr(state), pos_dev=_opt(pos_dev), ld=qkv.stride(0), ld_beta=0 if beta is None else beta.stride(0),
                            k_heads=spec.k_heads, heads=H, dim=spec.dim_p, vdim=spec.vdim_p, q_off=offsets[0], k_off=offsets[1], v_off=offsets[2], M=M, pos=pos)
    return ctypes.byref(a), torch.empty((M, spec.v_width), dtype=torch.float32, device=qkv.device)


def attention_and_state(heads, state, proj, off, q_norm, k_norm, eps, cache, offsets, memory, log2_decay, pos, norm_w, true_cols, gate_off, out, pos_dev=None,
                        nsplit=None):
    """One token through windowed attention (`heads`, as head_attention with the keys split) and, beside it in the same three launches, a
    recurrence with a decay per head (`state`, as recurrence) with the norm and gate of its read-outs: out [1, >=] = [attention | read-outs]."""
    lib = _lib.load_dense_library()
    if proj.shape[0] != 1 or norm_w.numel() != state.v_width or out.shape[1] < heads.heads * heads.vdim_p + state.v_width \
            or proj.shape[1] < gate_off + state.v_width:
        raise ValueError("attention_and_state: one token, and a norm weight, a gate and an output of the read-outs' width")
    _need_cuda(norm_w)
    _need_f32(norm_w)
    dt = dtype_code(proj)
    s, r, q = _head_args(heads, proj, off, q_norm, k_norm, eps, cache, pos, out, pos_dev)
    a, o = _recurrence_args(state, proj, offsets, memory, pos, log2_decay, None, None, None, None, None, pos_dev)
    _lib.check_dense(lib.dlm_head_state_begin(dt, s, r, _ptr(q), a, _ptr(o), _stream()))
    nsplit, part_o, part_ml = _head_parts(heads, 1, pos, nsplit, proj.device)
    _lib.check_dense(lib.dlm_head_decode(dt, s, r, _ptr(q), nsplit, _ptr(part_o), _ptr(part_ml), _stream()))
    _lib.check_dense(lib.dlm_head_state_end(dt, s, r, nsplit, _ptr(part_o), _ptr(part_ml), out.data_ptr(), _ptr(o), _ptr(norm_w), proj[:, gate_off:].data_ptr(),
                                            state.v_width, true_cols, eps, out[:, heads.heads * heads.vdim_p:].data_ptr(), _stream()))


def gated_norm(o, w, eps, groups, true_cols, gate, out):
    """out[:, :groups * cols] = o / rms * w * sigmoid(gate) with the mean over the true_cols of a group's columns; w fp32 [cols]."""
    lib = _lib.load_dense_library()
    _need_cuda(o, w)
    _need_f32(o, w)
    _same("gated_norm", out, gate)
    M, cols = o.shape[0], o.shape[1] // groups
    if w.numel() != cols or out.shape[0] != M or gate.shape[0] != M or min(out.shape[1], gate.shape[1]) < groups * cols:
        raise ValueError("gated_norm: shapes do not match")
    _lib.check_dense(lib.dlm_gated_norm(dtype_code(gate), _ptr(o), _ptr(w), gate.data_ptr(), gate.stride(0), out.data_ptr(), out.stride(0), M, groups, cols,
                                        true_cols, eps, _stream()))
