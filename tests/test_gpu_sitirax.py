"""The kernels of models with norms on their inputs, windowed grouped attention and linear recurrences one by one, and the Sitirax
model as a whole on the GPU, against the plain float64 implementation (oracle/sitirax.py)."""
import json
import os
import subprocess

import numpy as np
import pytest
import torch

from helpers import SITIRAX_MIXED, sitirax_config, sitirax_delta, sitirax_parallel, sitirax_weights, sitirax_write
from oracle import sitirax as ost

pytestmark = pytest.mark.gpu
F32, BF16 = torch.float32, torch.bfloat16
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


@pytest.fixture(scope="module")
def dense():
    from air_hip import dense as d
    return d


def say(*a):
    print(*a, flush=True)


def rounded(a):
    """The nearest values that bf16 holds, float64."""
    return torch.from_numpy(np.asarray(a, np.float32)).to(BF16).double().numpy()


def gpu(a, dtype=F32):
    return torch.from_numpy(np.ascontiguousarray(a)).to(dtype).cuda()


def host(t):
    return t.float().cpu().numpy().astype(np.float64)


def close(got, want, dtype, what="", f32=2e-5, bf16=1.2e-2):
    """Every error within tolerance x (the rms of what is expected + the expected element itself)."""
    got, want = host(got) if isinstance(got, torch.Tensor) else got, np.asarray(want, np.float64)
    err = np.abs(got - want) / (np.sqrt(np.mean(want ** 2)) + np.abs(want) + 1e-30)
    assert err.max() <= (f32 if dtype == F32 else bf16), (what, err.max(), np.unravel_index(err.argmax(), err.shape))


def close_rows(got, want, what=""):
    """bf16 logits: the rms error of every position is small."""
    d = host(got) - want
    err = np.sqrt((d ** 2).mean(-1) / (want ** 2).mean())
    assert err.max() < 0.06 and np.median(err) < 0.025, (what, np.sort(err)[-8:], np.median(err))


# ---- products and rows ---------------------------------------------------------------------------------------------------
def interleaved(gate, up):
    ff, K = gate.shape
    return np.stack([gate.reshape(ff // 16, 16, K), up.reshape(ff // 16, 16, K)], axis=1).reshape(2 * ff, K)


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("ff,K,width", [(16, 64, 40), (592, 576, 530), (48, 1088, 1088), (2064, 2112, 2100), (64, 4608, 4600)])
def test_normed_intake_activations_and_gates(dense, dtype, ff, K, width):
    say("normed intake", dtype, ff, K)
    rng, eps = np.random.default_rng(ff), 1e-3
    vec = lambda: np.where(np.arange(K) < width, rng.standard_normal(K), 0.0).astype(np.float32)
    res, y, nw = vec() * 3, vec(), vec()
    gate, up = (rounded(rng.standard_normal((ff, K)) * K ** -0.5) for _ in range(2))
    w = interleaved(gate, up)
    W = gpu(w, dtype)
    emb = rounded(rng.standard_normal((7, K)) * (np.arange(K) < width))
    norm = lambda v: v / np.sqrt((v ** 2).sum() / width + eps) * nw
    token = torch.tensor([5], dtype=torch.int32, device="cuda")
    for s, v in ((dense.Sum(gpu(res), gpu(y)), res.astype(np.float64) + y), (dense.Sum(gpu(res)), res.astype(np.float64)),
                 (dense.Sum(token=token, embed=gpu(emb, dtype), scale=0.7), emb[5] * 0.7)):
        x = norm(v)
        out, kept = dense.gemv_normed(s, gpu(nw), eps, width, W)
        close(kept, v, F32, "sum", f32=1e-6)
        close(out, w @ x, dtype, "plain")
        out, kept = dense.gemv_normed(s, gpu(nw), eps, width, W, keep=False, out_f32=True)
        assert kept is None
        close(out, w @ x, dtype, "fp32")
        a, b = 16, max(16, ff)
        want = w @ x
        want[a:b] = ost.silu(want[a:b])
        close(dense.gemv_normed(s, gpu(nw), eps, width, W, silu=(a, b))[0], want, dtype, "silu")
        close(dense.gemv_normed(s, gpu(nw), eps, width, W, gate=dense.GATE_GELU)[0], ost.gelu_tanh(gate @ x) * (up @ x), dtype, "gelu", bf16=2e-2)
        close(dense.gemv_normed(s, gpu(nw), eps, width, W, gate=dense.GATE_SILU)[0], ost.silu(gate @ x) * (up @ x), dtype, "silu gate", bf16=2e-2)
    keys = dense.new_keys(W)
    logits, _ = dense.gemv_normed(dense.Sum(gpu(res), gpu(y)), gpu(nw), eps, width, W, out_f32=True, keys=keys, n_valid=2 * ff - 5, keep=False)
    tok = torch.zeros((1,), dtype=torch.int32, device="cuda")
    dense.argmax(keys, tok)
    assert int(tok) == int(logits[:2 * ff - 5].argmax())


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("M,ff,K", [(2, 16, 64), (33, 80, 128), (300, 528, 384)])
def test_products_with_activations(dense, dtype, M, ff, K):
    say("gemm activations", dtype, M, ff, K)
    rng = np.random.default_rng(M)
    a, gate, up = rounded(rng.standard_normal((M, K))), *(rounded(rng.standard_normal((ff, K)) * K ** -0.5) for _ in range(2))
    w = interleaved(gate, up)
    A, W = gpu(a, dtype), gpu(w, dtype)
    close(dense.gemm(A, W, gate=dense.GATE_GELU), ost.gelu_tanh(a @ gate.T) * (a @ up.T), dtype, "gelu", bf16=2e-2)
    close(dense.gemm(A, W, gate=dense.GATE_SILU), ost.silu(a @ gate.T) * (a @ up.T), dtype, "silu gate", bf16=2e-2)
    want = a @ w.T
    want[:, 16:ff] = ost.silu(want[:, 16:ff])
    close(dense.gemm(A, W, silu=(16, ff)), want, dtype, "silu")


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_residual_rows_with_the_norm_of_the_next_sublayer(dense, dtype):
    rng = np.random.default_rng(2)
    M, K, width, eps = 5, 192, 150, 1e-2
    mask = np.arange(K) < width
    emb, nw = rounded(rng.standard_normal((11, K)) * mask), (rng.standard_normal(K) * mask).astype(np.float32)
    norm = lambda v: v / np.sqrt((v ** 2).sum(-1, keepdims=True) / width + eps) * nw
    ids = [3, 0, 10, 3, 7]
    res = torch.full((M, K), float("nan"), device="cuda")
    h = dense.add_norm_rows(res, None, gpu(nw), eps, width, dtype, tokens=torch.tensor(ids, dtype=torch.int32, device="cuda"), embed=gpu(emb, dtype), scale=0.3)
    x = emb[ids] * 0.3
    close(res, x, F32, f32=1e-6)
    close(h, norm(x), dtype)
    y = rng.standard_normal((M, K)).astype(np.float32) * mask
    close(dense.add_norm_rows(res, gpu(y), gpu(nw), eps, width, dtype), norm(x + y), dtype)
    close(res, x + y, F32, f32=1e-6)
    close(dense.add_norm_rows(res, None, gpu(nw), eps, width, dtype), norm(x + y), dtype)
    assert dense.add_norm_rows(res, gpu(y), None, eps, width, dtype) is None
    close(res, x + 2 * y, F32, f32=1e-6)


# ---- windowed attention ----------------------------------------------------------------------------------------------------
HEAD_SIZES = [   # heads, kv_heads, dim, vdim, window
    (4, 2, 24, 40, 37), (3, 3, 64, 64, 64), (8, 2, 128, 128, 65), (6, 1, 40, 200, 1), (2, 2, 288, 16, 100), (16, 4, 64, 64, 1000), (34, 2, 32, 32, 33),
]


class Heads:
    """Random inputs of one windowed attention over T positions; `far`: (query, key) pairs whose score stands out by ~30 for every
    head, by the first two channels."""

    OFF = 16

    def __init__(self, dense, sizes, T, dtype, ring, seed=0, far=(), out_scale=0.8):
        H, G, D, V, window = sizes
        self.dense, self.T, self.dtype, self.sizes = dense, T, dtype, sizes
        self.spec = s = dense.HeadSpec(H, G, D, V, window, 30.0 / D, out_scale)     # queries and keys are of length sqrt(D)
        self.eps = 1e-5
        rng = np.random.default_rng(seed)
        q, k = rng.standard_normal((T, H, D)) * 3, rng.standard_normal((T, G, D)) * 0.5
        q, k = q - q.mean(-1, keepdims=True), k - k.mean(-1, keepdims=True)
        for i, j in far:
            u = rng.standard_normal(D)
            k[j], q[i] = u, 5 * u
        self.q, self.k, self.v = rounded(q), rounded(k), rounded(rng.standard_normal((T, G, V)))
        self.qn, self.kn = 1 + 0.1 * rng.standard_normal(D).astype(np.float32), 1 + 0.1 * rng.standard_normal(D).astype(np.float32)
        p = np.full((T, self.OFF + s.proj_width + 8), 9.0)
        pad = lambda a, n: np.pad(a, ((0, 0), (0, 0), (0, n - a.shape[2]))).reshape(T, -1)
        p[:, self.OFF:self.OFF + s.proj_width] = np.concatenate([pad(self.q, s.dim_p), pad(self.k, s.dim_p), pad(self.v, s.vdim_p)], 1)
        self.proj = gpu(p, dtype)
        vec = lambda a: gpu(np.pad(a, (0, s.dim_p - D)))
        self.norms = vec(self.qn), vec(self.kn)
        self.cache = torch.full((G, ring, s.dim_p + s.vdim_p), float("nan"), dtype=dtype, device="cuda")   # rows not yet written must not be read

    def want(self):
        s = self.spec
        q, k = ost.rms_norm(self.q, self.qn, self.eps), ost.rms_norm(self.k, self.kn, self.eps)
        if self.dtype == BF16:
            q, k = rounded(q), rounded(k)                    # what is kept of them
        return ost.window_attention(q, k, self.v, range(self.T), s.scale, s.window).reshape(self.T, -1) * s.out_scale

    def run(self, form, a, b, **kw):
        s = self.spec
        out = torch.full((b - a, s.heads * s.vdim_p + 24), 7.0, dtype=self.dtype, device="cuda")
        self.dense.head_attention(s, self.proj[a:b], self.OFF, *self.norms, self.eps, self.cache, kw.pop("pos", a), out, rows_form=form == "rows", **kw)
        assert bool((out[:, s.heads * s.vdim_p:] == 7.0).all())
        out = out[:, :s.heads * s.vdim_p].reshape(b - a, s.heads, s.vdim_p)
        assert not bool(out[..., s.vdim:].any())
        return out[..., :s.vdim].reshape(b - a, -1)


def borders(window, T):
    """Pairs just inside and just outside the window, around the edges of blocks of 32 and 64 keys, and near ones."""
    pairs = [p for i in (max(window, 20), 71, 98, 130, T - 10) for p in ((i - 1, i - window), (i + 2, i + 2 - window))]
    out = []
    for i, j in pairs + [(45, 13), (64, 31), (104, 62), (160, 129), (147, 147)]:      # a query and a key belong to one pair
        if 0 <= j < T and 0 <= i < T and not any(i == a or j == b for a, b in out):
            out.append((i, j))
    return out


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("sizes", HEAD_SIZES)
@pytest.mark.parametrize("form", ["rows", "splits"])
def test_windowed_attention(dense, dtype, sizes, form):
    T, window = 200, sizes[4]
    say("windowed attention", dtype, sizes, form)
    far = borders(window, T)
    x = Heads(dense, sizes, T, dtype, 256, seed=sizes[0], far=far)
    want = x.want()
    tol = dict(f32=1e-4, bf16=3e-2)
    for i, j in far[:2]:                                     # inside the window the far key's value is what comes out, outside it is not
        inside = i - j < window
        assert inside == (np.abs(want[i, :sizes[3]] - 0.8 * x.v[j, 0]).max() < 0.05), (i, j)
    whole = x.run(form, 0, T)
    close(whole, want, dtype, "whole", **tol)
    for i, _ in far:                                         # each row against its own size
        close(whole[i], want[i], dtype, i, **tol)
    x.cache.fill_(float("nan"))
    cuts = (0, 3, 70, 72, 135, T)
    parts = torch.cat([x.run(form, a, b) for a, b in zip(cuts, cuts[1:])])
    close(parts, want, dtype, "portions", **tol)
    for i, _ in far:
        close(parts[i], want[i], dtype, i, **tol)


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("sizes", [(4, 2, 24, 40, 37), (8, 2, 128, 128, 65), (3, 3, 64, 64, 64), (2, 1, 32, 32, 1)])
def test_ring_of_rows_and_positions_on_the_device(dense, dtype, sizes):
    T, window = 330, sizes[4]
    ring = -(-(window - 1 + 40) // 64) * 64
    say("ring", dtype, sizes, ring)
    far = [(i, i - window + d) for i in (64, 127, 128, 129, 192, 255, 256, 300, 320) for d in (0, 1)]
    x = Heads(dense, sizes, T, dtype, ring, seed=5, far=far[::2] + far[1::4])
    want, tol = x.want(), dict(f32=1e-4, bf16=3e-2)
    for form in ("rows", "splits"):
        x.cache.fill_(float("nan"))
        got, i = [], 0
        for n in [40, 40, 7, 33, 40, 2, 30] + [40] * 10:
            if i < T:
                got.append(x.run(form, i, min(i + n, T)))
                i += n
        got = torch.cat(got)
        close(got, want, dtype, form, **tol)
        for i, _ in far:
            close(got[i], want[i], dtype, (form, i), **tol)
    x.cache.fill_(float("nan"))
    pos = torch.zeros((1,), dtype=torch.int32, device="cuda")
    got = []
    for i in range(T):
        pos.fill_(i)
        got.append(x.run("splits", i, i + 1, pos=0, pos_dev=pos, nsplit=(1, 2, 3, 7)[i % 4]))
    close(torch.cat(got), want, dtype, "token by token", **tol)


def test_a_ring_that_is_too_short_is_refused(dense):
    from air_hip import _lib

    x = Heads(dense, (2, 2, 32, 32, 100), 131, F32, 128)
    x.run("rows", 0, 100)
    with pytest.raises(_lib.DenseLmError):
        x.run("rows", 100, 131)


# ---- short convolution -------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("heads,k_heads,dim,vdim,taps", [(4, 2, 24, 40, 3), (3, 3, 72, 16, 1), (2, 1, 128, 128, 4), (5, 5, 200, 8, 7)])
def test_short_convolution(dense, dtype, heads, k_heads, dim, vdim, taps):
    say("short convolution", dtype, heads, dim, taps)
    T, off = 41, 8
    s = dense.StateSpec(heads, k_heads, dim, vdim)
    rng = np.random.default_rng(taps)
    x = {n: rounded(rng.standard_normal((T, h, d))) for n, h, d in (("q", k_heads, dim), ("k", k_heads, dim), ("v", heads, vdim))}
    w = {n: rounded(rng.standard_normal((a.shape[1], a.shape[2], taps))) for n, a in x.items()}
    padded = lambda n: s.vdim_p if n == "v" else s.dim_p
    grow = lambda a, n: np.pad(a, ((0, 0), (0, 0), (0, padded(n) - a.shape[2]))).reshape(a.shape[0], -1)
    proj = gpu(np.concatenate([np.full((T, off), 5.0)] + [grow(x[n], n) for n in "qkv"], 1), dtype)
    W = gpu(np.concatenate([grow(w[n].transpose(2, 0, 1), n) for n in "qkv"], 1))
    want = {n: ost.silu(ost.short_convolution(x[n].reshape(T, -1), w[n].reshape(-1, taps), np.zeros((taps - 1, x[n][0].size)))[0]).reshape(x[n].shape) for n in "qkv"}
    for cuts in ((0, T), (0, 1, 2, 3, 4, 5, 6, 7, 8, 9, 20, 21, T), (0, 2, 4, 7, 8, 12, 40, T)):
        history, pos = torch.full((taps, s.channels), float("nan"), dtype=dtype, device="cuda"), torch.zeros((1,), dtype=torch.int32, device="cuda")
        act, fac = [], []
        for a, b in zip(cuts, cuts[1:]):
            pos.fill_(a)
            kw = dict(pos=0, pos_dev=pos) if b - a == 1 and a % 2 else dict(pos=a)
            y, f = dense.short_conv(s, proj[a:b], off, W, history, q_scale=0.3, unit_eps=1e-6, **kw)
            act.append(y), fac.append(f)
        act, fac = host(torch.cat(act)), host(torch.cat(fac))
        at = 0
        for n, h, d in (("q", k_heads, dim), ("k", k_heads, dim), ("v", heads, vdim)):
            part = act[:, at:at + h * padded(n)].reshape(T, h, padded(n))
            close(part[..., :d], want[n], dtype, n)
            assert not part[..., d:].any()
            if n != "v":
                f = fac[:, k_heads * "qk".index(n):][:, :h]
                close(part[..., :d] * f[..., None], ost.unit(want[n]) * (0.3 if n == "q" else 1.0), dtype, "unit " + n)
            at += h * padded(n)


# ---- recurrences -----------------------------------------------------------------------------------------------------------------
class Recurrence:
    """Random inputs of one recurrence.  `far`: (query, key) pairs with a channel of their own, so that what the key wrote is
    read alone after a long way."""

    def __init__(self, dense, kind, heads, k_heads, dim, vdim, T, dtype, seed=0, far=(), strong=False):
        self.dense, self.kind, self.T, self.dtype = dense, kind, T, dtype
        self.spec = s = dense.StateSpec(heads, k_heads, dim, vdim)
        rng = np.random.default_rng(seed)
        q, k = rng.standard_normal((T, k_heads, dim)), rng.standard_normal((T, k_heads, dim)) * 0.3
        z = rng.standard_normal((T, heads, dim)) * (3.0 if strong else 1.0)
        bias, self.a_log = rng.standard_normal((heads, dim)) - 3.0, rng.standard_normal(heads) * 0.5 - 1.0
        if strong:
            bias[:, ::3] += 40.0                        # channels that are forgotten at once, beside others that stay
            z[5::11] += 60.0
        for n, (i, j) in enumerate(far):
            q[..., n], k[..., n] = 0.0, 0.0
            q[i], k[j] = 0.0, 0.0
            q[i, :, n], k[j, :, n] = 1.0, 1.0
            z[..., n], bias[:, n] = 0.0, -30.0            # this channel is not forgotten
        self.q, self.k, self.v, self.z, self.bias = rounded(q), rounded(k), rounded(rng.standard_normal((T, heads, vdim))), z.astype(np.float32), bias.astype(np.float32)
        self.beta = rounded(rng.standard_normal((T, heads)) * 2)
        self.decay = np.concatenate([[1.0, 0.0, 0.999, 0.5], rng.uniform(0.6, 1.0, heads)])[:heads]
        self.qs = dim ** -0.5
        pad = lambda a, n: np.pad(a, ((0, 0), (0, 0), (0, n - a.shape[2]))).reshape(T, -1)
        parts = [pad(self.q, s.dim_p), pad(self.k, s.dim_p), pad(self.v, s.vdim_p)]
        self.offsets = (8, 8 + s.qk_width, 8 + 2 * s.qk_width)
        self.qkv = gpu(np.concatenate([np.full((T, 8), 5.0)] + parts, 1), dtype)
        self.state = torch.full((heads, s.vdim_p, s.dim_p), float("nan"), device="cuda")      # not read at position 0
        if kind == "delta":
            f = lambda a: 1.0 / np.sqrt((a ** 2).sum(-1) + 1e-6)
            self.kw = dict(z=gpu(pad(self.z, s.dim_p)), a_log=gpu(self.a_log.astype(np.float32)), dt_bias=gpu(np.pad(self.bias, ((0, 0), (0, s.dim_p - dim))).reshape(-1)),
                           factors=gpu(np.concatenate([f(self.q) * self.qs, f(self.k)], 1).astype(np.float32)),
                           beta=gpu(np.pad(self.beta, ((0, 0), (0, 16 - heads % 16))), dtype))
        else:
            with np.errstate(divide="ignore"):
                self.kw = dict(log2_decay=gpu(np.maximum(np.log2(self.decay), -1e6).astype(np.float32)))

    def want(self):
        s = self.spec
        state = np.zeros((s.heads, s.dim, s.vdim))
        if self.kind == "delta":
            g = ost.channel_decay(self.z.astype(np.float64), self.a_log, self.bias.astype(np.float64))
            return ost.delta_rule(ost.unit(self.q) * self.qs, ost.unit(self.k), self.v, ost.sigmoid(self.beta), g, state), state
        return ost.lightning(self.q, self.k, self.v, self.decay, state), state

    def run(self, a, b, chunks, **kw):
        per_row = {n: t[a:b] for n, t in self.kw.items() if n in ("z", "factors", "beta")}
        o = self.dense.recurrence(self.spec, self.qkv[a:b], self.offsets, self.state, kw.pop("pos", a), chunks=chunks, **{**self.kw, **per_row}, **kw)
        s = self.spec
        o = o.reshape(b - a, s.heads, s.vdim_p)
        assert not bool(o[..., s.vdim:].any())
        return o[..., :s.vdim]

    def final(self):
        s = self.spec
        assert not bool(self.state[:, s.vdim:].any()) and not bool(self.state[:, :, s.dim:].any())
        return host(self.state)[:, :s.vdim, :s.dim].transpose(0, 2, 1)


RECURRENCE_SIZES = [(4, 4, 24, 40), (6, 3, 64, 64), (3, 1, 128, 128), (2, 2, 100, 16), (2, 1, 200, 24), (1, 1, 512, 32)]
STATE_TOL = dict(f32=1e-4, bf16=1e-4)    # the recurrence is 32-bit in either case and the inputs are exact


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("kind", ["lightning", "delta"])
@pytest.mark.parametrize("sizes", RECURRENCE_SIZES)
def test_recurrence_in_steps_and_chunks(dense, dtype, kind, sizes):
    heads, k_heads, dim, vdim = sizes
    if kind == "lightning":
        k_heads = heads
    T = 263
    far = [(260, 3), (130, 127), (128, 64), (127, 63), (66, 0), (64, 63), (63, 1)]
    say("recurrence", kind, dtype, sizes)
    x = Recurrence(dense, kind, heads, k_heads, dim, vdim, T, dtype, seed=dim, far=far)
    want, state = x.want()
    if kind == "delta":                                  # the far key's value comes back, as strong as it was written
        for i, j in far[:2]:
            got = want[i, 0] / want[i, 0].dot(x.v[j, 0]) * x.v[j, 0].dot(x.v[j, 0])
            assert np.abs(want[i, 0]).max() > 1e-3 and np.corrcoef(got, x.v[j, 0])[0, 1] > 0.9, (i, j)
    forms = [False] + ([True] if dim <= 128 else [])
    for chunks in forms:
        for cuts in ((0, T), (0, 64, 128, T), (0, 1, 3, 66, 67, 190, 192, T), (0, 63, 65, 100, T)):
            x.state.fill_(float("nan"))
            got = torch.cat([x.run(a, b, chunks) for a, b in zip(cuts, cuts[1:])])
            close(got, want, dtype, (chunks, cuts), **STATE_TOL)
            for i, _ in far:
                close(got[i], want[i], dtype, (chunks, cuts, i), **STATE_TOL)
            close(x.final(), state, dtype, "state", **STATE_TOL)
    if len(forms) == 2:                                  # the default goes from one to the other
        x.state.fill_(float("nan"))
        cuts, pos = (0, 70, 71, 72, 75, 140, T), torch.zeros((1,), dtype=torch.int32, device="cuda")
        got = []
        for a, b in zip(cuts, cuts[1:]):
            pos.fill_(a)
            got.append(x.run(a, b, None, **(dict(pos=0, pos_dev=pos) if b - a == 1 else {})))
        close(torch.cat(got), want, dtype, "both forms", **STATE_TOL)
    else:
        with pytest.raises(Exception):
            x.run(0, 64, True)


@pytest.mark.parametrize("chunks", [False, True])
def test_decays_of_any_strength(dense, chunks):
    say("strong decays", chunks)
    for dim in (64, 128):
        x = Recurrence(dense, "delta", 3, 3, dim, 32, 200, F32, seed=3, strong=True)
        want, state = x.want()
        got = torch.cat([x.run(a, b, chunks) for a, b in ((0, 90), (90, 200))])
        close(got, want, F32, dim, **STATE_TOL)
        close(x.final(), state, F32, "state", **STATE_TOL)
        x = Recurrence(dense, "delta", 2, 1, dim, 32, 150, F32, seed=4)
        x.a_log[:] = [5.0, -20.0]                            # one head forgets everything between two tokens, one nothing
        x.kw["a_log"] = gpu(x.a_log.astype(np.float32))
        want, state = x.want()
        close(x.run(0, 150, chunks), want, F32, dim, **STATE_TOL)


def test_many_chunks_and_several_segments(dense):
    say("segments")
    s = dense.StateSpec(256, 256, 64, 64)                    # enough heads for a segment of a few chunks
    x = Recurrence(dense, "lightning", 256, 256, 64, 64, 700, F32, seed=8, far=[(690, 2), (513, 510)])
    want, state = x.want()
    close(x.run(0, 700, True), want, F32, "lightning", f32=2e-4)
    x = Recurrence(dense, "delta", 256, 256, 64, 32, 700, F32, seed=9, far=[(690, 2), (513, 510)])
    want, state = x.want()
    close(x.run(0, 700, True), want, F32, "delta", f32=2e-4)
    close(x.final(), state, F32, "state", f32=2e-4)


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("groups,cols,true", [(1, 96, 70), (1, 1536, 1500), (5, 32, 24), (3, 128, 128), (2, 320, 300)])
def test_gated_norm(dense, dtype, groups, cols, true):
    rng = np.random.default_rng(cols)
    M, eps = 7, 1e-3
    mask = np.arange(cols) < true
    o, w = rng.standard_normal((M, groups, cols)) * mask, (rng.standard_normal(cols) * mask).astype(np.float32)
    z = rounded(rng.standard_normal((M, groups * cols + 16)) * 3)
    out = torch.full((M, groups * cols + 40), 7.0, dtype=dtype, device="cuda")
    dense.gated_norm(gpu(o.reshape(M, -1)), gpu(w), eps, groups, true, gpu(z, dtype)[:, 16:], out[:, 32:])
    want = o / np.sqrt((o ** 2).sum(-1, keepdims=True) / true + eps) * w * ost.sigmoid(z[:, 16:].reshape(M, groups, cols))
    close(out[:, 32:32 + groups * cols], want.reshape(M, -1), dtype)
    assert bool((out[:, :32] == 7.0).all()) and bool((out[:, -8:] == 7.0).all())


# ---- the model ---------------------------------------------------------------------------------------------------------------
def _model(config, seed, dtype, **kw):
    from air_hip import sitirax

    w = sitirax_weights(config, seed)
    return sitirax.SitiraxModel(sitirax.SitiraxConfig.from_json(config), lambda n, s: torch.from_numpy(w[n]), dtype, **kw), ost.Model(config, w)


def _tokens(n, vocab, seed=0):
    return np.random.default_rng(seed).integers(0, vocab, n).tolist()


# common head sizes (kernels of their own), and sizes for which forms are missing: keys too long for the kernel of many rows, a state
# that only runs token by token
TALL = sitirax_config([sitirax_parallel(heads=8, kv_heads=2, dim=128, vdim=128, window=80, right_heads=2, right_dim=128, right_vdim=64, ff=96),
                       sitirax_delta(heads=4, kv_heads=2, dim=64, vdim=128, conv=4, ff=96),
                       sitirax_parallel(heads=3, kv_heads=3, dim=64, vdim=64, window=33, right_heads=2, right_dim=64, right_vdim=64),
                       sitirax_delta(heads=2, kv_heads=2, dim=128, vdim=32, conv=2, weights_of=None)], vocab=130, width=128, logit_scale=1.0)
WIDE = sitirax_config([sitirax_parallel(heads=2, kv_heads=1, dim=544, vdim=32, window=50, right_heads=1, right_dim=300, right_vdim=32),
                       sitirax_delta(heads=2, kv_heads=1, dim=140, vdim=264, conv=6, ff=24)], vocab=30, width=64, logit_scale=3.0)
ONE_DELTA = sitirax_config([sitirax_delta(heads=1, kv_heads=1, dim=64, vdim=32, conv=2)], vocab=5, width=64)
ONE_PARALLEL = sitirax_config([sitirax_parallel(heads=1, kv_heads=1, dim=32, vdim=32, window=2, right_heads=1, right_dim=64, right_vdim=32, decay=[0.9], scale=-0.2)],
                              vocab=16, width=64)


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("config", [SITIRAX_MIXED, TALL, WIDE, ONE_DELTA, ONE_PARALLEL], ids=["mixed", "tall", "wide", "delta", "parallel"])
def test_model_whole_portions_and_token_by_token(config, dtype):
    say("model", dtype)
    m, plain = _model(config, 11, dtype, max_portion=90)
    toks = _tokens(150, config["vocab"])
    want = plain.step(toks)
    layers = plain.layers
    same = (lambda g, w, what: close(g, w, F32, what, f32=2e-4)) if dtype == F32 else close_rows
    cache, trace = m.new_cache(160), []
    same(m.step(cache, toks[:80], list(range(80)), trace=trace), want[:80], "first portion")
    assert len(trace) == len(layers)
    for i, (a, b) in enumerate(zip(trace, layers)):
        same(a[:, :config["width"]], b[:80], f"layer {i}")
        assert not bool(a[:, config["width"]:].any())
    for cuts in ([150], [1] * 150, [2] * 75, [70, 2, 3, 1, 74], [149, 1], [1, 149], [5, 64, 65, 16], [17, 16, 15, 64, 38]):
        cache.reset()
        got, i = [], 0
        for n in cuts:
            got.append(m.step(cache, toks[i:i + n], list(range(n))))
            i += n
        same(torch.cat(got), want, cuts[:4])


def test_wanted_places_and_limits():
    m, plain = _model(SITIRAX_MIXED, 12, F32, max_portion=5)
    toks = _tokens(20, 67)
    want = plain.step(toks)
    cache = m.new_cache(20)
    assert m.step(cache, toks[:7], []).shape == (0, 67)
    close(m.step(cache, toks[7:18], [9, 0, 10, 0, 4]), want[[16, 7, 17, 7, 11]], F32, f32=2e-4)   # out of order, over three portions
    assert m.step(cache, toks[18:19], []).shape == (0, 67)
    with pytest.raises(ValueError, match="holds 20"):
        m.step(cache, toks[:2], [])
    for bad in ([], [67], [-1]):
        with pytest.raises(ValueError):
            m.step(cache, bad, [])
    close(m.step(cache, toks[19:], [0, 0]), want[[19, 19]], F32, f32=2e-4)   # a refused step leaves the sequence where it was


def test_requests_side_by_side_and_caches_used_again():
    from air_hip.generation import CachePool

    say("requests side by side")
    m, plain = _model(SITIRAX_MIXED, 13, F32)
    reqs = {n: _tokens(k, 67, seed=k) for n, k in (("a", 90), ("b", 3), ("c", 41), ("d", 66), ("e", 17), ("f", 1))}
    want = {}
    for n, t in reqs.items():
        plain.reset()
        want[n] = plain.step(t)
    pool, at, got = CachePool(m, 96), {n: 0 for n in reqs}, {n: [] for n in reqs}

    def run(n, k):
        t = reqs[n][at[n]:at[n] + k]
        got[n].append(m.step(pool.get(n), t, list(range(len(t)))))
        at[n] += len(t)
        if at[n] == len(reqs[n]):
            pool.end(n)

    run("a", 65); run("b", 2); run("c", 1); run("a", 1); run("b", 1); run("c", 40)   # b and c end, their caches go on
    run("d", 33); run("e", 17); run("a", 24); run("d", 33); run("f", 1)
    assert len(pool.free) == 3 and not pool.live
    for n in reqs:
        close(torch.cat(got[n]), want[n], F32, n, f32=2e-4)


def _plain_greedy(plain, prompt, n):
    plain.reset()
    out = [int(plain.step(prompt)[-1].argmax())]
    for _ in range(n):
        out.append(int(plain.step([out[-1]])[0].argmax()))
    return out


@pytest.mark.parametrize("prompt_len", [1, 5, 70])
def test_generate_through_the_token_loop(prompt_len):
    from air_hip.generation import generate

    say("generate", prompt_len)
    m, plain = _model(SITIRAX_MIXED, 14, F32, max_portion=33)
    prompt, other = _tokens(prompt_len, 67, 5), _tokens(9, 67, 6)
    want, want2 = _plain_greedy(plain, prompt, 75), _plain_greedy(plain, other, 20)
    assert generate(m, prompt, 75) == want                    # the captured step, across the edges of windows and blocks
    seen = []
    assert generate(m, prompt, 75, on_token=seen.append) == want == seen
    cache = m.new_cache(160)
    for p, n, w in ((prompt, 75, want), (other, 20, want2), (prompt, 75, want)):   # one cache, its graph replayed for each
        assert generate(m, p, n, cache=cache) == w
        torch.cuda.synchronize()
    stop = want[10]
    assert generate(m, prompt, 75, eos_token_ids=(stop,)) == want[:want.index(stop, 1) + 1]


def test_generate_in_bf16_follows_its_own_logits():
    from air_hip.generation import generate

    m, _ = _model(TALL, 21, BF16)
    prompt = _tokens(20, 130, 1)
    out = generate(m, prompt, 100)
    logits = m.step(m.new_cache(140), prompt + out[:-1], list(range(19, 120)))     # the same sequence as one prompt
    best = logits.max(-1).values
    chosen = logits[torch.arange(101, device="cuda"), torch.tensor(out, device="cuda")]
    assert float(((best - chosen) / logits.std(-1)).max()) < 0.05


def test_generate_where_the_head_sizes_only_run_split():
    from air_hip.generation import generate

    m, plain = _model(WIDE, 19, F32)
    prompt = _tokens(4, 30, 5)
    assert generate(m, prompt, 60) == _plain_greedy(plain, prompt, 60)


def test_greedy_decode_inside_a_callers_graph():
    m, plain = _model(TALL, 15, F32)
    prompt = _tokens(6, 130, 2)
    want = _plain_greedy(plain, prompt, 12)
    cache = m.new_cache(64)
    _, first = m.prefill(cache, prompt)
    saved = [{n: t.clone() for n, t in c.items()} for c in cache.layers]
    stream = torch.cuda.Stream()
    stream.wait_stream(torch.cuda.current_stream())
    with torch.cuda.stream(stream):
        m.decode_greedy(cache, first, 2)
        stream.synchronize()
        graph = torch.cuda.CUDAGraph()
        cache.pos = 6
        with torch.cuda.graph(graph, stream=stream):
            ids = m.decode_greedy(cache, first, 12)
        for _ in range(3):
            for c, old in zip(cache.layers, saved):          # states go on: every replay starts from those behind the prompt
                for n, t in c.items():
                    t.copy_(old[n])
            graph.replay()
            stream.synchronize()
            assert ids.tolist() == want[1:]
            torch.ones(100, device="cuda").sum().item()


def test_long_decoding_keeps_to_the_plain_logits():
    say("long decoding")
    m, plain = _model(sitirax_config([sitirax_parallel(heads=2, kv_heads=1, dim=32, vdim=32, window=45, right_heads=2, right_dim=64, right_vdim=32, decay=[0.9995, 1.0]),
                                      sitirax_delta(heads=2, kv_heads=1, dim=64, vdim=32, conv=4, ff=32)], vocab=40, width=64), 16, F32, max_portion=30)
    toks = _tokens(420, 40, 3)
    want = plain.step(toks)
    cache = m.new_cache(420)
    m.step(cache, toks[:100], [])
    got = torch.cat([m.step(cache, [t], [0]) for t in toks[100:]])
    close(got, want[100:], F32, f32=2e-4)
    close(got[-40:], want[-40:], F32, "the last ones", f32=2e-4)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_run_program(tmp_path, dtype):
    say("bin/trace_run", dtype)
    w = sitirax_weights(SITIRAX_MIXED, 17)
    path = sitirax_write(tmp_path / "m", SITIRAX_MIXED, w)
    toks = _tokens(60, 67, 8)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": toks[:39], "want": [3, 38]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": toks[39:40], "want": [0]}], "end": []},
             {"step": 2, "entries": [{"id": "x", "tokens": toks[40:], "want": []}], "end": ["x"]},
             {"step": 3, "entries": [{"id": "y", "tokens": toks[:3], "want": [2]}], "end": ["y"]}]
    out = tmp_path / "out"
    out.mkdir()
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", path, "--dtype", dtype, "--out", str(out), "--max-tokens", "60"],
                       input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(4)]
    want = ost.Model(SITIRAX_MIXED, w).step(toks)
    for step, rows in ((0, [3, 38]), (1, [39]), (3, [2])):
        got = torch.from_numpy(np.fromfile(out / f"{step}.f32", "<f4").reshape(-1, 67))
        close(got, want[rows], F32, step, f32=2e-4) if dtype == "float32" else close_rows(got, want[rows], step)
    assert not (out / "2.f32").exists()


def test_generate_command_line(tmp_path, capsys):
    from air_hip import generate as cli

    w = sitirax_weights(SITIRAX_MIXED, 18)
    path = sitirax_write(tmp_path / "m", SITIRAX_MIXED, w)
    want = _plain_greedy(ost.Model(SITIRAX_MIXED, w), [4, 9, 33], 8)
    assert cli.main(["--model", path, "--prompt", "4,9,33", "-n", "8", "--dtype", "float32"]) == 0
    assert capsys.readouterr().out.strip().splitlines()[-1] == ",".join(map(str, want))
