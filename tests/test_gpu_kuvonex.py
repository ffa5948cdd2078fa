"""The dense-weight kernels one by one and the Kuvonex model as a whole on the GPU, against the plain float64
implementation (oracle/kuvonex.py) and float32 / float64 products on the CPU."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from helpers import KUVONEX_MIXED, kuvonex_config, kuvonex_layer, kuvonex_weights, kuvonex_write
from oracle import kuvonex as okv

pytestmark = pytest.mark.gpu
F32, BF16 = torch.float32, torch.bfloat16
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


@pytest.fixture(scope="module")
def dense():
    from air_hip import dense as d
    return d


def say(*a):
    print(*a, flush=True)


def rnd(shape, seed, scale=1.0, dtype=BF16):
    """Values that bf16 holds exactly, in `dtype`, on the GPU."""
    t = torch.randn(shape, generator=torch.Generator().manual_seed(seed)) * scale
    return t.to(BF16).to(dtype).cuda()


def close(got, want, dtype, what="", f32=2e-5, bf16=1.2e-2):
    """Every error within tolerance x (the rms of what is expected + the expected element itself)."""
    got, want = got.detach().float().cpu().numpy().astype(np.float64), np.asarray(want, np.float64)
    err = np.abs(got - want) / (np.sqrt(np.mean(want ** 2)) + np.abs(want) + 1e-30)
    assert err.max() <= (f32 if dtype == F32 else bf16), (what, err.max(), np.unravel_index(err.argmax(), err.shape))


def close_rows(got, want, what=""):
    """bf16 logits: the rms error of a position is small except where a close call of the router went the other way."""
    d = got.detach().float().cpu().numpy().astype(np.float64) - want
    err = np.sqrt((d ** 2).mean(-1) / (want ** 2).mean())
    assert (err > 0.15).mean() <= 0.04 and np.median(err) < 0.02, (what, np.sort(err)[-8:], np.median(err))


def host(t):
    return t.float().cpu().numpy().astype(np.float64)


# ---- products --------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("M,N,K", [(2, 16, 64), (33, 80, 128), (130, 208, 192), (300, 528, 384), (1030, 2576, 64)])
def test_gemm(dense, dtype, M, N, K):
    say("gemm", dtype, M, N, K)
    a, w = rnd((M, K), 1, dtype=dtype), rnd((N, K), 2, dtype=dtype)
    want = host(a) @ host(w).T
    close(dense.gemm(a, w), want, dtype, "element type")
    close(dense.gemm(a, w, out_f32=True), want, F32, "fp32", f32=2e-5)


@pytest.mark.parametrize("tile", [32, 128, 256])
def test_gemm_tiles_and_strides(dense, tile):
    from air_hip import _lib
    import ctypes

    say("gemm tile", tile)
    lib = _lib.load_dense_library()
    M, N, K = 517, 1040, 192
    big, w = rnd((M, K + 64), 3), rnd((N, K), 4)
    out = torch.full((M, N + 16), 7.0, dtype=F32, device="cuda")
    g = _lib.GemmArgs(a=big.data_ptr(), w=w.data_ptr(), out=out.data_ptr(), lda=K + 64, ldo=N + 16, M=M, N=N, K=K, epilogue=1, tile_rows=tile)
    _lib.check_dense(lib.dlm_gemm(0, ctypes.byref(g), torch.cuda.current_stream().cuda_stream))
    close(out[:, :N], host(big[:, :K]) @ host(w).T, F32)
    assert bool((out[:, N:] == 7.0).all())


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("N,K,width", [(16, 64, 40), (530, 576, 530), (1000, 1088, 1088), (4112, 2112, 2100), (600, 8192, 8192)])
def test_gemv_and_its_intakes(dense, dtype, N, K, width):
    say("gemv", dtype, N, K)
    eps = 1e-3
    w = rnd((N, K), 1, K ** -0.5, dtype)
    x = rnd((K,), 2, dtype=dtype)
    W = host(w)
    close(dense.gemv(x, w), W @ host(x), dtype, "plain")
    close(dense.gemv(x, w, out_f32=True), W @ host(x), F32, "plain fp32")

    def vec(seed, scale=1.0):
        v = torch.randn((K,), generator=torch.Generator().manual_seed(seed)) * scale
        v[width:] = 0
        return v.cuda()

    res, y, nw, fw = vec(3), vec(4, 5.0), vec(5), vec(6)
    R, Y = host(res), host(y)
    new = R + Y / np.sqrt((Y ** 2).sum() / width + eps) * host(nw)
    r = dense.Residual(res, y, nw, eps, width)
    out, res2, h = dense.gemv_residual(r, w, out_f32=True, want_h=True)
    close(res2, new, F32, "residual")
    close(h, new, dtype, "residual, element type")
    close(out, W @ new, dtype, "residual product")
    fin = new / np.sqrt((new ** 2).sum() / width + eps) * host(fw)
    keys = dense.new_keys(w)
    logits = dense.gemv_final(r, fw, w, keys, N - 3)
    close(logits, W @ fin, dtype, "final")
    tok = torch.full((1,), -1, dtype=torch.int32, device="cuda")
    pos, hist = torch.tensor([4], dtype=torch.int32, device="cuda"), torch.zeros((8,), dtype=torch.int32, device="cuda")
    dense.argmax(keys, tok, pos, hist)
    best = int(logits[:N - 3].argmax())
    assert int(tok) == best and int(pos) == 5 and hist.tolist() == [0] * 5 + [best, 0, 0]
    only = dense.Residual(res, None, None, eps, width)
    close(dense.gemv_final(only, fw, w), W @ (R / np.sqrt((R ** 2).sum() / width + eps) * host(fw)), dtype, "final without a pending output")
    emb = rnd((9, K), 7, dtype=dtype)
    out, res3, h = dense.gemv_embed(torch.tensor([5], dtype=torch.int32, device="cuda"), emb, 1.7, w, want_h=True)
    close(res3, host(emb)[5] * 1.7, F32, "embedding", f32=1e-6)
    close(out, W @ (host(emb)[5] * 1.7), dtype, "embedding product")


def test_argmax_takes_the_lowest_row_on_ties(dense):
    w = torch.zeros((700, 64), dtype=F32, device="cuda")
    w[[650, 33, 480]] = 1.0
    x = torch.ones((64,), dtype=F32, device="cuda")
    keys, tok = dense.new_keys(w), torch.zeros((1,), dtype=torch.int32, device="cuda")
    dense.gemv(x, w, out_f32=True, keys=keys, n_valid=700)
    dense.argmax(keys, tok)
    assert int(tok) == 33
    dense.gemv(-x, w, out_f32=True, keys=keys, n_valid=700)   # the largest is 0, first at row 0 (-0 counts as 0)
    dense.argmax(keys, tok)
    assert int(tok) == 0


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_row_steps(dense, dtype):
    say("row steps", dtype)
    M, K, width, eps, top = 5, 192, 150, 1e-2, 3
    emb = rnd((11, K), 1, dtype=dtype)
    ids = torch.tensor([3, 0, 10, 3, 7], dtype=torch.int32, device="cuda")
    res, h = dense.embed_rows(ids, emb, 0.3)
    close(res, host(emb)[ids.cpu().numpy()] * 0.3, F32, f32=1e-6)
    y = torch.randn((M, K), generator=torch.Generator().manual_seed(2)).cuda()
    nw = torch.randn((K,), generator=torch.Generator().manual_seed(3)).cuda()
    norm = lambda v, w: v / np.sqrt((v ** 2).sum(-1, keepdims=True) / width + eps) * w
    want = host(res) + norm(host(y), host(nw))
    h = dense.residual_norm_rows(res, y, nw, eps, width, dtype)
    close(res, want, F32)
    close(h, want, dtype)
    ys, wt = rnd((M * top, K), 4, dtype=dtype), torch.rand((M, top), generator=torch.Generator().manual_seed(5)).cuda()
    want = host(res) + norm(np.einsum("ms,msk->mk", host(wt), host(ys).reshape(M, top, K)), host(nw))
    dense.residual_norm_rows(res, ys, nw, eps, width, dtype, weights=wt)
    close(res, want, F32)
    rows = torch.tensor([4, 1, 1], dtype=torch.int32, device="cuda")
    close(dense.norm_rows(res, nw, eps, width, dtype, rows), norm(want, host(nw))[[4, 1, 1]], dtype)
    close(dense.norm_rows(res, nw, eps, width, dtype), norm(want, host(nw)), dtype)


# ---- router and experts -----------------------------------------------------------------------------------------------
@pytest.mark.parametrize("experts,top,groups,keep,shift", [(10, 2, 2, 1, 0.0), (10, 3, 2, 1, -3.0), (12, 12, 1, 1, -0.5), (6, 3, 6, 4, -0.5), (64, 6, 8, 3, 0.0),
                                                           (160, 8, 8, 3, -9.0), (1024, 32, 128, 20, 0.0), (1, 1, 1, 1, 0.0)])
def test_router_choice(dense, experts, top, groups, keep, shift):
    say("router", experts, top, groups, keep, shift)
    rng = np.random.default_rng(experts + top)
    M, ld = 37, (experts + 15) // 16 * 16
    z = (rng.standard_normal((M, ld)) * 2).astype(np.float32)
    z[:, experts:] = 50.0                                       # padding columns must not be looked at
    corr = (rng.standard_normal(experts) * 0.4 + shift).astype(np.float32)
    ids, wts = dense.moe_select(torch.from_numpy(z).cuda(), dense.RouterSpec(torch.from_numpy(corr).cuda(), experts, top, groups, keep))
    for m in range(M):
        want, wt = okv.route(np.ones(experts), np.diag(z[m, :experts].astype(np.float64)), corr.astype(np.float64), top, groups, keep)
        assert ids[m].tolist() == want, m
        assert np.allclose(wts[m].cpu().numpy(), wt, rtol=1e-5)


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("M,experts,top,groups,keep,K,ff,N", [(1, 10, 2, 2, 1, 64, 128, 128), (1, 16, 5, 4, 2, 1152, 576, 320), (2, 9, 2, 3, 1, 128, 64, 64),
                                                               (61, 6, 3, 6, 4, 192, 128, 192), (700, 5, 2, 1, 1, 64, 192, 64)])
def test_mixture(dense, dtype, M, experts, top, groups, keep, K, ff, N):
    say("mixture", dtype, M, experts)
    h = rnd((M, K), 1, dtype=dtype)
    gate, up = rnd((experts, ff, K), 2, K ** -0.5, dtype), rnd((experts, ff, K), 3, K ** -0.5, dtype)
    down = rnd((experts, N, ff), 4, ff ** -0.5, dtype)
    gu = torch.stack([gate.reshape(experts, ff // 16, 16, K), up.reshape(experts, ff // 16, 16, K)], dim=2).reshape(experts, 2 * ff, K).contiguous()
    logits = torch.randn((M, (experts + 15) // 16 * 16), generator=torch.Generator().manual_seed(5)).cuda() * 2
    if M > 100:
        logits[:, 0] = 9.0                                      # one expert has every token, one none
        logits[:, 1] = -30.0
    corr = torch.zeros((experts,), device="cuda")
    spec = dense.RouterSpec(corr, experts, top, groups, keep)
    if M == 1:
        got = dense.moe_gemv(h.reshape(-1), logits.reshape(-1), spec, gu, down).reshape(1, -1)
    else:
        y, wts = dense.moe_rows(h, logits, spec, gu, down)
        got = torch.einsum("ms,msn->mn", wts.cpu(), y.float().cpu().reshape(M, top, N))
    H, G, U, D = host(h), host(gate), host(up), host(down)
    want = np.zeros((M, N))
    for m in range(M):
        ids, wt = okv.route(np.ones(experts), np.diag(host(logits)[m, :experts]), np.zeros(experts), top, groups, keep)
        for e, a in zip(ids, wt):
            want[m] += a * okv.expert(H[m], G[e], U[e], D[e])
    close(got, want, dtype, bf16=3e-2)


# ---- latent attention -----------------------------------------------------------------------------------------------------
LATENT_SIZES = [   # heads, dim, rot, vdim, rank
    (3, 24, 8, 40, 56), (6, 64, 32, 64, 192), (5, 16, 6, 24, 40), (16, 128, 64, 128, 512), (2, 192, 64, 256, 320), (1, 300, 20, 288, 1000), (17, 32, 32, 32, 64),
]


class Latents:
    """Random inputs of one latent attention over T positions, and the plain result; `far`: (query, key) pairs whose score
    stands out by ~30."""

    def __init__(self, dense, sizes, T, dtype, seed=0, far=(), own=True):
        H, D, R, V, C = sizes
        self.spec = s = dense.LatentSpec(H, D, R, V, C, (D + R) ** -0.5)
        self.dense, self.T, self.dtype, self.own, self.base = dense, T, dtype, own, 300.0
        rng = np.random.default_rng(seed)
        b = lambda a: torch.from_numpy(np.asarray(a, np.float32)).to(BF16).double().numpy()
        q = rng.standard_normal((T, H, D + R))
        kr = rng.standard_normal((T, R))
        for i, j in far:
            u = rng.standard_normal(R)
            a = np.sqrt(40.0 / s.scale) / np.linalg.norm(u)
            back = lambda p: okv.rotate_interleaved((u * a)[None], [-p], self.base)[0]   # rotation brings both to u * a
            kr[j] = back(j)
            q[i, :, D:] = back(i)
        self.q, self.kr, self.lat, self.gate = b(q), b(kr), b(rng.standard_normal((T, C))), b(rng.standard_normal((T, H, V)))
        self.uk, self.uv = b(rng.standard_normal((H, D, C)) * C ** -0.5), b(rng.standard_normal((H, V, C)) * C ** -0.5)
        self.sink, self.norm_w, self.eps = rng.standard_normal(H), 1 + 0.2 * rng.standard_normal(C), 1e-4
        def gpu(a, dt=dtype):
            return torch.from_numpy(np.ascontiguousarray(a)).to(dt).cuda()
        Z = np.zeros
        pq = Z((T, H, s.dim_p + s.rot_p))
        pq[..., :D], pq[..., s.dim_p:s.dim_p + R] = self.q[..., :D], self.q[..., D:]
        pk = Z((T, s.rank_p + s.rot_p))
        pk[:, :C], pk[:, s.rank_p:s.rank_p + R] = self.lat, self.kr
        pg = Z((T, H, s.vdim_p))
        pg[..., :V] = self.gate
        parts = [pq.reshape(T, -1)] + ([pk] if own else []) + [pg.reshape(T, -1)]
        self.kv_off = parts[0].shape[1] if own else -1
        self.gate_off = sum(x.shape[1] for x in parts[:-1])
        self.proj = gpu(np.concatenate(parts, 1))
        uk, uv = Z((H, s.dim_p, s.rank_p)), Z((H, s.vdim_p, s.rank_p))
        uk[:, :D, :C], uv[:, :V, :C] = self.uk, self.uv
        self.w_ukv = gpu(np.concatenate([uk.reshape(-1, s.rank_p), uv.reshape(-1, s.rank_p)]))
        self.kv_norm = gpu(np.pad(self.norm_w, (0, s.rank_p - C)), F32)
        self.sink_d = gpu(self.sink, F32)
        from air_hip.kuvonex import rotation_table
        self.lut = rotation_table(self.base, R, T + 5, "cuda")
        self.cache = torch.full((T + 3, s.cache_width), float("nan"), dtype=dtype, device="cuda")   # rows not yet written must not be read

    def want(self):
        s = self.spec
        c = okv.rms_norm(self.lat, self.norm_w, self.eps)
        k = okv.rotate_interleaved(self.kr, range(self.T), self.base)
        o = okv.latent_attention(self.q.reshape(self.T, -1), c, k, self.uk.reshape(-1, s.rank), self.uv.reshape(-1, s.rank), self.sink, s.heads, s.dim, s.vdim,
                                 s.rot, s.scale, range(self.T), self.base)
        return o * okv.sigmoid(self.gate.reshape(self.T, -1))

    def fill(self):
        """Cache rows written as another layer's, for a layer without latents of its own."""
        s = self.spec
        self.cache[:self.T] = 0
        self.cache[:self.T, :s.rank] = torch.from_numpy(okv.rms_norm(self.lat, self.norm_w, self.eps)).to(self.dtype)
        self.cache[:self.T, s.rank_p:s.rank_p + s.rot] = torch.from_numpy(okv.rotate_interleaved(self.kr, range(self.T), self.base)).to(self.dtype)

    def run(self, form, a, b, **k):
        args = (self.spec, self.proj[a:b].clone(), self.kv_off, self.gate_off, self.lut, self.kv_norm, self.eps, self.cache, a, self.w_ukv, self.sink_d)
        out = self.dense.latent_attention_rows(*args) if form == "rows" else self.dense.latent_attention_absorbed(*args, **k)
        s = self.spec
        assert not bool(out[:, s.heads * s.vdim_p:].any())
        return out[:, :s.heads * s.vdim_p].reshape(b - a, s.heads, s.vdim_p)[..., :s.vdim].reshape(b - a, -1)


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("sizes", LATENT_SIZES)
@pytest.mark.parametrize("form", ["rows", "absorbed"])
def test_latent_attention(dense, dtype, sizes, form):
    T = 150
    if form == "absorbed" and not dense.LatentSpec(*sizes, 1.0).decode_supported(dtype):
        pytest.skip("such a latent only runs expanded")
    say("latent attention", dtype, sizes, form)
    # far keys around every block edge (32 and 64 keys), the first and the last visible key
    far = [(40, 0), (64, 31), (65, 32), (100, 63), (101, 64), (149, 1), (148, 147), (130, 127), (131, 128)]
    x = Latents(dense, sizes, T, dtype, seed=sizes[0], far=far)
    want = x.want()
    c = okv.rms_norm(x.lat, x.norm_w, x.eps)
    for i, j in far[:3] if sizes[2] >= 8 else []:            # the plain result is the far key's value
        v = (c[j] @ x.uv[0].T) * okv.sigmoid(x.gate[i, 0])
        assert np.allclose(want[i, :sizes[3]], v, atol=1e-6), (i, j)
    tol = dict(f32=5e-5, bf16=6e-2)
    got = torch.cat([x.run(form, a, b) for a, b in ((0, 70), (70, 72), (72, T))])
    close(got, want, dtype, "portions", **tol)
    for i, j in far:                                         # each row against its own size, not the matrix's
        close(got[i], want[i], dtype, (i, j), **tol)
    close(x.run(form, 0, T), want, dtype, "whole", **tol)


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_latent_attention_forms_agree_token_by_token_and_with_the_position_on_the_device(dense, dtype):
    x = Latents(dense, (6, 64, 32, 64, 192), 140, dtype, seed=4, far=[(139, 63), (138, 64)])
    want = x.want()
    say("token by token", dtype)
    one = torch.cat([x.run("absorbed", i, i + 1) for i in range(x.T)])
    close(one, want, dtype, f32=5e-5, bf16=6e-2)
    pos = torch.zeros((1,), dtype=torch.int32, device="cuda")
    for i in (0, 63, 64, 127, 128, 139):
        for nsplit in (1, 2, 7, 128):
            pos.fill_(i)
            got = x.dense.latent_attention_absorbed(x.spec, x.proj[i], x.kv_off, x.gate_off, x.lut, x.kv_norm, x.eps, x.cache, 0, x.w_ukv, x.sink_d,
                                                    pos_dev=pos, nsplit=nsplit)
            s = x.spec
            got = got[:, :s.heads * s.vdim_p].reshape(s.heads, s.vdim_p)[:, :s.vdim].reshape(-1)
            close(got, want[i], dtype, (i, nsplit), f32=5e-5, bf16=6e-2)


@pytest.mark.parametrize("form", ["rows", "absorbed"])
def test_latent_attention_over_another_layers_rows(dense, form):
    say("shared latents", form)
    x = Latents(dense, (3, 24, 8, 40, 56), 77, F32, seed=9, own=False, far=[(76, 0)])
    x.fill()
    before = x.cache.clone()
    close(torch.cat([x.run(form, 0, 40), x.run(form, 40, 77)]), x.want(), F32, f32=5e-5)
    assert torch.equal(before[:77], x.cache[:77])             # nothing appended


@pytest.mark.parametrize("form", ["rows", "absorbed"])
@pytest.mark.parametrize("dtype", [F32, BF16])
def test_sinks_large_and_small(dense, dtype, form):
    say("sinks", dtype, form)
    x = Latents(dense, (4, 64, 32, 64, 192), 70, dtype, seed=2)
    for sink in ([-80.0, 0.0, 6.0, 80.0], [300.0, -300.0, 2.0, -2.0]):
        x.sink = np.array(sink)
        x.sink_d = torch.tensor(sink, dtype=F32, device="cuda")
        got, want = x.run(form, 0, 70), x.want()
        for h in range(4):                                   # every head against its own size
            sl = slice(h * 64, (h + 1) * 64)
            if sink[h] > 40:
                assert float(got[:, sl].abs().max()) < 1e-8
            else:
                close(got[:, sl], want[:, sl], dtype, (sink[h]), f32=5e-5, bf16=6e-2)


# ---- the model ---------------------------------------------------------------------------------------------------------------
def _model(config, seed, dtype):
    from air_hip import kuvonex

    w = kuvonex_weights(config, seed)
    m = kuvonex.KuvonexModel(kuvonex.KuvonexConfig.from_json(config), lambda n, s: torch.from_numpy(w[n].reshape(s)), dtype)
    return m, okv.Model(config, w)


def _tokens(n, vocab, seed=0):
    return np.random.default_rng(seed).integers(0, vocab, n).tolist()


TALL = kuvonex_config([kuvonex_layer(heads=4, dim=64, rot_dim=32, vdim=64, kv_rank=192, mlp=(8, 3, 4, 2, 96)),
                       kuvonex_layer(heads=2, dim=128, rot_dim=64, vdim=128, kv_rank=64, mlp=None),
                       kuvonex_layer(heads=4, dim=64, rot_dim=32, vdim=64, kv_rank=192, kv_from=0, mlp=(3, 3, 1, 1, 64))], vocab=130, width=192, embed_scale=1.0)
# sizes for which only one of the two forms of attention exists (fp32: no latent form for the first, no expanded one for the second)
WIDE = kuvonex_config([kuvonex_layer(heads=2, dim=32, rot_dim=16, vdim=288, kv_rank=1000, mlp=(4, 2, 2, 2, 24)),
                       kuvonex_layer(heads=2, dim=512, rot_dim=34, vdim=32, kv_rank=64)], vocab=30, width=128, embed_scale=1.0)
ONE_LAYER = kuvonex_config([kuvonex_layer(heads=1, dim=32, rot_dim=2, vdim=32, kv_rank=64, mlp=(2, 1, 2, 1, 16))], vocab=5, width=64)


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("config", [KUVONEX_MIXED, TALL, WIDE, ONE_LAYER], ids=["mixed", "tall", "wide", "one"])
def test_model_whole_portions_and_token_by_token(config, dtype):
    say("model", dtype)
    m, plain = _model(config, 11, dtype)
    toks = _tokens(150, config["vocab"])
    want = plain.step(toks)
    layers = plain.layers
    same = (lambda g, w, what: close(g, w, F32, what, f32=1e-4)) if dtype == F32 else close_rows
    cache, trace = m.new_cache(160), []
    same(m.step(cache, toks, list(range(150)), trace=trace), want, "whole")
    assert len(trace) == len(layers)
    for i, (a, b) in enumerate(zip(trace, layers)):
        same(a[:, :config["width"]], b, f"layer {i}")
        assert not bool(a[:, config["width"]:].any())
    for cuts in ([1] * 150, [2] * 75, [70, 2, 3, 1, 74], [149, 1], [1, 149], [5, 64, 65, 16]):
        cache.reset()
        got, i = [], 0
        for n in cuts:
            got.append(m.step(cache, toks[i:i + n], list(range(n))))
            i += n
        same(torch.cat(got), want, cuts[:4])


def test_wanted_places_and_limits():
    m, plain = _model(KUVONEX_MIXED, 12, F32)
    toks = _tokens(20, 67)
    want = plain.step(toks)
    cache = m.new_cache(20)
    assert m.step(cache, toks[:7], []).shape == (0, 67)
    close(m.step(cache, toks[7:12], [4, 0, 0]), want[[11, 7, 7]], F32, f32=1e-4)
    assert m.step(cache, toks[12:13], []).shape == (0, 67)
    close(m.step(cache, toks[13:14], [0, 0]), want[[13, 13]], F32, f32=1e-4)
    with pytest.raises(ValueError, match="holds 20"):
        m.step(cache, toks[:7], [])
    for bad in ([], [67], [-1]):
        with pytest.raises(ValueError):
            m.step(cache, bad, [])
    close(m.step(cache, toks[14:], [5]), want[[19]], F32, f32=1e-4)   # a refused step leaves the sequence where it was


def test_requests_side_by_side_and_caches_used_again():
    from air_hip.generation import CachePool

    say("requests side by side")
    m, plain = _model(KUVONEX_MIXED, 13, F32)
    reqs = {n: _tokens(k, 67, seed=k) for n, k in (("a", 90), ("b", 3), ("c", 41), ("d", 66), ("e", 17))}
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
    run("d", 33); run("e", 17); run("a", 24); run("d", 33)
    assert len(pool.free) == 3 and not pool.live
    for n in reqs:
        close(torch.cat(got[n]), want[n], F32, n, f32=1e-4)


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
    m, plain = _model(KUVONEX_MIXED, 14, F32)
    prompt, other = _tokens(prompt_len, 67, 5), _tokens(9, 67, 6)
    want, want2 = _plain_greedy(plain, prompt, 75), _plain_greedy(plain, other, 20)
    assert generate(m, prompt, 75) == want                    # the captured step, across a block edge of 64 keys
    seen = []
    assert generate(m, prompt, 75, on_token=seen.append) == want == seen
    cache = m.new_cache(160)
    for p, n, w in ((prompt, 75, want), (other, 20, want2), (prompt, 75, want)):   # one cache, its graph replayed for each
        assert generate(m, p, n, cache=cache) == w
        torch.cuda.synchronize()
    stop = want[10]
    assert generate(m, prompt, 75, eos_token_ids=(stop,)) == want[:want.index(stop, 1) + 1]


def test_generate_where_the_position_cannot_lie_on_the_device():
    from air_hip.generation import generate

    m, plain = _model(WIDE, 19, F32)
    prompt = _tokens(4, 30, 5)
    assert generate(m, prompt, 6) == _plain_greedy(plain, prompt, 6)


def test_greedy_decode_inside_a_callers_graph():
    m, plain = _model(TALL, 15, F32)
    prompt = _tokens(6, 130, 2)
    want = _plain_greedy(plain, prompt, 12)
    cache = m.new_cache(64)
    _, first = m.prefill(cache, prompt)
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
            graph.replay()
            stream.synchronize()
            assert ids.tolist() == want[1:]
            torch.ones(100, device="cuda").sum().item()


def test_long_decoding_keeps_to_the_plain_logits():
    say("long decoding")
    m, plain = _model(kuvonex_config([kuvonex_layer(heads=2, dim=32, rot_dim=16, vdim=32, kv_rank=64, mlp=(4, 2, 2, 1, 32)),
                                      kuvonex_layer(heads=2, dim=32, rot_dim=16, vdim=32, kv_rank=64, kv_from=0)], vocab=40, width=64), 16, F32)
    toks = _tokens(420, 40, 3)
    want = plain.step(toks)
    cache = m.new_cache(420)
    m.step(cache, toks[:100], [])
    got = torch.cat([m.step(cache, [t], [0]) for t in toks[100:]])
    close(got, want[100:], F32, f32=1e-4)
    close(got[-40:], want[-40:], F32, "the last ones", f32=1e-4)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_run_program(tmp_path, dtype):
    say("bin/trace_run", dtype)
    w = kuvonex_weights(KUVONEX_MIXED, 17)
    path = kuvonex_write(tmp_path / "m", KUVONEX_MIXED, w)
    toks = _tokens(30, 67, 8)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": toks[:19], "want": [3, 18]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": toks[19:20], "want": [0]}], "end": []},
             {"step": 2, "entries": [{"id": "x", "tokens": toks[20:], "want": []}], "end": ["x"]},
             {"step": 3, "entries": [{"id": "y", "tokens": toks[:3], "want": [2]}], "end": ["y"]}]
    out = tmp_path / "out"
    out.mkdir()
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", path, "--dtype", dtype, "--out", str(out), "--max-tokens", "30"],
                       input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(4)]
    want = okv.Model(KUVONEX_MIXED, w).step(toks)
    dt = F32 if dtype == "float32" else BF16
    for step, rows in ((0, [3, 18]), (1, [19]), (3, [2])):
        got = torch.from_numpy(np.fromfile(out / f"{step}.f32", "<f4").reshape(-1, 67))
        close(got, want[rows], F32, step, f32=1e-4) if dt == F32 else close_rows(got, want[rows], step)
    assert not (out / "2.f32").exists()


def test_generate_command_line(tmp_path, capsys):
    from air_hip import generate as cli

    w = kuvonex_weights(KUVONEX_MIXED, 18)
    path = kuvonex_write(tmp_path / "m", KUVONEX_MIXED, w)
    want = _plain_greedy(okv.Model(KUVONEX_MIXED, w), [4, 9, 33], 8)
    assert cli.main(["--model", path, "--prompt", "4,9,33", "-n", "8", "--dtype", "float32"]) == 0
    assert capsys.readouterr().out.strip().splitlines()[-1] == ",".join(map(str, want))
    assert cli.main(["--model", path, "--prompt", "4,9,33", "-n", "8", "--dtype", "float32", "--stream"]) == 0
    assert [int(x) for x in capsys.readouterr().out.split()] == want


def test_llama_checkpoint_through_the_same_registry_loop_and_trace(tmp_path):
    from air_hip import decode, generation, models, trace
    from test_weights_cpu import CFG, _write_checkpoint

    say("llama through the registry")
    path = str(tmp_path / "ckpt")
    _write_checkpoint(path, tied=True, seed=11)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump({"architectures": ["LlamaForCausalLM"], "num_hidden_layers": CFG.n_layers, "hidden_size": CFG.emb_dim, "num_attention_heads": CFG.n_heads,
                   "num_key_value_heads": CFG.n_kv_heads, "head_dim": CFG.head_dim, "intermediate_size": CFG.hidden_dim, "vocab_size": CFG.vocab_size,
                   "rope_theta": CFG.rope_base, "rms_norm_eps": CFG.rms_eps}, f)
    with pytest.raises(generation.UnsupportedDtype):
        models.load_model(path, dtype=F32)
    m = models.load_model(path)
    prompt = _tokens(6, CFG.vocab_size, 1)
    lut = decode.generate_rope_lut(CFG, 16)
    want = decode.generate(prompt, m.layers, m.embed_table, m.final_norm, m.lm_head, CFG, lut, n_tokens=5, eos_token_ids=())
    assert generation.generate(m, prompt, 5) == want
    cache = m.new_cache(11)
    whole = m.step(cache, prompt, [5])
    cache.reset()
    parts = torch.cat([m.step(cache, prompt[:1], []), m.step(cache, prompt[1:], [0, 4])])
    assert parts.shape == (2, CFG.vocab_size) and bool(torch.isfinite(parts).all())
    d = host(parts[1]) - host(whole[0])
    assert np.sqrt((d ** 2).mean()) <= 0.05 * np.sqrt((host(whole) ** 2).mean())
