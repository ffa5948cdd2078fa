"""The plain Sitirax implementation against hand-made cases, and the product's configuration, loader, registry and argument checks
on the host (CPU only)."""
import ctypes

import numpy as np
import pytest
import torch

from helpers import SITIRAX_MIXED, sitirax_config, sitirax_delta, sitirax_parallel, sitirax_weights, sitirax_write
from oracle import sitirax as ost


def test_window_sees_itself_and_the_tokens_before_it():
    T, window = 9, 4
    q = np.ones((T, 2, 1))
    k = np.zeros((T, 1, 1))
    v = 2.0 ** np.arange(T)[:, None, None]
    out = ost.window_attention(q, k, v, range(T), 1.0, window)       # equal scores: the mean over what is seen
    for i in range(T):
        seen = v[max(0, i - 3):i + 1, 0, 0]
        assert np.allclose(out[i], seen.mean())


def test_query_heads_share_key_heads_in_order():
    q = np.ones((1, 6, 1))
    v = np.array([10.0, 20.0, 30.0])[None, :, None]
    assert ost.window_attention(q, np.zeros((1, 3, 1)), v, [0], 1.0, 5)[0, :, 0].tolist() == [10, 10, 20, 20, 30, 30]


def test_lightning_is_a_decayed_sum_that_sees_the_current_token():
    rng = np.random.default_rng(0)
    q, k, v = rng.standard_normal((5, 1, 3)), rng.standard_normal((5, 1, 3)), rng.standard_normal((5, 1, 2))
    s = np.zeros((1, 3, 2))
    out = ost.lightning(q, k, v, [0.5], s)
    for t in range(5):
        assert np.allclose(out[t, 0], sum(0.5 ** (t - j) * (q[t, 0] @ k[j, 0]) * v[j, 0] for j in range(t + 1)))


def test_convolution_ends_at_the_current_token_and_keeps_its_last_rows():
    x = np.arange(1.0, 7.0)[:, None]
    w = np.array([[100.0, 10.0, 1.0]])
    out, rest = ost.short_convolution(x, w, np.zeros((2, 1)))
    assert out[:, 0].tolist() == [1, 12, 123, 234, 345, 456] and rest[:, 0].tolist() == [5, 6]
    out, rest = ost.short_convolution(x[:1] * 7, w, rest)
    assert out[0, 0] == 567 and rest[:, 0].tolist() == [6, 7]
    out, rest = ost.short_convolution(x, np.array([[3.0]]), np.zeros((0, 1)))
    assert out[:, 0].tolist() == [3, 6, 9, 12, 15, 18] and rest.shape == (0, 1)


def test_delta_rule_replaces_what_a_key_holds():
    k = np.zeros((3, 1, 4))
    k[0, 0, 1] = k[1, 0, 2] = k[2, 0, 1] = 1.0
    v = np.array([[1.0, 2.0], [3.0, 4.0], [5.0, 6.0]])[:, None]
    s = np.zeros((1, 4, 2))
    out = ost.delta_rule(k, k, v, np.ones((3, 1)), np.ones((3, 1, 4)), s)
    assert np.allclose(out, v)                                          # read where it was just written
    assert np.allclose(s[0], [[0, 0], [5, 6], [3, 4], [0, 0]])           # the first value of its key is gone
    s[:] = 0
    g = np.ones((3, 1, 4))
    g[2, 0, 2] = 0.25                                                   # the channel's decay acts before the write
    ost.delta_rule(k, k, v, np.array([[1.0], [1.0], [0.5]]), g, s)
    assert np.allclose(s[0], [[0, 0], [3, 4], [0.75, 1], [0, 0]])


def test_decay_per_channel_and_gelu():
    z, a, d = np.array([[[0.0, 2.0]]]), np.array([np.log(3.0)]), np.array([0.0, -2.0])
    assert np.allclose(ost.channel_decay(z, a, d), np.exp(-3.0 * np.log(2.0)))
    assert np.isclose(ost.gelu_tanh(1.0), 0.841192, atol=1e-6) and ost.gelu_tanh(0.0) == 0.0


def test_portions_of_a_sequence_give_the_whole_sequence():
    w = sitirax_weights(SITIRAX_MIXED, 3)
    toks = np.random.default_rng(1).integers(0, 67, 15).tolist()
    whole = ost.Model(SITIRAX_MIXED, w).step(toks)
    m = ost.Model(SITIRAX_MIXED, w)
    parts = np.concatenate([m.step(toks[a:b]) for a, b in ((0, 2), (2, 3), (3, 9), (9, 15))])
    assert np.allclose(whole, parts, atol=1e-10)


def test_config_reads_sizes_and_rejects_what_it_does_not_know():
    from air_hip.sitirax import DeltaMixer, SitiraxConfig, tensor_shapes

    c = SitiraxConfig.from_json(SITIRAX_MIXED)
    assert [c.owner(i) for i in range(8)] == [0, 1, 0, 3, 4, 3, 6, 7] and c.layers[1].ff is None and c.layers[3].mixer.taps == 1
    assert isinstance(c.layers[6].mixer, DeltaMixer) and c.layers[0].mixer.left.window == 37 and c.logit_scale == 0.6
    names = tensor_shapes(c)
    assert not any(n.startswith(("l2.", "l5.")) for n in names) and "l1.norm2" not in names and names["l6.mix.a1"] == (None, 72)
    chain = SitiraxConfig.from_json(sitirax_config([sitirax_delta(), sitirax_delta(weights_of=0), sitirax_delta(weights_of=1)]))
    assert chain.owner(2) == 0
    assert SitiraxConfig.from_json(sitirax_config([sitirax_delta(weights_of=1), sitirax_delta()])).owner(0) == 1
    bad = [
        sitirax_config([{**sitirax_delta(), "type": "other"}]),
        sitirax_config([{**sitirax_delta(), "mlp": {"kind": "other", "ff": 8}}]),
        sitirax_config([sitirax_delta(heads=3)]),
        sitirax_config([sitirax_parallel(heads=3)]),
        sitirax_config([sitirax_delta(conv=0)]),
        sitirax_config([sitirax_parallel(window=0)]),
        sitirax_config([sitirax_parallel(scale=0.0)]),
        sitirax_config([sitirax_parallel(decay=[0.5, 0.5])]),
        sitirax_config([sitirax_parallel(decay=[0.5, 0.5, -0.5])]),
        sitirax_config([sitirax_delta(weights_of=0)]),
        sitirax_config([sitirax_delta(weights_of=2), sitirax_delta()]),
        sitirax_config([sitirax_delta(weights_of=1), sitirax_delta(weights_of=0)]),
        sitirax_config([sitirax_delta(), sitirax_delta(dim=32, weights_of=0)]),
        sitirax_config([sitirax_delta(), sitirax_delta(ff=32, weights_of=0)]),
    ]
    for i, b in enumerate(bad):
        with pytest.raises(ValueError):
            SitiraxConfig.from_json(b)
            pytest.fail(str(i))


def _layer(w, i):
    from air_hip import sitirax

    cfg = sitirax.SitiraxConfig.from_json(SITIRAX_MIXED)
    return sitirax.SitiraxLayer(cfg, i, lambda n, s: torch.from_numpy(w[n]), torch.float32, "cpu"), cfg.layers[i]


def _input(layer, seed):
    h = np.random.default_rng(seed).standard_normal(72).astype(np.float32)
    hp = np.zeros(layer.mixer.w_in.shape[1], np.float32)
    hp[:72] = h
    return h, layer.mixer.w_in.numpy() @ hp


def test_padded_forms_of_a_parallel_layer():
    w = sitirax_weights(SITIRAX_MIXED, 5)
    for i in (0, 4, 7):
        layer, l = _layer(w, i)
        x, a, b = layer.mixer, l.mixer.left, l.mixer.right
        h, proj = _input(layer, i)
        A, s, p = x.attn, x.state, f"l{i}.mix."
        at = 0
        for name, heads, dim, dim_p in (("left.q", a.heads, a.dim, A.dim_p), ("left.k", a.kv_heads, a.dim, A.dim_p), ("left.v", a.kv_heads, a.vdim, A.vdim_p),
                                        ("right.q", b.heads, b.dim, s.dim_p), ("right.k", b.heads, b.dim, s.dim_p), ("right.v", b.heads, b.vdim, s.vdim_p),
                                        ("right.g", b.heads, b.vdim, s.vdim_p)):
            assert at == {"right.q": x.offsets[0], "right.k": x.offsets[1], "right.v": x.offsets[2], "right.g": x.gate_off}.get(name, at)
            part = proj[at:at + heads * dim_p].reshape(heads, dim_p)
            assert np.allclose(part[:, :dim], (w[p + name] @ h).reshape(heads, dim), atol=1e-5) and not part[:, dim:].any(), name
            at += heads * dim_p
        assert at == proj.shape[0] and x.silu == (x.offsets[0], x.gate_off)
        left, right = np.random.default_rng(i).standard_normal((2, 400)).astype(np.float32)
        left, right = left[:a.heads * a.vdim], right[:b.heads * b.vdim]
        out = np.zeros(x.w_o.shape[1], np.float32)
        out[:a.heads * A.vdim_p].reshape(a.heads, A.vdim_p)[:, :a.vdim] = left.reshape(a.heads, -1)
        out[a.heads * A.vdim_p:x.out_columns].reshape(b.heads, s.vdim_p)[:, :b.vdim] = right.reshape(b.heads, -1)
        assert np.allclose((x.w_o.numpy() @ out)[:72], w[p + "left.o"] @ left + w[p + "right.o"] @ right, atol=1e-4)
        norm = x.norm.numpy().reshape(b.heads, s.vdim_p)
        assert np.allclose(norm[:, :b.vdim].reshape(-1), w[p + "right.norm"] * l.mixer.right_scale) and not norm[:, b.vdim:].any()
        assert A.out_scale == l.mixer.left_scale and np.allclose(2.0 ** x.log2_decay.numpy(), b.decay)


def test_padded_forms_of_a_delta_layer():
    w = sitirax_weights(SITIRAX_MIXED, 6)
    for i in (1, 3, 6):
        layer, l = _layer(w, i)
        x, m = layer.mixer, l.mixer
        h, proj = _input(layer, i)
        s, p = x.state, f"l{i}.mix."
        assert np.allclose(proj[x.a_off:x.a_off + 20], w[p + "a1"] @ h, atol=1e-5) and np.allclose(proj[x.g_off:x.g_off + 33], w[p + "g1"] @ h, atol=1e-5)
        assert np.allclose(proj[x.b_off:x.b_off + m.heads], w[p + "b"] @ h, atol=1e-5)
        assert all(o % 16 == 0 for o in (x.a_off, x.g_off, x.b_off))
        z = x.w_a2.numpy() @ proj[x.a_off:x.g_off]
        assert np.allclose(z.reshape(m.heads, s.dim_p)[:, :m.dim].reshape(-1), w[p + "a2"] @ w[p + "a1"] @ h, atol=1e-4)
        z = x.w_g2.numpy() @ proj[x.g_off:x.b_off]
        assert np.allclose(z.reshape(m.heads, s.vdim_p)[:, :m.vdim].reshape(-1), w[p + "g2"] @ w[p + "g1"] @ h, atol=1e-4)
        assert x.conv.shape == (m.taps, s.channels)
        v = x.conv[:, 2 * s.qk_width:].reshape(m.taps, m.heads, s.vdim_p).numpy()
        assert np.array_equal(v[:, :, :m.vdim].reshape(m.taps, -1).T, w[p + "v.conv"]) and not v[:, :, m.vdim:].any()


def test_key_value_ring_is_as_long_as_the_window_and_a_portion():
    from air_hip import dense

    s = dense.HeadSpec(4, 2, 32, 32, 100, 1.0)
    assert s.ring(5000, 64) == 192 and s.ring(5000, None) == 5056 and s.ring(70, 64) == 128


def test_loader_and_registry(tmp_path):
    from air_hip import models

    assert models.entry_for({"architecture": "Sitirax"}).library == "dense_lm"
    w = sitirax_weights(SITIRAX_MIXED, 7)
    path = sitirax_write(tmp_path / "m", SITIRAX_MIXED, w)
    m = models.load_model(path, dtype=torch.float32, device="cpu")   # (weights only: no op runs on the CPU)
    assert m.vocab == 67 and m.head is m.embed and m.layers[2] is m.layers[0] and m.layers[5] is m.layers[3] and len(m.layers) == 8
    assert np.allclose(m.final_norm.numpy()[:72], 0.6 * w["final.norm"])
    cache = m.new_cache(40)
    assert len(cache.layers) == 8 and cache.layers[2]["state"] is not cache.layers[0]["state"] and cache.layers[1]["history"].shape[0] == 3
    w["l3.mix.a2"] = np.zeros((3 * 72, 8), np.float32)                # another rank than a1's
    sitirax_write(tmp_path / "m", SITIRAX_MIXED, w)
    with pytest.raises(ValueError, match="l3.mix.a2"):
        models.load_model(path, dtype=torch.float32, device="cpu")
    del w["l0.mix.right.g"]
    sitirax_write(tmp_path / "m", SITIRAX_MIXED, w)
    with pytest.raises(KeyError, match="l0.mix.right.g"):
        models.load_model(path, dtype=torch.float32, device="cpu")


def test_sizes_without_a_kernel_are_refused_when_the_model_is_made():
    from air_hip import sitirax

    for config in (sitirax_config([sitirax_delta(dim=520)]), sitirax_config([sitirax_delta(), sitirax_parallel(right_dim=520)]),
                   sitirax_config([sitirax_parallel(dim=1100, vdim=1100)])):
        w, cfg = sitirax_weights(config, 1), sitirax.SitiraxConfig.from_json(config)
        with pytest.raises(ValueError, match="layer .: no"):
            sitirax.SitiraxModel(cfg, lambda n, s: torch.from_numpy(w[n]), torch.float32, "cpu")


def test_abi_rejects_bad_arguments_before_touching_the_gpu():
    from air_hip import _lib

    lib = _lib.load_dense_library()
    buf = (ctypes.c_char * 64)()
    p = (ctypes.addressof(buf) + 15) // 16 * 16
    NULL, SHAPE, ALIGN = -1, -2, -4
    ref = ctypes.byref
    intake = lambda **k: ref(_lib.Intake(**{**dict(mode=4, res=p, final_w=p, width=64, eps=1e-5), **k}))
    act = lambda i, N=32, **k: lib.dlm_gemv_act(0, p, i, ref(_lib.RowOutput(**k)), p, 64, N, None)
    assert act(intake(), gate=3) == SHAPE and act(intake(), N=48, gate=1) == SHAPE and act(intake(), gate=1, silu_end=16) == SHAPE
    assert act(intake(res=None)) == NULL and act(intake(embed=p)) == NULL and act(intake(width=65)) == SHAPE and act(intake(final_w=None)) == NULL
    assert act(ref(_lib.Intake(mode=1, res=p, y=p, norm_w=p, width=64)), gate=1) == SHAPE
    rows = lambda **k: lib.dlm_add_norm_rows(*{**dict(dt=0, res=p, y=p, tokens=None, embed=None, scale=1.0, w=p, eps=1e-5, true=64, h=p, M=1, width=64, s=None), **k}.values())
    assert rows(res=None) == NULL and rows(tokens=p) == NULL and rows(tokens=p, embed=p) == SHAPE and rows(w=None) == NULL and rows(width=72) == SHAPE
    assert rows(true=65) == SHAPE and rows(y=p + 4) == ALIGN
    shape = dict(heads=4, kv_heads=2, dim=32, vdim=64, true_dim=24, window=40, ring=128, scale=0.2, out_scale=1.0)
    hr = dict(proj=p, q_norm=p, k_norm=p, cache=p, ld=512, off=0, M=1, pos=0, eps=1e-5)
    head = lambda sk={}, rk={}, q=p: lib.dlm_head_prepare(0, ref(_lib.HeadShape(**{**shape, **sk})), ref(_lib.HeadRows(**{**hr, **rk})), q, None)
    for k in (dict(heads=3), dict(dim=24), dict(vdim=8), dict(true_dim=33), dict(window=0), dict(ring=100), dict(scale=0.0), dict(kv_heads=0)):
        assert head(k) == SHAPE, k
    assert head(rk=dict(M=90, pos=60)) == SHAPE and head(rk=dict(M=129)) == SHAPE and head(rk=dict(off=4)) == SHAPE     # the ring is too short
    assert head(rk=dict(cache=None)) == NULL and head(q=None) == NULL and head(q=p + 2) == ALIGN
    s, r = ref(_lib.HeadShape(**shape)), ref(_lib.HeadRows(**hr))
    assert lib.dlm_head_decode(0, s, r, p, 257, p, p, None) == SHAPE and lib.dlm_head_merge(0, s, r, 0, p, p, p, 256, None) == SHAPE
    assert lib.dlm_head_merge(0, s, r, 1, p, p, p, 248, None) == SHAPE and lib.dlm_head_prefill(0, s, r, p, p, 248, None) == SHAPE
    assert not lib.dlm_head_prefill_supported(0, ref(_lib.HeadShape(**{**shape, "dim": 544}))) and lib.dlm_head_prefill_supported(0, s)
    assert not lib.dlm_head_decode_supported(1, ref(_lib.HeadShape(**{**shape, "dim": 1024, "vdim": 1024}))) and lib.dlm_head_decode_supported(1, s)
    conv = dict(proj=p, w=p, history=p, factors=p, ld=512, k_heads=2, heads=4, dim=64, vdim=32, taps=3, off=0, M=2, pos=0, q_scale=1.0, unit_eps=1e-6)
    c = lambda **k: lib.dlm_short_conv(0, ref(_lib.ShortConvArgs(**{**conv, **k})), p, None)
    assert c(taps=0) == SHAPE and c(pos_dev=p) == SHAPE and c(M=0) == SHAPE and c(off=4) == SHAPE and c(history=None) == NULL and c(w=p + 4) == ALIGN
    rec = dict(qkv=p, log2_decay=p, state=p, ld=512, k_heads=2, heads=4, dim=64, vdim=32, M=1)
    step = lambda f=lib.dlm_recurrence_steps, **k: f(0, ref(_lib.RecurrenceArgs(**{**rec, **k})), *((p,) if f == lib.dlm_recurrence_steps else (p, p)), None)
    for k in (dict(dim=32), dict(dim=576), dict(vdim=16), dict(heads=3), dict(M=0), dict(q_off=4), dict(pos=-1)):
        assert step(**k) == SHAPE and step(lib.dlm_recurrence_chunks, **k) == SHAPE, k
    assert step(log2_decay=None) == NULL and step(z=p) == NULL and step(log2_decay=None, z=p) == NULL and step(state=p + 4) == ALIGN
    assert step(lib.dlm_recurrence_chunks, dim=192) == SHAPE and lib.dlm_recurrence_chunk_bytes(ref(_lib.RecurrenceArgs(**{**rec, "dim": 192}))) == 0
    assert lib.dlm_recurrence_chunk_bytes(ref(_lib.RecurrenceArgs(**rec))) > 0
    gn = lambda **k: lib.dlm_gated_norm(*{**dict(dt=0, o=p, w=p, gate=p, ldg=64, out=p, ldo=64, M=1, groups=2, cols=32, true=32, eps=1e-5, s=None), **k}.values())
    assert gn(o=None) == NULL and gn(true=33) == SHAPE and gn(ldo=32) == SHAPE and gn(cols=30) == SHAPE and gn(M=0) == SHAPE and gn(w=p + 4) == ALIGN
    begin = lambda rk={}, ak={}, q=p: lib.dlm_head_state_begin(0, s, ref(_lib.HeadRows(**{**hr, **rk})), q, ref(_lib.RecurrenceArgs(**{**rec, **ak})), p, None)
    assert begin(rk=dict(M=2)) == SHAPE and begin(ak=dict(M=2)) == SHAPE and begin(q=None) == NULL and begin(ak=dict(vdim=8)) == SHAPE
    finish = lambda nsplit=1, cols=64, true=64, o=p: lib.dlm_head_state_end(0, s, r, nsplit, p, p, p, o, p, p, cols, true, 1e-5, p, None)
    assert finish(nsplit=0) == SHAPE and finish(cols=62) == SHAPE and finish(true=65) == SHAPE and finish(o=None) == NULL
    prod = lambda **k: ref(_lib.ShortProduct(**{**dict(w=p, x=p, out=p, K=64, N=16), **k}))
    both = lambda a=prod(), b=prod(), **k: lib.dlm_conv_products(0, ref(_lib.ShortConvArgs(**{**conv, "M": 1, **k})), p, a, b, None)
    assert both(M=2) == SHAPE and both(a=prod(K=32)) == SHAPE and both(b=prod(N=8)) == SHAPE and both(a=prod(out=None)) == NULL and both(b=prod(x=p + 2)) == ALIGN
