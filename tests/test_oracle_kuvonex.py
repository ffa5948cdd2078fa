"""The plain Kuvonex implementation against hand-made cases, and the product's configuration, loader, registry, token loop
and trace replay on the host (CPU only)."""
import io
import json

import numpy as np
import pytest
import torch

from helpers import KUVONEX_MIXED, kuvonex_config, kuvonex_layer, kuvonex_weights, kuvonex_write
from oracle import kuvonex as okv


def test_rotation_turns_neighbouring_pairs_and_keeps_relative_positions():
    v = np.zeros((1, 4))
    v[0, 2] = 1.0                                     # second pair, angle p * base^(-1/2)
    out = okv.rotate_interleaved(v, [3], base=100.0)
    assert np.allclose(out[0], [0, 0, np.cos(0.3), np.sin(0.3)])
    rng = np.random.default_rng(0)
    q, k = rng.standard_normal((2, 1, 6))
    dot = lambda i, j: float(okv.rotate_interleaved(q, [i], 50.0)[0] @ okv.rotate_interleaved(k, [j], 50.0)[0])
    assert np.isclose(dot(7, 4), dot(103, 100)) and not np.isclose(dot(7, 4), dot(7, 5))


def test_sink_counts_once_in_the_denominator():
    p = okv.sink_softmax(np.log(np.array([1.0, 2.0])), np.log(5.0))
    assert np.allclose(p, [1 / 8, 2 / 8])
    assert np.allclose(okv.sink_softmax(np.array([3.0, 1.0]), 900.0), 0.0)


def test_router_by_hand():
    logit = lambda s: np.log(s / (1 - s))
    s = np.array([0.9, 0.1, 0.5, 0.6, 0.2, 0.95])
    w = np.diag(logit(s))                              # h = ones -> the logits themselves
    # groups (0, 1), (2, 3), (4, 5): sums 1.0, 1.1, 1.15
    ids, wt = okv.route(np.ones(6), w, np.zeros(6), top=2, groups=3, keep=1)
    assert ids == [5, 4] and np.allclose(wt, [0.95, 0.2])
    ids, wt = okv.route(np.ones(6), w, np.zeros(6), top=3, groups=3, keep=2)
    assert ids == [5, 3, 2] and np.allclose(wt, [0.95, 0.6, 0.5])
    # the correction moves the choice, not the weight; all choice scores may be negative
    c = np.array([0.0, 0.0, 0.0, 0.0, 2.0, 0.0]) - 5.0
    ids, wt = okv.route(np.ones(6), w, c, top=2, groups=3, keep=2)
    assert ids == [4, 5] and np.allclose(wt, [0.2, 0.95])
    ids, _ = okv.route(np.ones(6), w, np.zeros(6) - 5.0, top=2, groups=6, keep=2)   # groups of one
    assert ids == [5, 0]


def test_portions_of_a_sequence_give_the_whole_sequence():
    w = kuvonex_weights(KUVONEX_MIXED, 3)
    toks = np.random.default_rng(1).integers(0, 67, 15).tolist()
    whole = okv.Model(KUVONEX_MIXED, w).step(toks)
    m = okv.Model(KUVONEX_MIXED, w)
    parts = np.concatenate([m.step(toks[a:b]) for a, b in ((0, 2), (2, 3), (3, 9), (9, 15))])
    assert np.allclose(whole, parts, atol=1e-10)


def test_config_reads_sizes_and_rejects_what_it_does_not_know():
    from air_hip.kuvonex import KuvonexConfig

    c = KuvonexConfig.from_json(KUVONEX_MIXED)
    assert [l.mlp is None for l in c.layers] == [False, True, False, False]
    assert c.layers[2].mixer.kv_from == 0 and c.layers[2].mixer.heads == 5 and c.layers[0].mlp.groups == 3
    bad = [
        kuvonex_config([{**kuvonex_layer(), "type": "other"}]),
        kuvonex_config([kuvonex_layer(), kuvonex_layer(kv_from=1)]),                       # itself
        kuvonex_config([kuvonex_layer(), kuvonex_layer(kv_from=0), kuvonex_layer(kv_from=1)]),   # has no latent
        kuvonex_config([kuvonex_layer(), kuvonex_layer(kv_from=0, kv_rank=64)]),
        kuvonex_config([kuvonex_layer(), kuvonex_layer(kv_from=0, base=9.0)]),
        kuvonex_config([kuvonex_layer(rot_dim=7)]),
        kuvonex_config([kuvonex_layer(mlp=(8, 5, 4, 2, 16))]),                             # two groups of two give four
        kuvonex_config([kuvonex_layer(mlp=(8, 2, 3, 2, 16))]),
    ]
    for b in bad:
        with pytest.raises(ValueError):
            KuvonexConfig.from_json(b)


def test_padded_layer_forms_keep_every_weight_in_its_place():
    from air_hip import dense, kuvonex

    w = kuvonex_weights(KUVONEX_MIXED, 5)
    cfg = kuvonex.KuvonexConfig.from_json(KUVONEX_MIXED)
    for i, l in enumerate(cfg.layers):
        layer = kuvonex.prepare_layer(cfg, i, lambda n, s: torch.from_numpy(w[n].reshape(s)), torch.float32, "cpu")
        s, m = layer.spec, l.mixer
        assert s.dim_p % 32 == s.rot_p % 32 == s.vdim_p % 32 == s.rank_p % 64 == layer.w_in.shape[1] % 64 == 0
        h = np.random.default_rng(i).standard_normal(cfg.width).astype(np.float32)
        hp = np.zeros(layer.w_in.shape[1], np.float32)
        hp[:cfg.width] = h
        proj = layer.w_in.numpy() @ hp
        q = proj[:s.heads * (s.dim_p + s.rot_p)].reshape(s.heads, -1)
        want = (w[f"l{i}.mix.q"] @ h).reshape(m.heads, -1)
        assert np.allclose(q[:, :m.dim], want[:, :m.dim], atol=1e-5) and np.allclose(q[:, s.dim_p:s.dim_p + m.rot_dim], want[:, m.dim:], atol=1e-5)
        assert not q[:, m.dim:s.dim_p].any() and not q[:, s.dim_p + m.rot_dim:].any()
        g = proj[layer.gate_off:].reshape(s.heads, -1)
        assert np.allclose(g[:, :m.vdim], (w[f"l{i}.mix.g"] @ h).reshape(m.heads, -1), atol=1e-5)
        if m.kv_from is None:
            kv = proj[layer.kv_off:layer.gate_off]
            assert np.allclose(kv[:m.kv_rank], (w[f"l{i}.mix.dkv"] @ h)[:m.kv_rank], atol=1e-5)
            assert np.allclose(kv[s.rank_p:s.rank_p + m.rot_dim], (w[f"l{i}.mix.dkv"] @ h)[m.kv_rank:], atol=1e-5)
        else:
            assert layer.kv_off == -1 and layer.source == m.kv_from
        a = np.random.default_rng(i).standard_normal((m.heads, m.vdim)).astype(np.float32)
        ap = np.zeros((s.heads, s.vdim_p), np.float32)
        ap[:, :m.vdim] = a
        ap = np.pad(ap.reshape(-1), (0, s.out_width - s.heads * s.vdim_p))
        assert np.allclose((layer.w_o.numpy() @ ap)[:cfg.width], w[f"l{i}.mix.o"] @ a.reshape(-1), atol=1e-5)
        if l.mlp is not None:
            gu = layer.w_gate_up.numpy().reshape(l.mlp.experts, -1, 2, 16, layer.w_in.shape[1])
            gate = gu[:, :, 0].reshape(l.mlp.experts, -1, gu.shape[-1])
            assert np.array_equal(gate[1, :l.mlp.ff, :cfg.width], w[f"l{i}.mlp.e1.gate"]) and not gate[:, l.mlp.ff:].any()
            assert dense.pad_to(l.mlp.ff, 64) == gate.shape[1]


def test_loader_reads_a_directory_and_names_what_is_wrong(tmp_path):
    from air_hip import models

    w = kuvonex_weights(KUVONEX_MIXED, 7)
    path = kuvonex_write(tmp_path / "m", KUVONEX_MIXED, w)
    m = models.load_model(path, dtype=torch.float32, device="cpu")   # (weights only: no op runs on the CPU)
    assert m.vocab == 67 and np.array_equal(m.embed.numpy()[:67, :72], w["embed"]) and m.head.shape == (80, 128)
    del w["l2.mlp.e3.up"]
    kuvonex_write(tmp_path / "m", KUVONEX_MIXED, w)
    with pytest.raises(KeyError, match="l2.mlp.e3.up"):
        models.load_model(path, dtype=torch.float32, device="cpu")
    w["l2.mlp.e3.up"] = np.zeros((5, 5), np.float32)
    kuvonex_write(tmp_path / "m", KUVONEX_MIXED, w)
    with pytest.raises(ValueError, match="l2.mlp.e3.up"):
        models.load_model(path, dtype=torch.float32, device="cpu")


def test_registry_chooses_by_architecture():
    from air_hip import models

    assert models.entry_for({"architecture": "Kuvonex"}).library == "dense_lm"
    assert models.entry_for({"architectures": ["LlamaForCausalLM"]}).cls == "LlamaModel"
    with pytest.raises(ValueError, match="Unheard"):
        models.entry_for({"architecture": "Unheard"})
    with pytest.raises(ValueError):
        models.entry_for({})


def test_llama_config_from_hf_json():
    from air_hip.weights import LlamaConfig

    c = LlamaConfig.from_hf({"num_hidden_layers": 2, "hidden_size": 256, "num_attention_heads": 4, "num_key_value_heads": 2, "intermediate_size": 512,
                             "vocab_size": 99, "rope_theta": 1e4, "rms_norm_eps": 1e-6})
    assert c == LlamaConfig(2, 256, 4, 64, 2, 512, 99, 1e4, 1e-6)


class _Counting:
    """A model whose logits at position p after token t are one-hot at (t + p) mod vocab: shows which cache and position a
    step ran with."""

    vocab, device = 11, "cpu"

    class Cache:
        def __init__(self, n):
            self.capacity, self.pos = n, 0

        def reset(self):
            self.pos = 0

    def __init__(self):
        self.made = 0

    def new_cache(self, n):
        self.made += 1
        return self.Cache(n)

    def step(self, cache, tokens, want):
        out = torch.zeros((len(want), self.vocab))
        for i, w in enumerate(want):
            out[i, (tokens[w] + cache.pos + w) % self.vocab] = 1.0
        cache.pos += len(tokens)
        return out

    def _one(self, cache, token):
        logits = self.step(cache, [token], [0])[0]
        return logits, logits.argmax().to(torch.int32).reshape(1)

    def prefill(self, cache, tokens):
        logits = self.step(cache, tokens, [len(tokens) - 1])[0]
        return logits, logits.argmax().to(torch.int32).reshape(1)

    decode_token = _one

    def decode_greedy(self, cache, first, n):
        out, tok = [], int(first.item())
        for _ in range(n):
            _, best = self._one(cache, tok)
            tok = int(best.item())
            out.append(tok)
        return torch.tensor(out, dtype=torch.int32)

    def check_health(self):
        pass


def test_token_loop_streams_stops_and_reuses_its_cache():
    from air_hip.generation import generate

    m = _Counting()
    whole = generate(m, [3, 5], 6)
    assert whole[0] == (5 + 1) % 11 and whole[1] == (whole[0] + 2) % 11 and len(whole) == 7
    seen = []
    assert generate(m, [3, 5], 6, on_token=seen.append) == whole == seen
    stop = whole[3]
    assert generate(m, [3, 5], 6, eos_token_ids=(stop,)) == whole[:whole.index(stop, 1) + 1]
    cache = m.new_cache(8)
    assert generate(m, [3, 5], 6, cache=cache) == generate(m, [3, 5], 6, cache=cache) == whole
    assert generate(m, [3, 5], 0) == whole[:1]
    with pytest.raises(ValueError):
        generate(m, [], 3)


def test_trace_replay_keeps_requests_apart_and_reuses_ended_caches(tmp_path):
    from air_hip import trace

    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": [1, 2, 3], "want": [0, 2]}], "end": []},
        {"step": 1, "entries": [{"id": "b", "tokens": [4, 4], "want": []}], "end": []},
        {"step": 2, "entries": [{"id": "a", "tokens": [5], "want": [0]}, {"id": "b", "tokens": [6], "want": [0]}], "end": ["a"]},
        {"step": 3, "entries": [{"id": "c", "tokens": [7], "want": [0]}], "end": ["b", "c"]},
    ]
    m, said = _Counting(), []
    trace.replay(m, io.StringIO("\n".join(json.dumps(s) for s in steps) + "\n\n"), str(tmp_path), 16, said.append)
    assert said == ["done 0", "done 1", "done 2", "done 3"] and m.made == 2
    read = lambda n: np.fromfile(tmp_path / f"{n}.f32", "<f4").reshape(-1, 11).argmax(1).tolist()
    assert read(0) == [1, 5] and read(2) == [8, 8] and read(3) == [7]
    assert not (tmp_path / "1.f32").exists()


def test_dense_abi_rejects_bad_arguments_before_touching_the_gpu():
    import ctypes
    import os
    import re

    from air_hip import _lib

    lib = _lib.load_dense_library()
    header = open(os.path.join(os.path.dirname(__file__), "..", "include", "dense_lm.h")).read()
    declared = set(re.findall(r"\b(dlm_\w+)\(", re.sub(r"/\*.*?\*/", "", header, flags=re.S)))
    assert declared == set(_lib.DENSE_SYMBOLS)
    buf = (ctypes.c_char * 64)()
    p = (ctypes.addressof(buf) + 15) // 16 * 16
    NULL, SHAPE, ALIGN = -1, -2, -4
    i = _lib.Intake(mode=0, x=p)
    g = lambda inp=i, w=p, out=p, K=64, N=16, dt=0: lib.dlm_gemv(dt, w, ctypes.byref(inp), out, None, None, 0, K, N, None)
    assert g(w=None) == NULL and g(out=None) == NULL and g(K=40) == SHAPE and g(N=0) == SHAPE and g(dt=2) == SHAPE and g(w=p + 2) == ALIGN
    assert g(inp=_lib.Intake(mode=0)) == NULL and g(inp=_lib.Intake(mode=9)) == SHAPE
    assert g(inp=_lib.Intake(mode=1, res=p, y=p, norm_w=p, width=65)) == SHAPE
    r = lambda **k: ctypes.byref(_lib.Router(**{**dict(logits=p, correction=p, ld=16, experts=12, top=2, groups=3, keep=1), **k}))
    s = lambda q: lib.dlm_moe_select(q, 1, p, p, None)
    for k in (dict(groups=5), dict(top=5), dict(keep=4), dict(ld=11), dict(experts=0), dict(top=0)):
        assert s(r(**k)) == SHAPE, k
    assert s(r(logits=None)) == NULL
    a = lambda **k: lib.dlm_gemm(0, ctypes.byref(_lib.GemmArgs(**{**dict(a=p, w=p, out=p, lda=64, ldo=32, M=3, N=32, K=64, tile_rows=32), **k})), None)
    for k in (dict(K=96 - 8), dict(N=24), dict(lda=56), dict(ldo=16), dict(M=0), dict(tile_rows=64), dict(epilogue=4), dict(epilogue=2, N=16), dict(epilogue=3, N=48),
              dict(silu_begin=0, silu_end=8), dict(silu_begin=0, silu_end=16, epilogue=1)):
        assert a(**k) == SHAPE, k
    assert a(tiles=p) == NULL and a(tiles=p, order=p, n_tiles=1, w_stride=5) == SHAPE
    shape = dict(heads=2, dim=32, rot=32, vdim=32, rank=64, rot_pairs=4, true_rank=64, scale=1.0)
    rows = dict(proj=p, lut=p, cache=p, ld=128, kv_off=-1, gate_off=128, M=1)
    l = lambda sk={}, rk={}: lib.dlm_latent_prepare(0, ctypes.byref(_lib.LatentShape(**{**shape, **sk})), ctypes.byref(_lib.LatentRows(**{**rows, **rk})), None)
    for k in (dict(dim=24), dict(rank=96), dict(rot_pairs=17), dict(scale=0.0), dict(vdim=0), dict(true_rank=65)):
        assert l(k) == SHAPE, k
    assert l(rk=dict(M=0)) == SHAPE and l(rk=dict(kv_off=0)) == NULL and l(rk=dict(proj=None)) == NULL
    assert not lib.dlm_latent_decode_supported(0, ctypes.byref(_lib.LatentShape(**{**shape, "rank": 2048})))
