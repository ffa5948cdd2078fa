"""Shared input generators and comparison helpers for the parity tests."""
import numpy as np

from oracle import awq as oawq
from oracle.bf16 import bf16_bits_to_f32, f32_to_bf16_bits


def make_awq(K, N, gs=128, seed=0, z_range=(0, 16)):
    """Synthetic AWQ tensors in the benchmark distribution: q, z uniform uint4, scales = bf16(|N(0,1)|*0.02 + 1e-3)."""
    rng = np.random.default_rng(seed)
    q = rng.integers(0, 16, size=(K, N), dtype=np.uint8)
    z = rng.integers(z_range[0], z_range[1], size=(K // gs, N), dtype=np.uint8)
    s = f32_to_bf16_bits((np.abs(rng.standard_normal((K // gs, N))) * 0.02 + 1e-3).astype(np.float32))
    return oawq.pack_awq_int32(q), oawq.pack_awq_int32(z), s


def make_x(shape, seed=1):
    rng = np.random.default_rng(seed)
    return f32_to_bf16_bits(rng.standard_normal(shape).astype(np.float32))


def dense_f64(qweight, qzeros, scales, gs=128, rounded=False):
    """W[K, N] as float64: exact (q - z) * s, or the bf16-rounded weights."""
    if rounded:
        return bf16_bits_to_f32(oawq.dequant_to_bf16(qweight, qzeros, scales, gs)).astype(np.float64)
    return oawq.dequant_unrounded_f32(qweight, qzeros, scales, gs).astype(np.float64)


def bf16_ulp(v):
    """Spacing of bf16 numbers at magnitude |v| (float64 array)."""
    a = np.maximum(np.abs(np.asarray(v, dtype=np.float64)), 2.0**-126)
    return 2.0 ** (np.floor(np.log2(a)) - 7)


def assert_bf16_close(actual_bits, want_f64, ulps=1.0, atol=0.0, what=""):
    """|actual - want| <= ulps * ulp_bf16(want) + atol, elementwise."""
    got = bf16_bits_to_f32(np.asarray(actual_bits)).astype(np.float64).reshape(np.shape(want_f64))
    err = np.abs(got - want_f64)
    tol = ulps * bf16_ulp(want_f64) + atol
    bad = err > tol
    assert not bad.any(), (
        f"{what}: {int(bad.sum())}/{bad.size} elements outside {ulps} bf16 ulp + {atol}; "
        f"worst err {err.max():.4g} at {np.unravel_index(np.argmax(err - tol), err.shape)}")


# ---- Kuvonex ------------------------------------------------------------------------------------------------------------
def kuvonex_layer(heads=3, dim=24, rot_dim=8, vdim=40, kv_rank=56, kv_from=None, base=500.0, scale=None, mlp=None):
    """One entry of `layers` of a Kuvonex config.json.  mlp: (experts, top, groups, keep, ff) or None."""
    mixer = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank,
             "scale": (dim + rot_dim) ** -0.5 if scale is None else scale, "rot": {"base": base, "dims": rot_dim}}
    if kv_from is not None:
        mixer["kv_from"] = kv_from
    if mlp is not None:
        experts, top, groups, keep, ff = mlp
        mlp = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top, "groups": {"count": groups, "keep": keep}}}
    return {"type": "latent_attention", "mixer": mixer, "mlp": mlp}


def kuvonex_config(layers, vocab=67, width=72, eps=1e-5, embed_scale=1.7):
    return {"architecture": "Kuvonex", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": embed_scale}, "layers": layers}


def kuvonex_weights(config, seed=0):
    """Random weights as float32 arrays that hold bf16 values, by checkpoint name."""
    from air_hip import kuvonex

    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in kuvonex.tensor_shapes(kuvonex.KuvonexConfig.from_json(config)).items():
        if name.endswith("norm") or name.endswith("norm1") or name.endswith("norm2"):
            v = 1.0 + 0.3 * rng.standard_normal(shape)
        elif name.endswith("sink"):
            v = 1.5 * rng.standard_normal(shape)
        elif name.endswith("correction"):
            v = -0.6 + 0.5 * rng.standard_normal(shape)    # choice scores of either sign
        elif name == "embed":
            v = rng.standard_normal(shape) * 0.6
        else:
            v = rng.standard_normal(shape) * shape[-1] ** -0.5
            if name.endswith("router"):
                v *= 2.0                                     # scores well apart
        out[name] = bf16_bits_to_f32(f32_to_bf16_bits(v.astype(np.float32)))
    return out


def kuvonex_write(path, config, weights):
    """The checkpoint directory (config.json, model.safetensors)."""
    import json
    import os

    import torch
    from safetensors.torch import save_file

    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(config, f)
    save_file({k: torch.from_numpy(v).to(torch.bfloat16).contiguous() for k, v in weights.items()}, os.path.join(path, "model.safetensors"))
    return str(path)


# Layers that differ in every size, one without a feed-forward, one that attends over an earlier layer's cache with other
# head sizes than its source; groups of one, of two and no grouping at all.
KUVONEX_MIXED = kuvonex_config([
    kuvonex_layer(mlp=(12, 3, 3, 2, 40)),
    kuvonex_layer(heads=2, dim=40, rot_dim=12, vdim=16, kv_rank=72, base=90.0),
    kuvonex_layer(heads=5, dim=16, rot_dim=8, vdim=24, kv_rank=56, kv_from=0, scale=0.31, mlp=(6, 2, 6, 3, 72)),
    kuvonex_layer(heads=1, dim=8, rot_dim=12, vdim=8, kv_rank=72, base=90.0, kv_from=1, mlp=(4, 2, 1, 1, 8)),
], vocab=67, width=72)


# ---- Sitirax ------------------------------------------------------------------------------------------------------------
def sitirax_parallel(heads=4, kv_heads=2, dim=24, vdim=40, window=37, scale=None, right_heads=3, right_dim=40, right_vdim=24, decay=None, left_scale=0.7,
                     right_scale=1.3, ff=None, weights_of=None):
    """One 'parallel' entry of `layers` of a Sitirax config.json."""
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": dim ** -0.5 if scale is None else scale, "mask": {"size": window}}
    right = {"heads": right_heads, "dim": right_dim, "vdim": right_vdim, "decay": list(decay or np.linspace(0.4, 1.0, right_heads))}
    return _sitirax_layer("parallel", {"left": left, "right": right, "left_scale": left_scale, "right_scale": right_scale}, ff, weights_of)


def sitirax_delta(heads=4, kv_heads=2, dim=24, vdim=40, conv=3, ff=None, weights_of=None):
    """One 'channel_delta' entry."""
    return _sitirax_layer("channel_delta", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}, ff, weights_of)


def _sitirax_layer(kind, mixer, ff, weights_of):
    out = {"type": kind, "mixer": mixer, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}
    if weights_of is not None:
        out["weights_of"] = weights_of
    return out


def sitirax_config(layers, vocab=67, width=72, eps=1e-5, logit_scale=0.6):
    return {"architecture": "Sitirax", "vocab": vocab, "width": width, "norm": {"eps": eps}, "logit_scale": logit_scale, "layers": layers}


def sitirax_weights(config, seed=0, ranks=(20, 33)):
    """Random weights as float32 arrays that hold bf16 values, by checkpoint name; ranks: of the decay's and the gate's two factors."""
    from air_hip import sitirax

    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in sitirax.tensor_shapes(sitirax.SitiraxConfig.from_json(config)).items():
        shape = tuple((ranks[0] if ".a" in name else ranks[1]) if n is None else n for n in shape)
        v = rng.standard_normal(shape)
        if name.endswith(("norm", "norm1", "norm2")):
            v = 1.0 + 0.3 * v
        elif name.endswith("A_log"):
            v = 0.7 * v - 1.0
        elif name.endswith("dt_bias"):
            v = 2.0 * v - 1.0                # channels that forget at once and channels that hardly do
        elif name == "embed":
            v = v * 0.8
        else:
            v = v * shape[-1] ** -0.5 * (1.5 if ".b" in name or ".a" in name else 1.0)
        out[name] = bf16_bits_to_f32(f32_to_bf16_bits(v.astype(np.float32)))
    return out


sitirax_write = kuvonex_write

# Every size different; shared weights of either kind, with and without a feed-forward; a window of one, a convolution of one tap,
# one key / value head for all, heads of more than 64 channels.
SITIRAX_MIXED = sitirax_config([
    sitirax_parallel(ff=40),
    sitirax_delta(),
    sitirax_parallel(ff=40, weights_of=0),
    sitirax_delta(heads=3, kv_heads=3, dim=72, vdim=16, conv=1, ff=72),
    sitirax_parallel(heads=5, kv_heads=1, dim=8, vdim=8, window=1, right_heads=1, right_dim=8, right_vdim=72, decay=[0.999], left_scale=-0.4, right_scale=1.0),
    sitirax_delta(heads=3, kv_heads=3, dim=72, vdim=16, conv=1, ff=72, weights_of=3),
    sitirax_delta(heads=2, kv_heads=1, dim=40, vdim=72, conv=5),
    sitirax_parallel(heads=2, kv_heads=2, dim=72, vdim=24, window=70, scale=0.4, right_heads=4, right_dim=72, right_vdim=8, ff=24),
], vocab=67, width=72)
