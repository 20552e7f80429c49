"""Small Nafevik models on disk for the tests: config.json + model.safetensors."""
import json
import struct
from pathlib import Path

import numpy as np

import nafevik_ref as R


def attention(heads, kv_heads, dim, vdim, size=None, rot_dims=None, base=10000.0, scaling=None, scale=None, ff=None):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale or dim ** -0.5}
    if size:
        mixer["mask"] = {"size": size}
    if rot_dims:
        mixer["rot"] = {"dims": rot_dims, "base": base}
        if scaling:
            mixer["rot"]["scaling"] = scaling
    return {"type": "attention", "mixer": mixer, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def config(layers, width=80, vocab=67, taps=4, loop=None, positions=512, mult=0.6, eps=1e-5):
    c = {"architecture": "Nafevik", "width": width, "vocab": vocab, "canon": {"taps": taps}, "norm": {"eps": eps},
         "residual_mult": mult, "max_positions": positions, "layers": layers}
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


def bf16_bits(x):
    b = np.ascontiguousarray(x, np.float32).view(np.uint32)
    assert not (b & 0xFFFF).any(), "weights must be bf16 values already"
    return (b >> 16).astype(np.uint16)


def save(path: Path, cfg, weights, dtypes=None):
    path.mkdir(parents=True, exist_ok=True)
    (path / "config.json").write_text(json.dumps(cfg))
    header, blobs, off = {}, [], 0
    for name, w in weights.items():
        raw = bf16_bits(w).tobytes()
        header[name] = {"dtype": (dtypes or {}).get(name, "BF16"), "shape": list(w.shape), "data_offsets": [off, off + len(raw)]}
        blobs.append(raw)
        off += len(raw)
    h = json.dumps(header).encode()
    (path / "model.safetensors").write_bytes(struct.pack("<Q", len(h)) + h + b"".join(blobs))
    return path


YARN = {"factor": 4.0, "original": 64, "fast": 8.0, "slow": 0.5}

# Sizes that differ from one another wherever the design lets them, and the special values
CONFIGS = {
    # grouped heads, looped middle, value size other than the key size, partly rotated heads
    "mixed": config([attention(4, 2, 40, 24, 33, 24, 3000.0, YARN, ff=100), attention(6, 3, 32, 56, 50, 32, 500.0, None, ff=72),
                     attention(2, 1, 48, 48, 20, 16, 900.0, YARN, scale=0.3, ff=130)], width=84, vocab=67, taps=4, loop=(1, 3, 3)),
    # no loop, one tap, a layer without a feed-forward, as many kv heads as heads, no chunks, no rotation
    "plain": config([attention(3, 3, 16, 16), attention(5, 5, 20, 12, None, 20, 100.0, ff=33)], width=50, vocab=131, taps=1, mult=1.0),
    # the loop covers everything, once; two taps; ramp of the rotation collapsed to a step
    "once": config([attention(8, 2, 64, 64, 40, 64, 10000.0, {"factor": 16.0, "original": 8, "fast": 32.0, "slow": 30.0}, ff=64)],
                   width=128, vocab=33, taps=2, loop=(0, 1, 1)),
    # more query heads per kv head than one tile of columns; loop at the end
    "wide_group": config([attention(4, 4, 24, 40, 64, 8, 50.0, ff=48), attention(34, 2, 8, 8, 25, 8, 77.0, None, ff=16)],
                         width=64, vocab=50, taps=7, loop=(1, 2, 2)),
    # the largest head sizes; sizes that have instances of their own
    "big_heads": config([attention(2, 1, 256, 160, 70, 128, 20000.0, YARN, ff=96), attention(3, 1, 96, 96, 37, 64, 1000.0, ff=40),
                         attention(2, 2, 128, 128, 90, 128, 1000.0, YARN, ff=40)], width=96, vocab=40, taps=3, loop=(0, 2, 2)),
}


def tokens(cfg, n, seed):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n)


def rel(got, want):
    """rms of the difference over the rms of the expected logits, worst position."""
    d = np.sqrt(np.mean(np.square(np.asarray(got, np.float64) - want), axis=-1))
    return float(np.max(d / np.sqrt(np.mean(np.square(want)))))


def reference(cfg, w, toks):
    return R.forward(cfg, w, toks)
