"""Small Fidinex models for the tests: configurations, random weights, directories, and the calls over them."""
import math

import numpy as np

import fidinex_ref as R
import nafevik_util as N
from nafevik_ref import bf16_round

rel, tokens, bf16_bits, save = N.rel, N.tokens, N.bf16_bits, N.save


def latent(heads, dim, rot_dim, vdim, rank, base=10000.0, scale=None, ff=None):
    return {"type": "latent_attention", "mlp": {"kind": "dense", "ff": ff} if ff else None,
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": rank,
                      "rot": {"dims": rot_dim, "base": base}, "scale": scale or (dim + rot_dim) ** -0.5}}


def attention(heads, kv_heads, dim, vdim, temp=None, v_mix=False, scale=None, ff=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale or dim ** -0.5, "v_mix": v_mix}
    if temp:
        m["q_temp"] = dict(zip(("coef", "every"), temp))
    return {"type": "attention", "mlp": {"kind": "dense", "ff": ff} if ff else None, "mixer": m}


def config(layers, width=80, vocab=67, streams=3, eps=1e-5):
    return {"architecture": "Fidinex", "width": width, "vocab": vocab, "streams": streams, "norm": {"eps": eps}, "layers": layers}


CONFIGS = {
    # both mixers, uneven sizes everywhere, the mixing values not in the first layer
    "mixed": config([latent(3, 20, 12, 28, 72, 500.0, ff=100), attention(6, 3, 40, 24, (0.4, 16), True, ff=72),
                     attention(4, 2, 56, 18, None, False), attention(9, 3, 36, 24, (0.2, 7), True, 0.3, ff=130),
                     latent(5, 33, 6, 17, 40, 90.0, ff=34)], width=84),
    # one stream; as many kv heads as heads; a query factor that grows at every token; no feed-forward
    "plain": config([attention(3, 3, 16, 16, (0.5, 1), False), attention(5, 5, 20, 12, None, True), latent(1, 8, 2, 4, 10)],
                    width=50, vocab=131, streams=1),
    # the latent much larger than the heads: long portions expand it
    "deep_latent": config([latent(4, 24, 8, 16, 200, 1000.0, ff=64), latent(6, 20, 20, 44, 130, 70.0)], width=128, vocab=33, streams=2),
    # more query heads per kv head than one tile of columns; the most streams
    "wide_group": config([attention(34, 2, 8, 8, (0.3, 5), True, ff=16), attention(68, 2, 24, 8, None, True, ff=48)], width=64, vocab=50, streams=8),
    # head sizes with instances of their own; the largest latent
    "big_heads": config([attention(4, 2, 128, 128, (0.3, 32), True, ff=96), attention(2, 2, 64, 128, None, True, ff=40),
                         latent(2, 128, 64, 128, 512, 20000.0, ff=40), attention(3, 1, 64, 64, (0.1, 100)),
                         attention(2, 1, 330, 250)], width=96, vocab=40, streams=5),
}


def random_model(cfg, seed, scale=1.0):
    """Seeded weights for a config, already rounded to bfloat16 values (float32 arrays)."""
    rng = np.random.default_rng(seed)
    W, S, out = cfg["width"], cfg["streams"], {}

    def mat(name, m, k, s=1.0):
        out[name] = bf16_round(rng.standard_normal((m, k)).astype(np.float32) * np.float32(scale * s / math.sqrt(k)))

    def vec(name, shape, mean=0.0, s=0.1):
        out[name] = bf16_round(np.asarray(mean + s * rng.standard_normal(shape), np.float32)).reshape(shape)

    def streams(p):
        vec(p + "in", (S,), 1.0 / S, 0.15)
        vec(p + "out", (S,), 0.6, 0.3)
        vec(p + "mix", (S, S), 0.7 * np.eye(S), 0.15)

    vec("embed", (cfg["vocab"], W), 0.0, 1.0)
    for i, L in enumerate(cfg["layers"]):
        p, mx = f"l{i}.", L["mixer"]
        H, d, dv = mx["heads"], mx["dim"], mx["vdim"]
        vec(p + "norm1", (W,), 1.0)
        streams(p + "hc1.")
        vec(p + "mix.sink", (H,), 1.0, 1.0)
        mat(p + "mix.o", W, H * dv)
        if L["type"] == "latent_attention":
            rank, r = mx["kv_rank"], mx["rot_dim"]
            mat(p + "mix.q", H * (d + r), W)
            mat(p + "mix.dkv", rank + r, W, 1.2)
            vec(p + "mix.dkv.norm", (rank,), 1.0)
            mat(p + "mix.uk", H * d, rank)
            mat(p + "mix.uv", H * dv, rank)
        else:
            G = mx["kv_heads"]
            mat(p + "mix.q", H * d, W)
            mat(p + "mix.k", G * d, W)
            mat(p + "mix.v", G * dv, W)
            vec(p + "mix.q.norm", (d,), 1.3, 0.3)
            vec(p + "mix.k.norm", (d,), 1.3, 0.3)
            vec(p + "mix.vmix", (), 0.45, 0.2)
        if L.get("mlp"):
            vec(p + "norm2", (W,), 1.0)
            streams(p + "hc2.")
            mat(p + "mlp.up", L["mlp"]["ff"], W)
            mat(p + "mlp.down", W, L["mlp"]["ff"])
    vec("final.norm", (W,), 1.0)
    return out


VECTORS = ("norm1", "norm2", ".norm", ".sink", ".vmix", ".in", ".out", ".mix")


def as_arrays(w):
    """For hip_api.LayeredModel: matrices as bf16 bits, vectors as they are."""
    return {k: v if k.endswith(VECTORS) else bf16_bits(v) for k, v in w.items()}


def reference(cfg, w, toks):
    return R.forward(cfg, w, toks)
