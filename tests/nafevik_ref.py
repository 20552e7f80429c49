"""Plain numpy statement of the Nafevik decoder, one function per mechanism, float64 throughout.

Test infrastructure only: whole sequences at once, no cache, no batching, nothing shared with the
product's loader, model or kernels.  ``weights`` maps tensor names to float arrays; ``cfg`` is the
parsed config.json.
"""
from __future__ import annotations

import math

import numpy as np

F = np.float64


def rms_norm(x, w, eps):
    ms = np.mean(np.square(x), axis=-1, keepdims=True)
    return x / np.sqrt(ms + eps) * w


def causal_conv(h, w):
    """Depthwise over time: out[t, c] = sum_j w[c, j] h[t - taps + 1 + j, c], zero before t = 0."""
    n, taps = h.shape[0], w.shape[1]
    out = np.zeros_like(h)
    for t in range(n):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                out[t] += w[:, j] * h[s]
    return out


def rotary_frequencies(rot):
    """Per-pair angular frequency and the common magnitude of cos and sin (YaRN blending)."""
    dims, base = int(rot["dims"]), float(rot["base"])
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return np.array(f, F), 1.0
    factor, original = float(sc["factor"]), float(sc["original"])

    def dim_of(turns):
        return dims * math.log(original / (2 * math.pi * turns)) / (2 * math.log(base))

    lo = max(math.floor(dim_of(float(sc["fast"]))), 0)
    hi = min(math.ceil(dim_of(float(sc["slow"]))), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / factor * ramp + fi * (1.0 - ramp))
    return np.array(out, F), 0.1 * math.log(factor) + 1.0


def rotate(x, positions, rot):
    """x [n, heads, dim]: adjacent pairs of the first rot.dims columns turn by position * frequency."""
    if not rot:
        return x
    freq, mag = rotary_frequencies(rot)
    out = np.array(x, F)
    for i, f in enumerate(freq):
        a = np.asarray(positions, F) * f
        c, s = (np.cos(a) * mag)[:, None], (np.sin(a) * mag)[:, None]
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def sigmoid(z):
    e = np.exp(-np.abs(z))
    return np.where(z >= 0, 1.0 / (1.0 + e), e / (1.0 + e))


def visible(n, size):
    """[query, key]: causal, and both in the same chunk of `size` positions (None: no chunks)."""
    i, j = np.arange(n)[:, None], np.arange(n)[None, :]
    ok = j <= i
    return ok & (i // size == j // size) if size else ok


def sigmoid_attention(q, k, v, scale, bias, size):
    """q [n, H, d], k [n, G, d], v [n, G, dv] -> [n, H, dv]: unnormalised sigmoid weights."""
    n, H, _ = q.shape
    per = H // k.shape[1]
    ok = visible(n, size)
    out = np.zeros((n, H, v.shape[2]), F)
    for h in range(H):
        s = q[:, h] @ k[:, h // per].T * scale + bias[h]
        out[:, h] = np.where(ok, sigmoid(s), 0.0) @ v[:, h // per]
    return out


def attention_mixer(h, p, w, mx):
    n = h.shape[0]
    H, G, d, dv = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    pos = np.arange(n)
    q = rotate((h @ w[p + "q"].T).reshape(n, H, d), pos, mx.get("rot"))
    k = rotate((h @ w[p + "k"].T).reshape(n, G, d), pos, mx.get("rot"))
    v = (h @ w[p + "v"].T).reshape(n, G, dv)
    size = (mx.get("mask") or {}).get("size")
    o = sigmoid_attention(q, k, v, mx["scale"], w[p + "pb"], size)
    o = o * sigmoid(h @ w[p + "g"].T)[:, :, None]
    return o.reshape(n, H * dv) @ w[p + "o"].T


def silu(z):
    return z * sigmoid(z)


def dense_ff(h, p, w):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def layer(x, i, w, cfg):
    spec, p = cfg["layers"][i], f"l{i}."
    h = rms_norm(x, w[p + "norm1"], cfg["norm"]["eps"])
    y = attention_mixer(h + causal_conv(h, w[p + "canon1"]), p + "mix.", w, spec["mixer"])
    if spec.get("mlp"):
        y = y + dense_ff(h + causal_conv(h, w[p + "canon2"]), p + "mlp.", w)
    return x + cfg["residual_mult"] * y


def layer_runs(cfg):
    """(layer index, pass number or None) in execution order; a pass number only on its first layer."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, None) for i in range(n)]
    a, b = lp["start"], lp["stop"]
    runs = [(i, None) for i in range(a)]
    for t in range(lp["times"]):
        runs += [(i, t if i == a else None) for i in range(a, b)]
    return runs + [(i, None) for i in range(b, n)]


def forward(cfg, weights, tokens, collect=None):
    """Logits [n, vocab] of a whole sequence; `collect` (a list) receives the residual after every layer run."""
    w = {k: np.asarray(v, F) for k, v in weights.items()}
    tokens = np.asarray(tokens, int)
    x0 = w["embed"][tokens] + w["pos"][:len(tokens)]
    x = x0
    for i, t in layer_runs(cfg):
        if t is not None:
            x = np.concatenate([x, x0], axis=1) @ w["loop.in"].T + w["loop.step"][t]
        x = layer(x, i, w, cfg)
        if collect is not None:
            collect.append(x.copy())
    return rms_norm(x, w["final.norm"], cfg["norm"]["eps"]) @ w["head"].T


def random_model(cfg, seed, scale=1.0):
    """Seeded weights for a config, already rounded to bfloat16 values (float32 arrays)."""
    rng = np.random.default_rng(seed)
    W, V, taps = cfg["width"], cfg["vocab"], cfg["canon"]["taps"]
    out = {}

    def mat(name, m, k, s=1.0):
        out[name] = bf16_round(rng.standard_normal((m, k)).astype(np.float32) * np.float32(scale * s / math.sqrt(k)))

    def vec(name, shape, mean=0.0, s=0.1):
        out[name] = bf16_round((mean + s * rng.standard_normal(shape)).astype(np.float32))

    vec("embed", (V, W), 0.0, 1.0)
    vec("pos", (cfg["max_positions"], W), 0.0, 0.5)
    if cfg.get("loop"):
        mat("loop.in", W, 2 * W, 1.4)
        vec("loop.step", (cfg["loop"]["times"], W), 0.0, 0.5)
    for i, L in enumerate(cfg["layers"]):
        p, mx = f"l{i}.", L["mixer"]
        vec(p + "norm1", (W,), 1.0)
        vec(p + "canon1", (W, taps), 0.0, 0.4)
        H, G = mx["heads"], mx["kv_heads"]
        mat(p + "mix.q", H * mx["dim"], W, 1.5)
        mat(p + "mix.k", G * mx["dim"], W, 1.5)
        mat(p + "mix.v", G * mx["vdim"], W)
        vec(p + "mix.pb", (H,), -2.0, 0.7)
        mat(p + "mix.g", H, W, 1.5)
        mat(p + "mix.o", W, H * mx["vdim"])
        if L.get("mlp"):
            vec(p + "canon2", (W, taps), 0.0, 0.4)
            ff = L["mlp"]["ff"]
            mat(p + "mlp.gate", ff, W)
            mat(p + "mlp.up", ff, W)
            mat(p + "mlp.down", W, ff)
    vec("final.norm", (W,), 1.0)
    mat("head", V, W)
    return out


def bf16_round(x):
    b = np.ascontiguousarray(x, np.float32).view(np.uint32)
    r = (b + 0x7FFF + ((b >> 16) & 1)) & np.uint32(0xFFFF0000)
    return r.view(np.float32)
