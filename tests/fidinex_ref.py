"""Plain numpy statement of the Fidinex decoder, one function per mechanism, float64 throughout.

Test infrastructure only: whole sequences at once, no cache, no batching, nothing shared with the
product's loader, model or kernels.  ``weights`` maps tensor names to float arrays; ``cfg`` is the
parsed config.json.
"""
from __future__ import annotations

import math

import numpy as np

F = np.float64


def rms_norm(x, w, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def rotate_pairs(x, positions, base, dims):
    """x [n, heads, d]: the pairs (2i, 2i + 1) of the first `dims` entries turn by position * base^(-2i / dims)."""
    y = np.array(x, F)
    for i in range(dims // 2):
        a = np.asarray(positions, F)[:, None] * base ** (-2.0 * i / dims)
        y[..., 2 * i] = x[..., 2 * i] * np.cos(a) - x[..., 2 * i + 1] * np.sin(a)
        y[..., 2 * i + 1] = x[..., 2 * i + 1] * np.cos(a) + x[..., 2 * i] * np.sin(a)
    return y


def query_temperature(positions, spec):
    """Factor of the query at each position; 1 without a spec."""
    if not spec:
        return np.ones(len(positions), F)
    return np.array([1.0 + spec["coef"] * math.log(math.floor((p + 1) / spec["every"]) + 1) for p in positions], F)


def sink_softmax(scores, sink):
    """Causal scores [n, n] -> weights; exp(sink) joins the denominator of every row only."""
    n = len(scores)
    s = np.where(np.arange(n)[None, :] <= np.arange(n)[:, None], scores, -np.inf)
    m = np.maximum(s.max(axis=1, keepdims=True), sink)
    e = np.exp(s - m)
    return e / (e.sum(axis=1, keepdims=True) + np.exp(sink - m))


def softmax_attention(q, k, v, scale, sink):
    """q [n, H, d], k [n, G, d], v [n, G, dv] -> [n, H, dv]."""
    per = q.shape[1] // k.shape[1]
    out = np.zeros((q.shape[0], q.shape[1], v.shape[2]), F)
    for h in range(q.shape[1]):
        out[:, h] = sink_softmax(q[:, h] @ k[:, h // per].T * scale, sink[h]) @ v[:, h // per]
    return out


def mix_values(v, v_first, lam):
    return (1.0 - lam) * v + lam * v_first


def attention_mixer(h, p, w, mx, eps, first):
    """`first`: one-entry list shared by the layers of a pass, holding the first mixing layer's values (or None)."""
    n = len(h)
    H, G, d, dv = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q = rms_norm((h @ w[p + "q"].T).reshape(n, H, d), w[p + "q.norm"], eps)
    k = rms_norm((h @ w[p + "k"].T).reshape(n, G, d), w[p + "k.norm"], eps)
    v = (h @ w[p + "v"].T).reshape(n, G, dv)
    q = q * query_temperature(range(n), mx.get("q_temp"))[:, None, None]
    if mx.get("v_mix"):
        if first[0] is None:
            first[0] = v
        else:
            v = mix_values(v, first[0], float(w[p + "vmix"]))
    return softmax_attention(q, k, v, mx["scale"], w[p + "sink"]).reshape(n, H * dv) @ w[p + "o"].T


def latent_mixer(h, p, w, mx, eps):
    n = len(h)
    H, d, r, dv, rank = mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"], mx["kv_rank"]
    base, dims = mx["rot"]["base"], mx["rot"]["dims"]
    q = (h @ w[p + "q"].T).reshape(n, H, d + r)
    down = h @ w[p + "dkv"].T
    c = rms_norm(down[:, :rank], w[p + "dkv.norm"], eps)
    kr = rotate_pairs(down[:, None, rank:], range(n), base, dims)
    qr = rotate_pairs(q[..., d:], range(n), base, dims)
    k = (c @ w[p + "uk"].T).reshape(n, H, d)
    v = (c @ w[p + "uv"].T).reshape(n, H, dv)
    q = np.concatenate([q[..., :d], qr], axis=2)
    k = np.concatenate([k, np.repeat(kr, H, axis=1)], axis=2)
    return softmax_attention(q, k, v, mx["scale"], w[p + "sink"]).reshape(n, H * dv) @ w[p + "o"].T


def dense_ff(h, p, w):
    return np.square(np.maximum(h @ w[p + "up"].T, 0.0)) @ w[p + "down"].T


def read_streams(xs, w_in):
    return sum(w_in[s] * x for s, x in enumerate(xs))


def write_streams(xs, y, w_out, w_mix):
    return [sum(w_mix[s, t] * x for s, x in enumerate(xs)) + w_out[t] * y for t in range(len(xs))]


def layer(xs, i, w, cfg, first):
    spec, p, eps = cfg["layers"][i], f"l{i}.", cfg["norm"]["eps"]
    h = rms_norm(read_streams(xs, w[p + "hc1.in"]), w[p + "norm1"], eps)
    if spec["type"] == "latent_attention":
        y = latent_mixer(h, p + "mix.", w, spec["mixer"], eps)
    else:
        y = attention_mixer(h, p + "mix.", w, spec["mixer"], eps, first)
    xs = write_streams(xs, y, w[p + "hc1.out"], w[p + "hc1.mix"])
    if spec.get("mlp"):
        h = rms_norm(read_streams(xs, w[p + "hc2.in"]), w[p + "norm2"], eps)
        xs = write_streams(xs, dense_ff(h, p + "mlp.", w), w[p + "hc2.out"], w[p + "hc2.mix"])
    return xs


def forward(cfg, weights, tokens, collect=None):
    """Logits [n, vocab] of a whole sequence; `collect` (a list) receives the sum of the streams after every layer."""
    w = {k: np.asarray(v, F) for k, v in weights.items()}
    xs = [w["embed"][np.asarray(tokens, int)]] * cfg["streams"]
    first = [None]
    for i in range(len(cfg["layers"])):
        xs = layer(xs, i, w, cfg, first)
        if collect is not None:
            collect.append(sum(xs))
    return rms_norm(sum(xs), w["final.norm"], cfg["norm"]["eps"]) @ w["embed"].T
