"""Fidinex models on the GPU through the framework's own loader and Model calls, against the plain
implementation (fidinex_ref.py): in f32 to rounding, in bf16 to what bf16 operands cost."""
import json
import subprocess

import numpy as np
import pytest

import fidinex_util as U
from nafevik_ref import bf16_round
from cera_amd import _build, hip_api, llama_api

pytestmark = pytest.mark.gpu

TOL = {True: 1e-5, False: 4e-2}   # f32, bf16
DTYPES = pytest.mark.parametrize("f32", [True, False], ids=["f32", "bf16"])


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    """name -> (config, weights, directory); weights and directories are made once."""
    made = {}

    def get(name):
        if name not in made:
            cfg = U.CONFIGS[name]
            w = U.random_model(cfg, seed=len(made) + 3)
            made[name] = (cfg, w, U.save(tmp_path_factory.mktemp(name), cfg, w))
        return made[name]

    return get


def _open(d, f32, ctx=512):
    return llama_api.HipLlama(str(d), ctx, f32=f32)


def _feed(m, toks, cuts):
    """Logits of every position, the prompt handed over in pieces of the given sizes (cycled)."""
    out, at, i = [], 0, 0
    while at < len(toks):
        n = min(cuts[i % len(cuts)], len(toks) - at)
        out.append(m.forward(int(toks[at]), at)[None] if n == 1 else m.forward_prefill_logits_all(toks[at:at + n], at))
        at, i = at + n, i + 1
    return np.concatenate(out)


@DTYPES
@pytest.mark.parametrize("name", list(U.CONFIGS))
def test_whole_prompts(models, name, f32):
    cfg, w, d = models(name)
    m = _open(d, f32)
    for n in (1, 2, 17, 33, 70, 150):
        toks = U.tokens(cfg, n, n)
        want = U.reference(cfg, w, toks)
        err = U.rel(_feed(m, toks, [n]), want)
        print(f"{name} f32={f32} n={n}: {err:.2e}", flush=True)
        assert err < TOL[f32]
        assert U.rel(m.forward_prefill(toks, 0)[None], want[-1:]) < TOL[f32]
    m.close()


@DTYPES
@pytest.mark.parametrize("name", list(U.CONFIGS))
def test_token_by_token_decoding_and_portions(models, name, f32):
    cfg, w, d = models(name)
    m = _open(d, f32)
    toks = U.tokens(cfg, 110, 5)
    want = U.reference(cfg, w, toks)
    for cuts in ([1], [2], [3, 2], [5, 1, 17, 2], [64, 1], [50, 60], [1, 109], [37, 1, 1, 1, 2]):
        err = U.rel(_feed(m, toks, cuts), want)
        print(f"{name} f32={f32} cuts={cuts}: {err:.2e}", flush=True)
        assert err < TOL[f32], cuts
    m.close()


# ---- one mechanism at a time: the others switched off through the weights ---------------------------
def _single(mech):
    """One or two layers with everything but the mechanism as plain as the weights can make it."""
    S = 3 if mech == "streams" else 1
    lat = [U.latent(3, 24, 10, 20, 52, 100.0, ff=56 if mech == "ff" else None)]
    att = [U.attention(4, 2, 28, 20, (0.7, 9) if mech == "temperature" else None, False)]
    if mech in ("latent", "rotation", "latent_sink", "ff"):
        layers = lat
    elif mech == "v_mix":
        layers = [U.attention(4, 2, 28, 20), U.attention(6, 2, 16, 20, None, True), U.attention(4, 2, 28, 20, None, False), U.attention(2, 2, 12, 20, None, True)]
    else:
        layers = att
    cfg = U.config(layers, width=72, vocab=45, streams=S)
    w = U.random_model(cfg, 17)
    if mech != "streams":
        for i in range(len(layers)):
            for q in ("hc1.", "hc2."):
                for n in ("in", "out", "mix"):
                    if f"l{i}.{q}{n}" in w:
                        w[f"l{i}.{q}{n}"][...] = 1.0
    if "sink" in mech:
        w["l0.mix.sink"][:] = np.linspace(-3, 6, len(w["l0.mix.sink"])).astype(np.float32)
        w["l0.mix.sink"] = bf16_round(w["l0.mix.sink"])
    else:
        for i in range(len(layers)):
            w[f"l{i}.mix.sink"][:] = -60.0
    if mech == "rotation":   # the same content everywhere: only the rotation tells keys apart, and values by a late position
        w["l0.mix.q"] *= 4
        w["embed"][2:] = w["embed"][1:2]
    if mech == "ff":
        w["l0.mix.o"][:] = 0
    if mech != "qk_norm" and "l0.mix.q.norm" in w:
        w["l0.mix.q.norm"][:] = w["l0.mix.k.norm"][:] = 1.0
    if mech == "qk_norm":
        w["l0.mix.q"] *= 16      # a norm that is left out shows
        w["l0.mix.k"] *= 0.125
    return cfg, w


@DTYPES
@pytest.mark.parametrize("mech", ["latent", "rotation", "latent_sink", "ff", "attention", "attention_sink", "temperature", "qk_norm", "v_mix", "streams"])
def test_each_mechanism_alone(tmp_path, mech, f32):
    cfg, w = _single(mech)
    m = _open(U.save(tmp_path / "m", cfg, w), f32)
    toks = U.tokens(cfg, 64, 2)
    want = U.reference(cfg, w, toks)
    for cuts in ([64], [1], [7, 2], [20, 44]):
        err = U.rel(_feed(m, toks, cuts), want)
        assert err < TOL[f32], (cuts, err)
    m.close()


# ---- keys that stand out: a marked query token meets one marked key token ----------------------------
def _marked(kind):
    """Token 1 is a key that only token 2 (the query) scores highly; every other score lies far below the sink.
    The key's value is large, so seeing it or not shows."""
    rng = np.random.default_rng(6)
    d, dv = 40, 32
    layer = U.latent(2, d, 8, dv, 48, 1000.0, 1.0) if kind == "latent" else U.attention(2, 1, d, dv, (0.2, 16), False, 1.0)
    cfg = U.config([layer], width=64, vocab=29, streams=2)
    w = U.random_model(cfg, 23)
    w["embed"][:, 58:] = 0
    w["embed"][1, 60] = w["embed"][2, 61] = 8.0
    w["l0.norm1"][:] = 1.0
    w["l0.mix.sink"][:] = 4.0
    w["l0.hc1.in"][:], w["l0.hc1.out"][:] = 0.5, 1.0
    w["l0.hc1.mix"][:] = np.eye(2)
    if kind == "latent":
        w["l0.mix.dkv"][:], w["l0.mix.uk"][:], w["l0.mix.uv"][:], w["l0.mix.q"][:] = 0, 0, 0, 0
        w["l0.mix.dkv.norm"][:] = 1.0
        w["l0.mix.dkv"][:40, :40] = np.eye(40)         # ordinary tokens have latents of their own, with no key
        w["l0.mix.dkv"][44, 60] = 16.0                 # the marked token's latent is one loud entry
        w["l0.mix.uk"][[36, d + 36], 44] = 1.0         # which both heads turn into a key
        w["l0.mix.q"][[36, d + 8 + 36], 61] = 1.0
        w["l0.mix.uv"][:, 44] = bf16_round(rng.standard_normal(2 * dv).astype(np.float32))
    else:
        w["l0.mix.q"][:], w["l0.mix.k"][:] = 0, 0
        w["l0.mix.q.norm"][:] = w["l0.mix.k.norm"][:] = 0.5
        w["l0.mix.q"][[36, d + 36], 61] = 3.0
        w["l0.mix.k"][36, 60] = 3.0
        w["l0.mix.k"][0, :40] = 1.0                    # ordinary keys point elsewhere
        w["l0.mix.v"][:, 60] = 2.0
    return cfg, w


# (key position, query position): 32-key blocks, cache steps of 64, shares of several workgroups, the first tokens, far apart
PAIRS = [(0, 1), (1, 2), (0, 31), (0, 32), (31, 32), (32, 33), (63, 64), (64, 65), (31, 64), (0, 127), (127, 128), (95, 128), (128, 255), (0, 255),
         (0, 256), (255, 256), (100, 383), (1, 420), (419, 420)]


@DTYPES
@pytest.mark.parametrize("kind", ["latent", "attention"])
def test_one_key_among_many(tmp_path, kind, f32):
    cfg, w = _marked(kind)
    m = _open(U.save(tmp_path / "m", cfg, w), f32)
    rng = np.random.default_rng(4)
    for key, query in PAIRS:
        toks = rng.integers(3, cfg["vocab"], query + 3)
        toks[key], toks[query] = 1, 2
        plain = toks.copy()
        plain[key] = 3
        want, without = U.reference(cfg, w, toks), U.reference(cfg, w, plain)
        assert U.rel(without[query:query + 1], want[query:query + 1]) > 0.1, (key, query)   # the plain implementation shows the key
        for cuts in ([len(toks)], [query, 1], [query - 1, 2] if query > 1 else [1], [key + 1, query - key, 1], [13, 2]):
            err = U.rel(_feed(m, toks, cuts)[query:], want[query:])
            assert err < TOL[f32], (key, query, cuts, err)
    m.close()


@DTYPES
@pytest.mark.parametrize("kind", ["latent", "attention"])
def test_long_decoding(tmp_path, kind, f32):
    """The marked key repeats now and then while 300 tokens are decoded one at a time."""
    cfg, w = _marked(kind)
    m = _open(U.save(tmp_path / "m", cfg, w), f32)
    rng = np.random.default_rng(9)
    toks = rng.integers(3, cfg["vocab"], 310)
    toks[rng.integers(0, 310, 12)] = 1
    toks[rng.integers(0, 310, 60)] = 2
    assert U.rel(_feed(m, toks, [10] + [1] * 300), U.reference(cfg, w, toks)) < TOL[f32]
    m.close()


@DTYPES
def test_very_large_and_very_small_scores(tmp_path, f32):
    """Scores far beyond exp's range on both sides of the sink: the running maximum moves, or never does."""
    for scale, sink in ((40.0, 2.0), (40.0, -80.0), (0.5, 90.0)):
        cfg = U.config([U.attention(2, 1, 16, 16, None, False, scale)], width=48, vocab=20, streams=1)
        w = U.random_model(cfg, 11)
        w["l0.mix.sink"][:] = sink
        if not f32:
            w["l0.mix.q"][:], w["l0.mix.k"][:] = np.sign(w["l0.mix.q"]) * 0.125, 0        # queries and keys that bf16 holds exactly:
            w["l0.mix.k"][:, :16] = 0.25 * np.eye(16)                                      # one entry each, one above the others
            w["l0.mix.q"][:, 1:] = 0
            w["l0.mix.q.norm"][:] = w["l0.mix.k.norm"][:] = 1.0
            w["embed"][:, :16] = np.eye(20, 16)
        m = _open(U.save(tmp_path / f"m{scale}{sink}", cfg, w), f32)
        toks = U.tokens(cfg, 90, 2)
        want = U.reference(cfg, w, toks)
        tol = 2e-4 if f32 else TOL[f32]     # scores in the hundreds: their f32 rounding is exp's relative error
        for cuts in ([90], [1], [33, 2, 1]):
            err = U.rel(_feed(m, toks, cuts), want)
            assert err < tol, (scale, sink, cuts, err)
        m.close()


# ---- the cache and the state over several sequences --------------------------------------------------
@DTYPES
@pytest.mark.parametrize("name", ["mixed", "wide_group", "deep_latent"])
def test_a_new_sequence_sees_nothing_of_the_last(models, name, f32):
    cfg, w, d = models(name)
    long, short = U.tokens(cfg, 200, 1), U.tokens(cfg, 40, 2)
    fresh, used = _open(d, f32), _open(d, f32)
    _feed(used, long, [90, 1, 1, 2])
    for cuts in ([40], [1], [3, 2]):
        assert np.array_equal(_feed(fresh, short, cuts), _feed(used, short, cuts))
        _feed(used, long, [77, 1])
    fresh.close(), used.close()


@DTYPES
def test_cutting_back_and_going_on(models, f32):
    cfg, w, d = models("mixed")
    m = _open(d, f32)
    toks, other = U.tokens(cfg, 120, 3), U.tokens(cfg, 120, 4)
    _feed(m, toks, [100, 1])
    for keep in (119, 100, 64, 33, 5, 1):
        m.truncate_kv(keep)
        both = np.concatenate([toks[:keep], other[keep:]])
        want = U.reference(cfg, w, both)[keep:keep + 2]
        got = m.forward_prefill_logits_all(both[keep:keep + 2], keep) if keep + 2 <= 120 else m.forward(int(both[keep]), keep)[None]
        assert U.rel(got, want[:len(got)]) < TOL[f32], keep
        m.truncate_kv(keep)
    m.close()


@DTYPES
@pytest.mark.parametrize("name", ["mixed", "deep_latent"])
def test_snapshots(models, name, f32):
    cfg, w, d = models(name)
    m, n = _open(d, f32), _open(d, f32)
    a, b = U.tokens(cfg, 90, 5), U.tokens(cfg, 90, 6)
    _feed(m, a[:57], [57])
    snap = m.snapshot_state()
    assert snap.seq_len == 57
    _feed(m, b, [31, 1, 2])
    for target in (m, n):
        target.restore_state(snap)
        got = np.concatenate([target.forward(int(a[57]), 57)[None], target.forward_prefill_logits_all(a[58:], 58)])
        assert U.rel(got, U.reference(cfg, w, a)[57:]) < TOL[f32]
    snap.close(), m.close(), n.close()


def test_the_cache_holds_latents_and_one_key_part_only(hip, models):
    cfg, w, _ = models("deep_latent")
    def size(positions):
        m = hip_api.LayeredModel(hip, cfg, U.as_arrays(w), positions)
        n = hip.lib.cera_hip_memory_bytes(m.h)
        m.close()
        return n
    # rows of 256 + 32 and 192 + 32 elements, padded to 64, and the two layers' rotation tables
    assert size(2048) - size(1024) == 1024 * (2 * (320 + 256) + 4 * (8 + 20))


def test_greedy_generation(models, tmp_path):
    cfg, w, d = models("mixed")
    prompt, new = U.tokens(cfg, 50, 8), 40
    toks, margins = list(prompt), []
    for _ in range(new):
        l = U.reference(cfg, w, toks)[-1]
        top = np.sort(l)[-2:]
        margins.append((top[1] - top[0]) / np.sqrt(np.mean(l ** 2)))
        toks.append(int(np.argmax(l)))
    assert min(margins) > 1e-4, "pick another seed: a near tie decides nothing"
    m = _open(d, True)
    for ubatch in (512, 7, 2):
        out, _, _ = m.generate_greedy(prompt, new, ubatch)
        assert out.tolist() == toks[50:]
    m.close()
    # the command line takes the same directory
    r = subprocess.run([str(_build.CLI_BIN), "run", "--model", str(d), "--dtype", "f32", "--prompt-len", "30", "--n-predict", "8", "--ctx", "64",
                        "--tokens-out", str(tmp_path / "t")], capture_output=True, text=True, timeout=60)
    assert r.returncode == 0, r.stderr
    assert json.loads(r.stdout)["arch"] == "Fidinex"
    p, o = ([int(t) for t in line.split()] for line in (tmp_path / "t").read_text().splitlines())
    for t in o:
        assert t == int(np.argmax(U.reference(cfg, w, p)[-1]))
        p.append(t)


@DTYPES
def test_long_prompts_take_the_large_tiles(tmp_path, f32):
    """Enough rows and columns for the 128 x 128 GEMM tiles, two column tiles per wavefront, and a second pass."""
    n = 2200 if not f32 else 1100
    cfg = U.config([U.attention(16, 2, 64, 64, (0.1, 200), True, ff=2048), U.latent(8, 128, 64, 128, 192, 10000.0, ff=96),
                    U.attention(16, 2, 128, 128, None, False), U.latent(16, 24, 8, 32, 256, 500.0)], width=128, vocab=64, streams=4)
    w = U.random_model(cfg, 41)
    m = _open(U.save(tmp_path / "m", cfg, w), f32, 2304)
    toks = U.tokens(cfg, n, 3)
    want = U.reference(cfg, w, toks)
    for cuts in ([n], [n - 3, 1, 2], [n // 2]):
        err = U.rel(_feed(m, toks, cuts), want)
        print(f"f32={f32} cuts={cuts}: {err:.2e}", flush=True)
        assert err < TOL[f32]
    m.close()


@DTYPES
def test_steps_behind_a_very_long_context(tmp_path, f32):
    """Thousands of visible keys: decode steps and short portions split them over many workgroups."""
    cfg = U.config([U.attention(4, 2, 64, 64, (0.1, 1000), True, ff=48), U.latent(2, 24, 8, 36, 68, 900.0), U.attention(2, 1, 24, 64, None, False),
                    U.latent(4, 24, 64, 36, 512, 5000.0)], width=48, vocab=30, streams=2)
    w = U.random_model(cfg, 43)
    m = _open(U.save(tmp_path / "m", cfg, w), f32, 4400)
    toks = U.tokens(cfg, 4330, 3)
    want = U.reference(cfg, w, toks)[4300:]
    m.forward_prefill(toks[:4300], 0)
    got = np.concatenate([m.forward(int(toks[4300]), 4300)[None], m.forward_prefill_logits_all(toks[4301:4303], 4301),
                          m.forward_prefill_logits_all(toks[4303:4312], 4303)] + [m.forward(int(t), 4312 + i)[None] for i, t in enumerate(toks[4312:])])
    assert U.rel(got, want) < TOL[f32]
    m.close()


def test_inputs_too_wide_for_the_gemv_take_the_gemm(hip):
    """A feed-forward wider than a workgroup's LDS: the decode step runs as a pass of one token."""
    cfg = U.config([U.attention(2, 1, 32, 32, (0.5, 3), True, ff=16400), U.latent(2, 16, 8, 16, 40)], width=64, vocab=24, streams=2)
    w = U.random_model(cfg, 5)
    m = hip_api.LayeredModel(hip, cfg, U.as_arrays(w), 64, f32=True)
    toks = U.tokens(cfg, 40, 1)
    want = U.reference(cfg, w, toks)
    got = np.concatenate([m.forward_prefill_logits_all(toks[:20], 0)] + [m.forward(int(t), 20 + i)[None] for i, t in enumerate(toks[20:])])
    assert U.rel(got, want) < TOL[True]
    m.close()


def test_what_does_not_fit_is_refused(hip, models):
    cfg, w, _ = models("plain")
    m = hip_api.LayeredModel(hip, cfg, U.as_arrays(w), 32)
    for call in (lambda: m.set_reference_order(True), lambda: hip.check(hip.lib.cera_hip_shift_kv(m.h, 0, 1)),
                 lambda: hip.check(hip.lib.cera_hip_configure_kv(m.h, 1)), m.drop_decode_copies):
        with pytest.raises(hip_api.HipError, match="not available for this model family"):
            call()
    with pytest.raises(hip_api.HipError, match="does not fit"):
        m.forward_prefill(U.tokens(cfg, 33, 1), 0)
    with pytest.raises(hip_api.HipError):
        m.forward(cfg["vocab"], 0)
    m.close()

    def refused(cfg, match):
        with pytest.raises(hip_api.HipError, match=match):
            hip_api.LayeredModel(hip, cfg, U.as_arrays(U.random_model(cfg, 1)), 32)

    refused(U.config([U.attention(2, 1, 600, 64)], width=16), "key and value entries")
    refused(U.config([U.latent(1, 8, 4, 8, 540)], width=16), "kernels' limits")
    refused(U.config([U.attention(2, 1, 8, 8)], width=16, streams=9), "streams")
    refused(U.config([U.attention(2, 1, 8, 8, None, True), U.attention(2, 2, 8, 8, None, True)], width=16), "another shape")


@DTYPES
def test_trace_runner_interleaves_requests(models, tmp_path, f32):
    cfg, w, d = models("mixed")
    a, b = U.tokens(cfg, 70, 11), U.tokens(cfg, 45, 12)
    ra, rb = U.reference(cfg, w, a), U.reference(cfg, w, b)
    entry = lambda i, t, want: {"id": i, "tokens": [int(x) for x in t], "want": want}  # noqa: E731
    steps = [
        ([entry("a", a[:40], [0, 5, 39])], []),
        ([entry("b", b[:2], [1]), entry("a", a[40:41], [0])], []),
        ([entry("b", b[2:44], [])], []),
        ([entry("a", a[41:], [28]), entry("b", b[44:], [0])], ["a", "b"]),
        ([entry("a", b[:7], [3, 4])], ["a"]),            # the name is free again
    ]
    text = "".join(json.dumps({"step": i, "entries": e, "end": end}) + "\n" for i, (e, end) in enumerate(steps))
    for extra in (["--max-tokens", "120"], []):
        r = subprocess.run([str(_build.TRACE_BIN), "--model", str(d), "--out", str(tmp_path), "--dtype", "float32" if f32 else "bfloat16", *extra],
                           input=text, capture_output=True, text=True, timeout=60)
        assert r.returncode == 0, r.stderr
        assert r.stdout.split("\n")[:5] == [f"done {i}" for i in range(5)]
        got = lambda i: np.fromfile(tmp_path / f"{i}.f32", "<f4").reshape(-1, cfg["vocab"])  # noqa: E731
        want = [ra[[0, 5, 39]], np.stack([rb[1], ra[40]]), None, np.stack([ra[69], rb[44]]), rb[[3, 4]]]
        for i, x in enumerate(want):
            if x is None:
                assert not (tmp_path / f"{i}.f32").exists()
            else:
                assert U.rel(got(i), x) < TOL[f32], i
