"""Nafevik models on the GPU through the framework's own loader and Model calls, against the plain
implementation (nafevik_ref.py): in f32 to rounding, in bf16 to what bf16 operands cost."""
import json
import subprocess

import numpy as np
import pytest

import nafevik_ref as R
import nafevik_util as U
from cera_amd import _build, hip_api, llama_api

pytestmark = pytest.mark.gpu

TOL = {True: 1e-5, False: 3e-2}   # f32, bf16
DTYPES = pytest.mark.parametrize("f32", [True, False], ids=["f32", "bf16"])


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    """name -> (config, weights, directory); weights and directories are made once."""
    made = {}

    def get(name):
        if name not in made:
            cfg = U.CONFIGS[name]
            w = R.random_model(cfg, seed=len(made) + 3)
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
    cfg = U.config([U.attention(4, 2, 32, 24, 21, 16, 200.0, U.YARN, ff=56)], width=72, vocab=45, taps=3,
                   loop=(0, 1, 2) if mech == "loop" else None, mult=0.8)
    w = R.random_model(cfg, 17)
    off = lambda name: w[name].fill(0)  # noqa: E731
    if mech != "positions":
        off("pos")
    if mech != "conv":
        off("l0.canon1"), off("l0.canon2")
    if mech in ("ff", "positions"):
        off("l0.mix.o")
    if mech in ("attention", "rotation", "gate", "bias", "conv"):
        off("l0.mlp.down")
    if mech != "gate":
        off("l0.mix.g")
    if mech != "bias":
        off("l0.mix.pb")
    if mech == "loop":
        off("l0.mix.o"), off("l0.mlp.down")
    if mech == "rotation":   # the same content everywhere: only the rotation tells keys apart
        w["embed"][:] = w["embed"][:1]
        w["l0.mix.q"] *= 4
    if mech == "gate":
        w["l0.mix.g"] *= 4
    if mech == "bias":
        w["l0.mix.pb"] = R.bf16_round(np.array([-3.0, 2.0, 0.5, -0.5], np.float32))
    return cfg, w


@DTYPES
@pytest.mark.parametrize("mech", ["ff", "positions", "attention", "rotation", "gate", "bias", "conv", "loop"])
def test_each_mechanism_alone(tmp_path, mech, f32):
    cfg, w = _single(mech)
    m = _open(U.save(tmp_path / "m", cfg, w), f32)
    toks = U.tokens(cfg, 64, 2)
    want = U.reference(cfg, w, toks)
    for cuts in ([64], [1], [7, 2]):
        assert U.rel(_feed(m, toks, cuts), want) < TOL[f32], cuts
    m.close()


# ---- keys that stand out: a marked query token meets one marked key token ----------------------------
CHUNK = 48


def _marked():
    """Token 1 is a key that only token 2 (the query) scores highly, on a dimension that is not rotated;
    every other weight is sigmoid(-9).  The key's value is large, so seeing it or not shows."""
    cfg = U.config([U.attention(2, 1, 40, 32, CHUNK, 32, 1000.0, U.YARN, scale=1.0)], width=64, vocab=29, taps=1, positions=512)
    w = R.random_model(cfg, 23)
    w["pos"][:] = 0
    w["l0.canon1"][:] = 0
    w["embed"][:, 60:] = 0
    w["embed"][1, 60] = w["embed"][2, 61] = 8.0
    w["l0.mix.q"][:], w["l0.mix.k"][:] = 0, 0
    w["l0.mix.q"][[36, 76], 61] = 3.0     # both heads, dimension 36
    w["l0.mix.k"][36, 60] = 3.0
    w["l0.mix.v"][:, 60] = 2.0
    w["l0.mix.pb"][:] = -9.0
    return cfg, w


# (key position, query position): chunk edges, 32-key blocks, cache borders, far apart, the sequence's first tokens
PAIRS = [(0, 47), (0, 48), (47, 48), (48, 95), (47, 95), (48, 48 + 47), (0, 1), (1, 2), (31, 32), (32, 33), (63, 64), (96, 143), (95, 143),
         (95, 96), (143, 144), (144, 191), (191, 192), (192, 239), (127, 128), (128, 143), (144, 145)]


@DTYPES
def test_a_key_just_inside_and_just_outside_its_chunk(tmp_path, f32):
    cfg, w = _marked()
    m = _open(U.save(tmp_path / "m", cfg, w), f32)
    rng = np.random.default_rng(4)
    for key, query in PAIRS:
        toks = rng.integers(3, cfg["vocab"], query + 3)
        toks[key], toks[query] = 1, 2
        plain = toks.copy()
        plain[key] = 3
        want, without = U.reference(cfg, w, toks), U.reference(cfg, w, plain)
        seen = key // CHUNK == query // CHUNK
        effect = U.rel(without[query:query + 1], want[query:query + 1])
        assert (effect > 0.1) == seen, (key, query, effect)      # the plain implementation shows the key, or not at all
        for cuts in ([len(toks)], [query, 1], [query - 1, 2] if query > 1 else [1], [key + 1, query - key, 1], [13, 2]):
            err = U.rel(_feed(m, toks, cuts)[query:], want[query:])
            assert err < TOL[f32], (key, query, cuts, err)
    m.close()


@DTYPES
def test_long_decoding_over_chunk_edges(tmp_path, f32):
    """The marked key repeats now and then while 300 tokens are decoded one at a time."""
    cfg, w = _marked()
    m = _open(U.save(tmp_path / "m", cfg, w), f32)
    rng = np.random.default_rng(9)
    toks = rng.integers(3, cfg["vocab"], 310)
    toks[rng.integers(0, 310, 25)] = 1
    toks[rng.integers(0, 310, 60)] = 2
    want = U.reference(cfg, w, toks)
    assert U.rel(_feed(m, toks, [10] + [1] * 300), want) < TOL[f32]
    m.close()


def test_history_of_the_input_convolutions(tmp_path):
    """A single loud token: the rows it reaches through the convolution differ, at every kind of edge."""
    cfg = U.config([U.attention(2, 2, 16, 16, 30, 16, 100.0, ff=32)] * 2, width=48, vocab=20, taps=5, loop=(0, 2, 2))
    w = R.random_model(cfg, 31)
    w["embed"][1] *= 8
    m = _open(U.save(tmp_path / "m", cfg, w), True)
    for loud in (0, 1, 29, 30, 63, 64, 65, 99):
        toks = np.random.default_rng(loud).integers(2, 20, 110)
        toks[loud] = 1
        want = U.reference(cfg, w, toks)
        for cuts in ([110], [loud + 1, 1], [loud + 1, 2], [max(loud, 1), 1, 1, 3, 1], [2]):
            assert U.rel(_feed(m, toks, cuts), want) < TOL[True], (loud, cuts)
    m.close()


# ---- the cache and the state over several sequences --------------------------------------------------
@DTYPES
@pytest.mark.parametrize("name", ["mixed", "wide_group"])
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
    for keep in (119, 100, 97, 61):
        m.truncate_kv(keep)
        mixed = np.concatenate([toks[:keep], other[keep:]])
        want = U.reference(cfg, w, mixed)
        got = np.concatenate([m.forward_prefill_logits_all(mixed[keep:keep + 2], keep)] if keep + 2 <= 120 else [m.forward(int(mixed[keep]), keep)[None]])
        assert U.rel(got, want[keep:keep + len(got)]) < TOL[f32], keep
        m.truncate_kv(keep)
        m.forward_prefill(toks[keep:keep + 1], keep)
    # the convolution rows go back 64 positions and no further
    m2 = _open(d, f32)
    _feed(m2, toks, [120])
    with pytest.raises(llama_api.BackendError, match="convolution state"):
        m2.truncate_kv(40)
    assert m2.seq_len == 120
    m2.truncate_kv(0)
    assert U.rel(_feed(m2, other, [120]), U.reference(cfg, w, other)) < TOL[f32]
    m.close(), m2.close()


@DTYPES
def test_snapshots(models, f32):
    cfg, w, d = models("mixed")
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


def test_greedy_generation(models, tmp_path):
    cfg, w, d = models("once")
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
    assert json.loads(r.stdout)["arch"] == "Nafevik"
    p, o = ([int(t) for t in line.split()] for line in (tmp_path / "t").read_text().splitlines())
    for t in o:
        assert t == int(np.argmax(U.reference(cfg, w, p)[-1]))
        p.append(t)


@DTYPES
def test_long_prompts_take_the_large_tiles(tmp_path, f32):
    """Enough rows and columns for the 128 x 128 GEMM tiles, the two-tile attention columns and a second pass."""
    n = 2200 if not f32 else 1100
    cfg = U.config([U.attention(16, 2, 64, 64, 700, 64, 10000.0, U.YARN, ff=2048), U.attention(16, 2, 128, 128, 1500, 128, 10000.0, ff=96)],
                   width=128, vocab=64, taps=3, positions=2304)
    w = R.random_model(cfg, 41)
    m = _open(U.save(tmp_path / "m", cfg, w), f32, 2304)
    toks = U.tokens(cfg, n, 3)
    want = U.reference(cfg, w, toks)
    for cuts in ([n], [n - 3, 1, 2]):
        err = U.rel(_feed(m, toks, cuts), want)
        print(f"f32={f32} cuts={cuts}: {err:.2e}", flush=True)
        assert err < TOL[f32]
    m.close()


@DTYPES
def test_steps_behind_a_very_long_context(tmp_path, f32):
    """Thousands of visible keys: decode steps and short portions split them over many workgroups."""
    cfg = U.config([U.attention(4, 2, 64, 64, None, 64, 10000.0, U.YARN, ff=48), U.attention(2, 1, 24, 36, 4320, 16, 900.0)],
                   width=48, vocab=30, taps=3, positions=4400)
    w = R.random_model(cfg, 43)
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
    cfg = U.config([U.attention(2, 1, 32, 32, 16, 32, 100.0, ff=16400)], width=64, vocab=24, taps=3)
    w = R.random_model(cfg, 5)
    raw = {k: (v if k.endswith(R_VECTORS) else U.bf16_bits(v)) for k, v in w.items()}
    m = hip_api.LayeredModel(hip, cfg, raw, 64, f32=True)
    toks = U.tokens(cfg, 40, 1)
    want = U.reference(cfg, w, toks)
    got = np.concatenate([m.forward_prefill_logits_all(toks[:20], 0)] + [m.forward(int(t), 20 + i)[None] for i, t in enumerate(toks[20:])])
    assert U.rel(got, want) < TOL[True]
    m.close()


R_VECTORS = ("norm1", "canon1", "canon2", ".pb", "loop.step", "final.norm")


def test_calls_only_a_llama_has_are_refused(hip, models):
    cfg, w, _ = models("plain")
    raw = {k: (v if k.endswith(R_VECTORS) else U.bf16_bits(v)) for k, v in w.items()}
    m = hip_api.LayeredModel(hip, cfg, raw, 32)
    for call in (lambda: m.set_reference_order(True), lambda: hip.check(hip.lib.cera_hip_shift_kv(m.h, 0, 1)),
                 lambda: hip.check(hip.lib.cera_hip_configure_kv(m.h, 1)), m.drop_decode_copies):
        with pytest.raises(hip_api.HipError, match="not available for this model family"):
            call()
    with pytest.raises(hip_api.HipError, match="does not fit"):
        m.forward_prefill(U.tokens(cfg, 33, 1), 0)
    with pytest.raises(hip_api.HipError):
        m.forward(cfg["vocab"], 0)
    m.close()


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
    r = subprocess.run([str(_build.TRACE_BIN), "--model", str(d), "--out", str(tmp_path), "--dtype", "float32" if f32 else "bfloat16",
                        "--max-tokens", "120"], input=text, capture_output=True, text=True, timeout=60)
    assert r.returncode == 0, r.stderr
    assert r.stdout.split("\n")[:5] == [f"done {i}" for i in range(5)]
    got = lambda i: np.fromfile(tmp_path / f"{i}.f32", "<f4").reshape(-1, cfg["vocab"])  # noqa: E731
    want = [ra[[0, 5, 39]], np.stack([rb[1], ra[40]]), None, np.stack([ra[69], rb[44]]), rb[[3, 4]]]
    for i, x in enumerate(want):
        if x is None:
            assert not (tmp_path / f"{i}.f32").exists()
        else:
            assert U.rel(got(i), x) < TOL[f32], i
