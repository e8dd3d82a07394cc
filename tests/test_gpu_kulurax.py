"""Kulurax models through the framework's own entry points (evaluation, portions, greedy generation, trace
replay) against the plain numpy restatement in np_kulurax.py: small models with seeded weights."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import kulurax_util as ku
import np_kulurax as ref

pytestmark = pytest.mark.gpu

LIMIT = {"float32": 3e-5, "bfloat16": 4e-2}
DTYPES = ("float32", "bfloat16")


def pair(hip, cfg, seed, dtype, context_length=600, decay_rank=7, **kw):
    w = ku.random_weights(cfg, seed, decay_rank=decay_rank, **kw)
    return hip.create_model(cfg, w, dtype=dtype, context_length=context_length), ref.NumpyKulurax(cfg, ku.as_floats(w))


def feed(model, toks, cuts):
    """Logits of every position, the tokens fed in portions of the given sizes (the last one repeats)."""
    out, at, i = [], 0, 0
    while at < len(toks):
        n = min(cuts[min(i, len(cuts) - 1)], len(toks) - at)
        out.append(model.eval(toks[at:at + n]))
        at += n
        i += 1
    return np.concatenate(out)


MIXED = ku.config([ku.linear_attention(mlp=ku.mlp()), ku.attention(), ku.linear_attention(heads=3, dim=33, vdim=20, tau=1.0),
                   ku.attention(heads=5, dim=16, vdim=16, window=30, mlp=ku.mlp(50, 2.0))])

SINGLE = {
    "attention": ku.config([ku.attention()]),
    "attention_mlp": ku.config([ku.attention(mlp=ku.mlp())]),
    "gla": ku.config([ku.linear_attention()]),
    "gla_mlp": ku.config([ku.linear_attention(mlp=ku.mlp(ff=33))]),
    # sizes that are not multiples of anything, one of everything
    "attention_odd": ku.config([ku.attention(heads=3, dim=13, vdim=21, kv_rank=37, q_rank=29, window=6, scale=1.0)], vocab=67,
                               width=50),
    "attention_ones": ku.config([ku.attention(heads=1, dim=1, vdim=1, kv_rank=1, q_rank=1, window=1)], vocab=5, width=6),
    "gla_odd": ku.config([ku.linear_attention(heads=5, dim=7, vdim=11, tau=3.0)], vocab=67, width=50),
    "gla_ones": ku.config([ku.linear_attention(heads=1, dim=1, vdim=1, tau=1.0)], vocab=5, width=6),
    "odd_width": ku.config([ku.attention(), ku.linear_attention()], width=53),
    # head sizes of every tile form
    "attention_wide": ku.config([ku.attention(heads=2, dim=136, vdim=200, kv_rank=300, q_rank=520, window=70, scale=0.1)]),
    "attention_mid": ku.config([ku.attention(heads=2, dim=96, vdim=72, kv_rank=64, q_rank=64, window=64, scale=0.1)]),
    "attention_unequal": ku.config([ku.attention(heads=2, dim=32, vdim=256, kv_rank=128, q_rank=128, window=33)]),
    "attention_beyond_tiles": ku.config([ku.attention(heads=2, dim=264, vdim=300, window=20, scale=0.1)]),
    "gla_wide": ku.config([ku.linear_attention(heads=2, dim=260, vdim=130, tau=16.0)]),
    "gla_full": ku.config([ku.linear_attention(heads=2, dim=64, vdim=256, tau=2.0)]),
    "gla_wide_values": ku.config([ku.linear_attention(heads=3, dim=130, vdim=66, tau=2.0)]),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(SINGLE))
def test_each_layer_alone(hip, name, dtype):
    """A prompt in one pass, and its tail token by token, for every mechanism and many sizes."""
    cfg = SINGLE[name]
    model, plain = pair(hip, cfg, 11, dtype, context_length=200)
    toks = ku.tokens(cfg, 150, 5)
    want = plain.forward(toks)
    got = model.eval(toks)
    assert ku.error(got, want) <= LIMIT[dtype]
    model.reset()
    got = feed(model, toks, [110, 1])
    assert ku.error(got, want) <= LIMIT[dtype]
    model.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_embedding_and_positions_alone(hip, dtype):
    """Sublayers whose output norm is zero leave the embedding, its position vector and the head; far positions
    are exact too (an angle of thousands of radians must not lose its fraction)."""
    cfg = ku.config([ku.linear_attention()], width=90)

    def silence(w):
        w["l0.norm1b"][:] = 0

    model, plain = pair(hip, cfg, 3, dtype, context_length=9000, edit=silence)
    toks = ku.tokens(cfg, 8200, 1)
    got = model.eval(toks, want=[0, 1, 2, 63, 64, 4095, 4096, 8199])
    x = plain.w["embed"][toks] + ref.sinusoid(np.arange(len(toks)), cfg["width"])
    want = ref.rms_norm(x, plain.w["final.norm"], cfg["norm"]["eps"]) @ plain.w["embed"].T
    assert ku.error(got, want[[0, 1, 2, 63, 64, 4095, 4096, 8199]]) <= LIMIT[dtype]
    model.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cuts", [[1], [2], [3], [2, 5, 3], [4], [7], [15, 16], [17], [40, 2, 64, 3, 1], [63, 64, 65, 2], [300]])
def test_portions_of_every_size(hip, cuts, dtype):
    """However a sequence is cut, every position's logits are the plain forward's."""
    model, plain = pair(hip, MIXED, 21, dtype)
    toks = ku.tokens(MIXED, 210, 2)
    assert ku.error(feed(model, toks, cuts), plain.forward(toks)) <= LIMIT[dtype]
    assert model.past == len(toks)
    model.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_long_run_laps_the_cache_ring(hip, dtype, monkeypatch):
    """Passes of 8 tokens make rings of window + 7 rows: a prompt and a long decode go around them many times,
    and prompts longer than a pass are cut by the framework itself."""
    monkeypatch.setenv("LITENN_HIP_PASS_ROWS", "8")
    model, plain = pair(hip, MIXED, 22, dtype)
    toks = ku.tokens(MIXED, 420, 3)
    want = plain.forward(toks)
    assert ku.error(feed(model, toks, [90, 1, 1, 1, 1, 1, 100, 1]), want) <= LIMIT[dtype]
    monkeypatch.setenv("LITENN_HIP_PASS_ROWS", "33")
    model.close()
    model, plain = pair(hip, MIXED, 22, dtype)
    got = model.eval(toks, want=[419, 0, 32, 33, 34, 65, 66, 200])  # any order, across passes
    assert ku.error(got, want[[419, 0, 32, 33, 34, 65, 66, 200]]) <= LIMIT[dtype]
    model.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_cache_is_the_context_when_that_is_shorter(hip, dtype):
    model, plain = pair(hip, MIXED, 23, dtype, context_length=40)
    toks = ku.tokens(MIXED, 40, 4)
    assert ku.error(feed(model, toks, [18, 1, 20, 1]), plain.forward(toks)) <= LIMIT[dtype]
    with pytest.raises(hip.LiteNNHipError, match="context length exceeded"):
        model.eval([1])
    model.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_sequence_does_not_see_the_one_before(hip, dtype):
    """After a reset a sequence's logits are bit for bit those of a fresh model, whatever ran before."""
    w = ku.random_weights(MIXED, 24)
    first, second = ku.tokens(MIXED, 130, 5), ku.tokens(MIXED, 61, 6)
    fresh = hip.create_model(MIXED, w, dtype=dtype, context_length=300)
    want = feed(fresh, second, [40, 1, 1, 5, 1])
    fresh.close()
    used = hip.create_model(MIXED, w, dtype=dtype, context_length=300)
    feed(used, first, [100, 1])
    used.generate(first[:20], 30)
    used.reset()
    assert used.past == 0
    assert np.array_equal(feed(used, second, [40, 1, 1, 5, 1]), want)
    used.close()


def sharp(window, scale):
    """A model with one attention layer whose scores spread so far that few keys carry a query; embeddings
    drown the position vectors, sinks stay below the scores."""
    cfg = ku.config([ku.attention(heads=2, dim=16, vdim=16, kv_rank=32, q_rank=32, window=window, scale=scale)], vocab=48,
                    width=64)

    def edit(w):
        w["embed"] *= 6.0
        w["l0.norm1b"] *= 12.0
        w["l0.mix.sink"][:] = -3.0
    weights = ku.random_weights(cfg, 31, edit=edit)
    return cfg, weights


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", [1, 2, 31, 32, 33, 63, 64, 65, 100])
def test_window_edges_in_models(hip, window, dtype):
    """Sharp scores make one key carry a query: a window one position off, in a prompt or in decoding, would
    move the logits by far more than the tolerance (the plain form with such a window shows by how much)."""
    cfg, w = sharp(window, 1.0)
    plain = ref.NumpyKulurax(cfg, ku.as_floats(w))
    toks = ku.tokens(cfg, 180, 9)
    want = plain.forward(toks)
    for off in (-1, 1):
        if window + off < 1:
            continue
        wrong = json.loads(json.dumps(cfg))
        wrong["layers"][0]["mixer"]["mask"]["size"] = window + off
        assert ku.error(ref.NumpyKulurax(wrong, ku.as_floats(w)).forward(toks), want) > 0.05
    limit = {"float32": 1e-4, "bfloat16": 0.15}[dtype]  # sharp scores amplify the operands' rounding
    model = hip.create_model(cfg, w, dtype=dtype, context_length=200)
    for cuts in ([180], [100, 1], [37, 2, 64, 3]):
        model.reset()
        assert ku.error(feed(model, toks, cuts), want) <= limit, cuts
    model.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_sink_gate_and_first_tokens(hip, dtype):
    """Sinks around the scores' size: leaving them out, scaling them or counting them twice changes the first
    tokens most; the device agrees with the plain form from the very first token on."""
    cfg = ku.config([ku.attention(window=12, scale=0.5)])
    w = ku.random_weights(cfg, 41)
    plain = ref.NumpyKulurax(cfg, ku.as_floats(w))
    toks = ku.tokens(cfg, 40, 8)
    want = plain.forward(toks)
    for change in (lambda s: s * 0 - 1e4, lambda s: s * 0.5, lambda s: s + np.log(2.0)):
        f = ku.as_floats(w)
        f["l0.mix.sink"] = change(f["l0.mix.sink"])
        assert ku.error(ref.NumpyKulurax(cfg, f).forward(toks), want) > 2 * LIMIT["bfloat16"]
    model = hip.create_model(cfg, w, dtype=dtype, context_length=64)
    for cuts in ([40], [1], [2], [16, 1]):
        model.reset()
        assert ku.error(feed(model, toks, cuts), want) <= LIMIT[dtype], cuts
    model.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("bias,tau", [((-30.0, -20.0), 1.0), ((-60.0, 6.0), 1.0), ((8.0, 12.0), 16.0), ((-2.0, 2.0), 0.25)])
def test_decays_from_instant_to_endless(hip, bias, tau, dtype):
    """Channels that forget within one token beside channels that keep hundreds: no factor of the chunked form
    may overflow or vanish where the recurrence does not."""
    cfg = ku.config([ku.linear_attention(heads=2, dim=40, vdim=24, tau=tau), ku.linear_attention(heads=1, dim=70, vdim=48, tau=tau)])
    model, plain = pair(hip, cfg, 51, dtype, decay_bias=bias)
    toks = ku.tokens(cfg, 330, 10)
    want = plain.forward(toks)
    assert np.all(np.isfinite(want))
    for cuts in ([330], [129, 1, 1, 64, 1, 70, 3]):
        model.reset()
        errors = ku.row_errors(feed(model, toks, cuts), want)
        if dtype == "float32":
            assert errors.max() <= LIMIT[dtype], cuts
        else:
            # a head that forgets at once is q . k times v, normalised: where q . k comes out near zero the
            # operands' rounding decides its sign, so single rows may be far off in 16 bits
            assert np.median(errors) <= LIMIT[dtype] / 2 and np.mean(errors > LIMIT[dtype]) <= 0.2, cuts
    model.close()


def test_the_state_is_carried_in_32_bits(hip):
    """A slowly decaying state over a long sequence, in the serving precisions: a state kept in 16 bits would
    lose the small additions."""
    cfg = ku.config([ku.linear_attention(heads=2, dim=16, vdim=16, tau=16.0)])
    model, plain = pair(hip, cfg, 52, "bfloat16", context_length=1200, decay_bias=(9.0, 10.0))
    toks = ku.tokens(cfg, 1100, 11)
    want = plain.forward(toks)
    assert ku.error(feed(model, toks, [700, 1]), want) <= LIMIT["bfloat16"]
    model.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_clamped_feed_forward(hip, dtype):
    """Gate and up values on both sides of the limit; a clamp of the gate from below or an unclamped up shows."""
    cfg = ku.config([ku.attention(mlp=ku.mlp(ff=70, limit=0.5))])

    def edit(w):
        for name in ("gate", "up"):
            w[f"l0.mlp.{name}"] *= 2.0
    w = ku.random_weights(cfg, 61, edit=edit)
    plain = ref.NumpyKulurax(cfg, ku.as_floats(w))
    toks = ku.tokens(cfg, 70, 12)
    want = plain.forward(toks)
    wrong = json.loads(json.dumps(cfg))
    wrong["layers"][0]["mlp"]["limit"] = 0.7
    assert ku.error(ref.NumpyKulurax(wrong, ku.as_floats(w)).forward(toks), want) > 2 * LIMIT["bfloat16"]
    model = hip.create_model(cfg, w, dtype=dtype, context_length=80)
    for cuts in ([70], [1]):
        model.reset()
        assert ku.error(feed(model, toks, cuts), want) <= LIMIT[dtype]
    model.close()


def lively(w):
    """Small embeddings under full-size sublayers: the tied head then does not answer every token with itself."""
    w["embed"] *= 0.1


def test_greedy_generation(hip):
    """generate(): the prompt in passes, then the captured step, against the plain form's greedy tokens; again
    after other work on the same model (replays of the same captured step), and continued."""
    model, plain = pair(hip, MIXED, 71, "float32", edit=lively)
    prompt = ku.tokens(MIXED, 45, 12)
    want, margins = plain.greedy(prompt, 40)
    assert min(margins) > 2e-3 and len(set(want)) > 15  # no near-tie in this sequence, no single repeated token
    for _ in range(3):
        model.reset()
        got, _, _ = model.generate(prompt, 40)
        assert got.tolist() == want
        assert model.past == 45 + 39
        model.eval(ku.tokens(MIXED, 30, 14))
        model.eval([1], want=[0])
    model.reset()
    head, _, _ = model.generate(prompt, 15)
    tail, _, _ = model.generate(head[-1:], 25)
    assert head.tolist() + tail.tolist() == want
    model.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_captured_step_equals_the_eager_one(hip, dtype, monkeypatch):
    w = ku.random_weights(MIXED, 72, edit=lively)
    prompt = ku.tokens(MIXED, 37, 15)
    got = []
    for graph in ("1", "0"):
        monkeypatch.setenv("LITENN_HIP_GRAPH", graph)
        model = hip.create_model(MIXED, w, dtype=dtype, context_length=300)
        got.append(model.generate(prompt, 120)[0].tolist())
        model.close()
    assert got[0] == got[1]


@pytest.mark.parametrize("dtype", DTYPES)
def test_generation_in_portions_of_the_prompt(hip, dtype):
    """The prompt fed ahead in portions, or all by generate() itself: the same tokens."""
    model, plain = pair(hip, MIXED, 73, dtype, edit=lively)
    prompt = ku.tokens(MIXED, 90, 15)
    whole, _, _ = model.generate(prompt, 12)
    model.reset()
    model.eval(prompt[:50], want=[])
    model.eval(prompt[50:53], want=[])
    parts, _, _ = model.generate(prompt[53:], 12)
    if dtype == "float32":
        assert parts.tolist() == whole.tolist() == plain.greedy(prompt, 12)[0]
    else:
        # rounding may decide a near-tie: up to there the tokens agree
        margin = plain.greedy(prompt, 12)[1]
        first = next((i for i in range(12) if parts[i] != whole[i]), 12)
        assert first == 12 or margin[first] < 0.2
    model.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_replay(hip, tmp_path, dtype):
    """bin/trace_run on a folder: requests one after the other, in portions, wanted places in any order."""
    cfg = ku.config([ku.attention(window=14, mlp=ku.mlp()), ku.linear_attention()])
    w = ku.random_weights(cfg, 81)
    folder = ku.write_folder(tmp_path / "model", cfg, w)
    out = tmp_path / "out"
    out.mkdir()
    plain = ref.NumpyKulurax(cfg, ku.as_floats(w))
    a, b = ku.tokens(cfg, 60, 17), ku.tokens(cfg, 21, 18)
    plan = [("a", a[:33], [32, 0, 5]), ("a", a[33:35], []), ("a", a[35:36], [0]), ("a", a[36:], [23, 1]), ("b", b[:20], [3]),
            ("b", b[20:], [0])]
    lines, at = [], {"a": 0, "b": 0}
    expected = []
    for n, (rid, toks, want) in enumerate(plan):
        ends = [rid] if (n + 1 == len(plan) or plan[n + 1][0] != rid) else []
        lines.append(json.dumps({"step": n, "entries": [{"id": rid, "tokens": toks.tolist(), "want": want}], "end": ends}))
        expected.append((rid, [at[rid] + p for p in want]))
        at[rid] += len(toks)
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    run = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", folder, "--dtype", dtype, "--out",
                          str(out), "--max-tokens", "64"], input="\n".join(lines) + "\n", capture_output=True, text=True,
                         timeout=100)
    assert run.returncode == 0, run.stderr
    assert [x for x in run.stdout.splitlines() if x.startswith("done ")] == [f"done {n}" for n in range(len(plan))]
    full = {"a": plain.forward(a), "b": plain.forward(b)}
    for n, (rid, places) in enumerate(expected):
        path = out / f"{n}.f32"
        assert path.exists() == bool(places)
        if places:
            got = np.fromfile(path, "<f4").reshape(len(places), cfg["vocab"])
            d = got - full[rid][places]
            d -= d.mean(axis=1, keepdims=True)
            assert np.sqrt((d * d).mean(axis=1)).max() <= LIMIT[dtype] * full[rid].std()


def test_models_of_both_kinds_side_by_side(hip, oracle):
    """The registry's other loader: the handle of a LLaMA model behaves as any model's."""
    from llama_util import hip_model
    from litenn_amd import synth, _lib
    from litenn_amd.formats import Q4_0
    cfg = synth.tiny_llama(Q4_0)
    llama = hip_model(hip, cfg, 5)
    prompt = synth.prompt_tokens(cfg, 8, 3)
    want, _, _ = llama.generate(prompt, 8)
    import ctypes
    handle = ctypes.c_void_p(_lib.load().litenn_hip_llama_model(llama._h))
    as_model = hip.Model(handle)
    assert as_model.architecture == "llama" and as_model.vocab_size == cfg.vocab
    other, plain = pair(hip, SINGLE["gla"], 91, "float32")
    toks = ku.tokens(SINGLE["gla"], 20, 1)
    as_model.reset()
    got = as_model.eval(prompt, want=[7, 2], precise=True)
    assert ku.error(other.eval(toks), plain.forward(toks)) <= LIMIT["float32"]
    llama.reset()
    assert np.array_equal(got, llama.eval(prompt)[[7, 2]])
    as_model.reset()
    assert as_model.generate(prompt, 8)[0].tolist() == want.tolist()
    as_model._h = ctypes.c_void_p()  # one owner
    llama.close()
    other.close()
