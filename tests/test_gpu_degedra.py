"""Degedra models through the framework's own entry points (evaluation, portions, greedy generation, trace
replay) against the plain numpy restatement in np_degedra.py: small models with seeded weights."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import degedra_util as du
import np_degedra as ref

pytestmark = pytest.mark.gpu

LIMIT = {"float32": 3e-5, "bfloat16": 4e-2}
DTYPES = ("float32", "bfloat16")


def pair(hip, cfg, seed, dtype, context_length=600, **kw):
    w = du.random_weights(cfg, seed, **kw)
    return hip.create_model(cfg, w, dtype=dtype, context_length=context_length), ref.NumpyDegedra(cfg, du.as_floats(w))


def feed(model, toks, cuts):
    """Logits of every position, the tokens fed in portions of the given sizes (the last one repeats)."""
    out, at, i = [], 0, 0
    while at < len(toks):
        n = min(cuts[min(i, len(cuts) - 1)], len(toks) - at)
        out.append(model.eval(toks[at:at + n]))
        at += n
        i += 1
    return np.concatenate(out)


# (parts of a norm that hold one head each would let single tokens whose state cancels dominate the 16-bit errors)
_OWN = [du.layer(ff=72), du.layer(du.attention(4, 4, 40, 21, 0.2, 40, 1e4), du.state_space(4, 36, 33, 1, 2, 3), left_scale=1.1),
        du.layer(du.attention(10, 1, 16, 70, 0.25, 8), du.state_space(2, 70, 65, 2, 1, 2), ff=50, right_scale=-0.7)]
MIXED = du.config([_OWN[0], _OWN[1], du.again(_OWN, 0), _OWN[2], {**_OWN[1], "weights_of": 1}])


def left_only(a):
    return du.layer(a, right_scale=0.0)


def right_only(r):
    return du.layer(None, r, left_scale=0.0)


SINGLE = {
    "attention": left_only(du.attention()),
    "attention_odd": left_only(du.attention(3, 3, 13, 6, 1.0, 4)),
    "attention_ones": left_only(du.attention(1, 1, 1, 1, 1.0, 0)),
    "attention_pair": left_only(du.attention(2, 1, 2, 2, 1.0, 2)),
    "attention_unrotated": left_only(du.attention(rot_dims=0)),
    "attention_one_group": left_only(du.attention(20, 1, 32, 33, 0.2, 32)),   # more query heads than a workgroup takes
    "attention_wide_share": left_only(du.attention(27, 3, 72, 50, 0.1, 20)),
    "attention_own_keys": left_only(du.attention(5, 5, 64, 64, 0.1, 64)),
    "attention_mid": left_only(du.attention(2, 2, 136, 70, 0.1, 100)),
    "attention_256": left_only(du.attention(4, 2, 256, 100, 0.05, 256)),
    "attention_beyond_tiles": left_only(du.attention(4, 1, 264, 40, 0.05, 130)),
    "attention_largest": left_only(du.attention(3, 1, 512, 20, 0.05, 512)),
    "attention_many_queries": left_only(du.attention(32, 2, 128, 33, 0.09, 128)),
    "attention_more_queries": left_only(du.attention(40, 2, 200, 33, 0.07, 96)),
    "attention_most_queries": left_only(du.attention(48, 2, 256, 33, 0.06, 256)),
    "attention_many_odd_queries": left_only(du.attention(90, 5, 33, 40, 0.2, 18)),
    "attention_sees_all": left_only(du.attention(4, 2, 32, 5000, 0.1, 32)),
    "ssm": right_only(du.state_space()),
    "ssm_ones": right_only(du.state_space(1, 1, 1, 1, 1, 1)),
    "ssm_odd": right_only(du.state_space(3, 7, 5, 3, 7, 2)),
    "ssm_one_group": right_only(du.state_space(8, 16, 64, 1, 1, 4)),
    "ssm_no_history": right_only(du.state_space(4, 24, 16, 2, 4, 1)),
    "ssm_many_taps": right_only(du.state_space(4, 24, 16, 2, 3, 9)),
    "ssm_wide_state": right_only(du.state_space(2, 33, 300, 1, 2, 4)),
    "ssm_largest_state": right_only(du.state_space(1, 64, 512, 1, 1, 4)),
    "ssm_wide_values": right_only(du.state_space(2, 130, 70, 2, 5, 3)),
    "ssm_each_its_norm": right_only(du.state_space(6, 10, 17, 6, 60, 3)),
    "both": du.layer(),
    "both_odd": du.layer(du.attention(3, 1, 13, 6, 1.0, 4), du.state_space(3, 7, 5, 3, 1, 2), ff=33),
    "feed_forward": du.layer(ff=88),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(SINGLE))
def test_each_mechanism_alone(hip, name, dtype):
    """A prompt in one pass, its tail token by token, and all of it in short portions, for many sizes."""
    cfg = du.config([SINGLE[name]], **({"vocab": 67, "width": 50} if name.endswith(("odd", "ones")) else {}))
    model, plain = pair(hip, cfg, 11, dtype, context_length=200)
    toks = du.tokens(cfg, 150, 5)
    want = plain.forward(toks)
    for cuts in ([150], [110, 1], [2, 33, 5, 64, 7]):
        model.reset()
        assert du.error(feed(model, toks, cuts), want) <= LIMIT[dtype], cuts
    model.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [6, 53, 64, 200])
def test_embedding_norms_and_head(hip, width, dtype):
    """Sublayers whose output norm is zero leave the embedding, the last norm and the capped head."""
    cfg = du.config([du.layer(ff=20)], width=width, softcap=1.5)

    def silence(w):
        w["l0.norm1"][:] = w["l0.norm2"][:] = 0

    model, plain = pair(hip, cfg, 3, dtype, edit=silence)
    toks = du.tokens(cfg, 40, 1)
    x = plain.w["embed"][toks]
    raw = x / np.sqrt(np.mean(x * x, -1, keepdims=True) + cfg["norm"]["eps"]) * plain.w["final.norm"] @ plain.w["head"].T
    want = 1.5 * np.tanh(raw / 1.5)
    assert du.error(raw, want) > 0.2  # the cap shows
    for cuts in ([40], [1]):
        model.reset()
        assert du.error(feed(model, toks, cuts), want) <= LIMIT[dtype]
    model.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cuts", [[1], [2], [3], [2, 5, 3], [4], [7], [15, 16], [17], [40, 2, 64, 3, 1], [63, 64, 65, 2], [300]])
def test_portions_of_every_size(hip, cuts, dtype):
    """However a sequence is cut, every position's logits are the plain forward's."""
    model, plain = pair(hip, MIXED, 21, dtype)
    toks = du.tokens(MIXED, 210, 2)
    assert du.error(feed(model, toks, cuts), plain.forward(toks)) <= LIMIT[dtype]
    assert model.past == len(toks)
    model.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_long_run_laps_the_cache_ring(hip, dtype, monkeypatch):
    """Passes of 8 tokens make rings of window + 7 rows: a prompt and a long decode go around them many times,
    and prompts longer than a pass are cut by the framework itself."""
    monkeypatch.setenv("LITENN_HIP_PASS_ROWS", "8")
    model, plain = pair(hip, MIXED, 22, dtype)
    toks = du.tokens(MIXED, 420, 3)
    want = plain.forward(toks)
    assert du.error(feed(model, toks, [90, 1, 1, 1, 1, 1, 100, 1]), want) <= LIMIT[dtype]
    model.close()
    monkeypatch.setenv("LITENN_HIP_PASS_ROWS", "33")
    model, plain = pair(hip, MIXED, 22, dtype)
    got = model.eval(toks, want=[419, 0, 32, 33, 34, 65, 66, 200])  # any order, across passes
    assert du.error(got, want[[419, 0, 32, 33, 34, 65, 66, 200]]) <= LIMIT[dtype]
    model.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_cache_is_the_context_when_that_is_shorter(hip, dtype):
    model, plain = pair(hip, MIXED, 23, dtype, context_length=40)
    toks = du.tokens(MIXED, 40, 4)
    assert du.error(feed(model, toks, [18, 1, 20, 1]), plain.forward(toks)) <= LIMIT[dtype]
    with pytest.raises(hip.LiteNNHipError, match="context length exceeded"):
        model.eval([1])
    model.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_sequence_does_not_see_the_one_before(hip, dtype):
    """After a reset a sequence's logits are bit for bit those of a fresh model, whatever ran before."""
    w = du.random_weights(MIXED, 24)
    first, second = du.tokens(MIXED, 130, 5), du.tokens(MIXED, 61, 6)
    cuts = [1, 2, 37, 1, 1, 5, 1]
    fresh = hip.create_model(MIXED, w, dtype=dtype, context_length=300)
    want = feed(fresh, second, cuts)
    fresh.close()
    used = hip.create_model(MIXED, w, dtype=dtype, context_length=300)
    feed(used, first, [100, 1])
    used.generate(first[:20], 30)
    used.reset()
    assert used.past == 0
    assert np.array_equal(feed(used, second, cuts), want)
    used.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_layers_that_share_weights_hold_their_own_state(hip, dtype):
    """The owner may stand ahead or behind, and may be named through another layer that shares."""
    own = [du.layer(ff=30), du.layer(du.attention(2, 1, 16, 12, 0.3, 16), ff=None)]
    layers = [{**own[1], "weights_of": 3}, own[0], {**own[0], "weights_of": 1}, own[1], {**own[1], "weights_of": 0}]
    model, plain = pair(hip, du.config(layers), 25, dtype)
    toks = du.tokens(du.config(layers), 90, 7)
    assert du.error(feed(model, toks, [50, 1, 2, 9, 1]), plain.forward(toks)) <= LIMIT[dtype]
    model.close()


BEACON, ASKER = 3, 7


def beacon_model(window, kv_heads=2):
    """One attention layer in which token ASKER looks for token BEACON among keys that carry nothing: one
    component of the embeddings marks either, and one unrotated dimension of a head holds the mark."""
    cfg = du.config([du.layer(du.attention(4, kv_heads, 24, window, 1.0, 16), right_scale=0.0)], vocab=40, width=64)

    def edit(w):
        w["embed"][:, :2] = 0
        w["embed"][BEACON, 0] = w["embed"][ASKER, 1] = 6.0
        w["l0.mix.left.q.norm"][:] = w["l0.mix.left.k.norm"][:] = 1
        for name, mark in (("q", 1), ("k", 0)):
            rows = w[f"l0.mix.left.{name}"]
            rows[:, :2] = 0
            rows[20::24, mark] = 4.0  # dimension 20 of every head
        w["l0.norm1"] *= 3.0
    return cfg, du.random_weights(cfg, 33, edit=edit)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", [2, 31, 64, 65, 128, 300])
def test_a_far_key_is_seen_up_to_the_windows_edge(hip, window, dtype, monkeypatch):
    """The asked-for key lies right behind the asker, just inside and just outside the window, in prompts and in
    decoding, at several places of the ring; a window one position off moves those logits."""
    monkeypatch.setenv("LITENN_HIP_PASS_ROWS", "48")
    cfg, w = beacon_model(window)
    plain = ref.NumpyDegedra(cfg, du.as_floats(w))
    model = hip.create_model(cfg, w, dtype=dtype, context_length=1000)
    limit = {"float32": 1e-4, "bfloat16": 0.1}[dtype]
    for at in (0, 47, 130):
        toks = np.random.default_rng([6, at]).integers(8, 40, at + window + 70).astype(np.int32)
        toks[at] = BEACON
        toks[[at + 1, at + window - 1, at + window]] = ASKER
        want = plain.forward(toks)
        for off, place in ((-1, at + window - 1), (1, at + window)):
            wrong = json.loads(json.dumps(cfg))
            wrong["layers"][0]["mixer"]["left"]["mask"]["size"] = window + off
            assert du.row_errors(ref.NumpyDegedra(wrong, du.as_floats(w)).forward(toks), want)[place] > 0.3
        for cuts in ([1000], [at + 1, 1], [37, 2, 64, 3], [1] * (at + window - 5) + [2, 9, 1000]):
            model.reset()
            assert du.error(feed(model, toks, cuts), want) <= limit, (at, cuts)
    model.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", [1, 3, 32, 63, 64, 65, 100])
def test_window_edges_with_sharp_scores(hip, window, dtype):
    """Scores spread so far that few keys carry a query: a window one position off, in a prompt or in decoding,
    would move the logits by far more than the tolerance."""
    cfg = du.config([du.layer(du.attention(4, 2, 16, window, 1.0, 8), right_scale=0.0)], vocab=48, width=64)
    w = du.random_weights(cfg, 31, edit=lambda w: w["l0.norm1"].__imul__(4.0))
    plain = ref.NumpyDegedra(cfg, du.as_floats(w))
    toks = du.tokens(cfg, 180, 9)
    want = plain.forward(toks)
    for off in (-1, 1):
        if window + off < 1:
            continue
        wrong = json.loads(json.dumps(cfg))
        wrong["layers"][0]["mixer"]["left"]["mask"]["size"] = window + off
        assert du.error(ref.NumpyDegedra(wrong, du.as_floats(w)).forward(toks), want) > 0.2
    model = hip.create_model(cfg, w, dtype=dtype, context_length=200)
    for cuts in ([180], [100, 1], [37, 2, 64, 3]):
        model.reset()
        assert du.error(feed(model, toks, cuts), want) <= {"float32": 1e-4, "bfloat16": 0.15}[dtype], cuts
    model.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_rotation_at_far_positions(hip, dtype):
    """Angles of thousands of radians, across two passes and into decoding: a fraction lost there would turn
    neighbouring keys against each other."""
    cfg = du.config([du.layer(du.attention(2, 1, 8, 40, 1.0, 8, 3.0), right_scale=0.0)], vocab=50, width=24)
    model, plain = pair(hip, cfg, 34, dtype, context_length=4300)
    toks = du.tokens(cfg, 4260, 10)
    want = plain.forward(toks)
    got = model.eval(toks[:4200])
    got = np.concatenate([got, feed(model, toks[4200:], [1])])
    assert du.error(got, want) <= {"float32": 1e-4, "bfloat16": 0.1}[dtype]
    model.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rates,steps", [((4.0, 6.0), (2.0, 4.0)), ((-9.0, 6.0), (-2.0, 3.0)), ((-8.0, -6.0), (-6.0, -4.0)),
                                         ((-2.0, 2.0), (-30.0, -20.0)), ((0.0, 1.0), (20.0, 40.0))])
def test_decays_from_instant_to_endless(hip, rates, steps, dtype):
    """Heads that forget within one token beside heads that keep hundreds, and step sizes from next to nothing
    to large ones: no factor of the chunked form may overflow or vanish where the recurrence does not."""
    cfg = du.config([du.layer(None, du.state_space(6, 24, 40, 2, 6), left_scale=0.3),
                     du.layer(None, du.state_space(3, 48, 70, 1, 3), left_scale=0.3)])
    model, plain = pair(hip, cfg, 51, dtype, rates=rates, steps=steps)
    toks = du.tokens(cfg, 330, 10)
    want = plain.forward(toks)
    assert np.all(np.isfinite(want))
    for cuts in ([330], [129, 1, 1, 64, 1, 70, 3]):
        model.reset()
        errors = du.row_errors(feed(model, toks, cuts), want)
        if dtype == "float32":
            assert errors.max() <= LIMIT[dtype], cuts
        else:
            # a head that forgets at once is C . B times x, normalised: where C . B comes out near zero the operands'
            # rounding decides its sign, so single rows may be far off in 16 bits
            assert np.median(errors) <= LIMIT[dtype] / 2 and np.mean(errors > LIMIT[dtype]) <= 0.2, cuts
    model.close()


def test_the_state_is_carried_in_32_bits(hip):
    """A slowly decaying state over a long sequence, in the serving precisions: a state kept in 16 bits would
    lose the small additions."""
    cfg = du.config([right_only(du.state_space(2, 16, 16, 1, 1))])
    model, plain = pair(hip, cfg, 52, "bfloat16", context_length=1200, rates=(-6.0, -5.0), steps=(-3.0, -2.0))
    toks = du.tokens(cfg, 1100, 11)
    assert du.error(feed(model, toks, [700, 1]), plain.forward(toks)) <= LIMIT["bfloat16"]
    model.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("taps", [1, 2, 3, 5, 8])
def test_the_convolution_across_portions(hip, taps, dtype):
    """Only the oldest tap has weight: a token's inputs come from the portion before, or from nowhere."""
    cfg = du.config([right_only(du.state_space(4, 20, 9, 2, 2, taps))])

    def edit(w):
        w["l0.mix.right.conv"][:, 1:] = 0
        w["l0.mix.right.conv"][:, 0] = 1.5
    model, plain = pair(hip, cfg, 53, dtype, edit=edit)
    toks = du.tokens(cfg, 60, 12)
    want = plain.forward(toks)
    for cuts in ([60], [1], [2], [5, 1, 4, 2], [3, 1, 33, 1]):
        model.reset()
        assert du.error(feed(model, toks, cuts), want) <= LIMIT[dtype], cuts
    model.close()


def test_no_projection_norm_by_heads(hip):
    """Queries and keys are normalised as whole projections: heads of very different size keep their ratio."""
    cfg = du.config([left_only(du.attention(6, 3, 16, 30, 0.5, 16))])

    def edit(w):
        for name, rows in (("q", 96), ("k", 48)):
            w[f"l0.mix.left.{name}"] *= np.repeat([4.0, 1.0, 0.1], rows // 3)[:, None].astype(np.float32)
    model, plain = pair(hip, cfg, 54, "float32", edit=edit)
    toks = du.tokens(cfg, 80, 13)
    want = plain.forward(toks)
    assert du.error(feed(model, toks, [50, 1]), want) <= LIMIT["float32"]
    model.close()


def test_greedy_generation(hip):
    """generate(): the prompt in passes, then the captured step, against the plain form's greedy tokens; again
    after other work on the same model (replays of the same captured step), and continued."""
    model, plain = pair(hip, MIXED, 71, "float32")
    prompt = du.tokens(MIXED, 45, 12)
    want, margins = plain.greedy(prompt, 40)
    assert min(margins) > 1e-3 and len(set(want)) > 10  # no near-tie in this sequence, no single repeated token
    for _ in range(3):
        model.reset()
        got, _, _ = model.generate(prompt, 40)
        assert got.tolist() == want
        assert model.past == 45 + 39
        model.eval(du.tokens(MIXED, 30, 14))
        model.eval([1], want=[0])
    model.reset()
    head, _, _ = model.generate(prompt, 15)
    tail, _, _ = model.generate(head[-1:], 25)
    assert head.tolist() + tail.tolist() == want
    model.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_captured_step_equals_the_eager_one(hip, dtype, monkeypatch):
    w = du.random_weights(MIXED, 72)
    prompt = du.tokens(MIXED, 37, 15)
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
    model, plain = pair(hip, MIXED, 73, dtype)
    prompt = du.tokens(MIXED, 90, 15)
    whole, _, _ = model.generate(prompt, 12)
    model.reset()
    model.eval(prompt[:50], want=[])
    model.eval(prompt[50:53], want=[])
    parts, _, _ = model.generate(prompt[53:], 12)
    want, margin = plain.greedy(prompt, 12)
    for got in (whole, parts):
        # rounding may decide a near-tie: up to there the tokens agree
        first = next((i for i in range(12) if got[i] != want[i]), 12)
        assert first == 12 or margin[first] < {"float32": 1e-3, "bfloat16": 0.2}[dtype]
    model.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_replay(hip, tmp_path, dtype):
    """bin/trace_run on a folder: requests one after the other, in portions, wanted places in any order."""
    layers = [du.layer(ff=40), du.layer(du.attention(4, 1, 16, 14, 0.3, 16))]
    cfg = du.config(layers + [du.again(layers, 0)])
    w = du.random_weights(cfg, 81)
    folder = du.write_folder(tmp_path / "model", cfg, w)
    out = tmp_path / "out"
    out.mkdir()
    plain = ref.NumpyDegedra(cfg, du.as_floats(w))
    a, b = du.tokens(cfg, 60, 17), du.tokens(cfg, 21, 18)
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


def random_config(seed):
    """Two or three layers of sizes drawn at random, one perhaps with another's weights."""
    rng = np.random.default_rng([seed, 91])

    def pick(*values):
        return values[int(rng.integers(len(values)))]

    layers = []
    for _ in range(int(rng.integers(1, 4))):
        kv_heads, dim = int(rng.integers(1, 5)), int(rng.integers(1, 100))
        left = du.attention(kv_heads * int(rng.integers(1, 12)), kv_heads, dim, int(rng.integers(1, 150)),
                            float(rng.uniform(0.3, 1.0) / np.sqrt(dim)), 2 * int(rng.integers(0, dim // 2 + 1)),
                            float(rng.uniform(2.0, 1e5)))
        groups, per_group, vdim = int(rng.integers(1, 4)), int(rng.integers(1, 5)), int(rng.integers(1, 100))
        inner = groups * per_group * vdim
        parts = pick(*[n for n in range(1, 9) if inner % n == 0 and inner // n >= 16] or [1])
        right = du.state_space(groups * per_group, vdim, int(rng.integers(1, 150)), groups, parts, int(rng.integers(1, 7)))
        layers.append(du.layer(left, right, pick(None, int(rng.integers(1, 300))), float(rng.uniform(0.3, 1.5)),
                               float(rng.uniform(0.3, 1.5))))
    if pick(0, 1):
        layers.append(du.again(layers, int(rng.integers(len(layers)))))
    return du.config(layers, int(rng.integers(2, 300)), int(rng.integers(8, 300)), 10.0 ** -int(rng.integers(3, 7)),
                     float(rng.uniform(2.0, 50.0)))


@pytest.mark.parametrize("seed", range(24))
def test_random_configurations(hip, seed):
    """Sizes nobody chose, in portions nobody chose; 16 bits beside 32 on the same tokens."""
    cfg = random_config(seed)
    rng = np.random.default_rng([seed, 92])
    w = du.random_weights(cfg, seed)
    plain = ref.NumpyDegedra(cfg, du.as_floats(w))
    toks = du.tokens(cfg, int(rng.integers(100, 260)), seed)
    want = plain.forward(toks)
    cuts = [int(n) for n in rng.integers(1, rng.integers(4, 90), 40)] + [1]
    for dtype in DTYPES:
        model = hip.create_model(cfg, w, dtype=dtype, context_length=300)
        errors = du.row_errors(feed(model, toks, cuts), want)
        model.close()
        # in 16 bits a token whose mixers nearly cancel may be far off
        assert (errors.max() if dtype == "float32" else np.quantile(errors, 0.9)) <= LIMIT[dtype], (dtype, cfg, cuts)
