"""Host side of the Degedra decoder: configuration errors come back as messages before any device work, and the
plain numpy forms used by the device tests agree with independent restatements."""
import json

import numpy as np
import pytest

import degedra_util as du
import np_degedra as ref
import litenn_amd as ln

LAYERS = [du.layer(ff=40), du.layer()]
CFG = du.config(LAYERS + [du.again(LAYERS, 0)])


@pytest.mark.parametrize("change,text", [
    (lambda c: c.pop("width"), "no 'width'"),
    (lambda c: c.update(layers={}), "'layers' is not a list"),
    (lambda c: c.update(logit_softcap=0), "'logit_softcap' must be greater"),
    (lambda c: c["layers"][1].update(type="gla"), "unknown layer type 'gla'"),
    (lambda c: c["layers"][0]["mixer"].pop("left_scale"), "no 'left_scale'"),
    (lambda c: c["layers"][0]["mixer"]["left"].update(kv_heads=4), "'heads' is not a multiple of 'kv_heads'"),
    (lambda c: c["layers"][0]["mixer"]["left"].update(vdim=32), "'vdim' is not 'dim'"),
    (lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=7), "even number of dimensions"),
    (lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=26), "'dims'"),
    (lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(base=0), "base greater than zero"),
    (lambda c: c["layers"][0]["mixer"]["left"]["mask"].update(size=0), "'size'"),
    (lambda c: c["layers"][0]["mixer"]["right"].update(groups=4), "'heads' is not a multiple of 'groups'"),
    (lambda c: c["layers"][0]["mixer"]["right"].update(norm_groups=7), "'norm_groups' does not divide"),
    (lambda c: c["layers"][0]["mixer"]["right"].update(state=513), "'state'"),
    (lambda c: c["layers"][0]["mixer"]["right"].update(conv=0), "'conv'"),
    (lambda c: c["layers"][0]["mlp"].update(kind="sparse"), "unknown feed-forward kind 'sparse'"),
    (lambda c: c["layers"][2].update(weights_of=3), "'weights_of'"),
    (lambda c: c["layers"][0].update(weights_of=2), "in a circle"),
])
def test_configuration_errors(tmp_path, change, text):
    cfg = json.loads(json.dumps(CFG))
    change(cfg)
    folder = du.write_folder(tmp_path, cfg, du.random_weights(CFG, 1))
    with pytest.raises(ln.LiteNNHipError) as e:
        ln.load_model(folder)
    assert text in str(e.value)


def test_recurrence_against_the_sum_over_earlier_tokens():
    """y_t as the explicit double sum  sum_s (C_t . B_s) dt_s prod_(s < r <= t) a_r  x_s."""
    rng = np.random.default_rng(3)
    t, h, n, v = 9, 2, 4, 3
    b, c = rng.normal(size=(2, t, h, n))
    x = rng.normal(size=(t, h, v))
    log_a, dt = -rng.uniform(0, 2, (t, h)), rng.uniform(0, 1, (t, h))
    y, state = ref.ssm_recurrence(x, b, c, log_a, dt)
    total = np.cumsum(log_a, axis=0)
    for i in range(t):
        for head in range(h):
            want = sum((c[i, head] @ b[s, head]) * dt[s, head] * np.exp(total[i, head] - total[s, head]) * x[s, head]
                       for s in range(i + 1))
            assert np.allclose(y[i, head], want)
    head, tail = ref.ssm_recurrence(x[:5], b[:5], c[:5], log_a[:5], dt[:5])
    rest, last = ref.ssm_recurrence(x[5:], b[5:], c[5:], log_a[5:], dt[5:], tail)
    assert np.allclose(np.concatenate([head, rest]), y) and np.allclose(last, state)


def test_window_attention_against_one_query_at_a_time():
    rng = np.random.default_rng(4)
    t, h, g, d, window = 11, 6, 2, 5, 4
    q, k = rng.normal(size=(t, h, d)), rng.normal(size=(t, g, d))
    v = rng.normal(size=(t, g, d))
    got = ref.window_softmax(q, k, v, 0.7, window)
    for i in range(t):
        for head in range(h):
            of = 0 if head < 3 else 1
            seen = [j for j in range(t) if 0 <= i - j < window]
            w = np.array([np.exp(0.7 * q[i, head] @ k[j, of]) for j in seen])
            assert np.allclose(got[i, head], (w[:, None] * v[seen, of]).sum(0) / w.sum())


def test_rotation_against_complex_numbers():
    """A pair as a complex number turns by its angle; scores of rotated vectors depend on the distance only."""
    rng = np.random.default_rng(5)
    x = rng.normal(size=(4, 2, 9))
    got = ref.rotate_half(x, [0, 1, 7, 100], 6, 50.0)
    for r, p in enumerate([0, 1, 7, 100]):
        for i in range(3):
            z = (x[r, :, i] + 1j * x[r, :, i + 3]) * np.exp(1j * p * 50.0 ** (-2 * i / 6))
            assert np.allclose(got[r, :, i], z.real) and np.allclose(got[r, :, i + 3], z.imag)
    assert np.array_equal(got[..., 6:], x[..., 6:])
    a, b = rng.normal(size=(2, 1, 1, 8))
    near = ref.rotate_half(a, [9], 8, 50.0).ravel() @ ref.rotate_half(b, [4], 8, 50.0).ravel()
    far = ref.rotate_half(a, [1009], 8, 50.0).ravel() @ ref.rotate_half(b, [1004], 8, 50.0).ravel()
    assert np.allclose(near, far)


def test_convolution_gate_and_norm():
    x = np.arange(8.0).reshape(4, 2)
    w, b = np.array([[1.0, 10.0, 100.0], [0.0, 0.0, 1.0]]), np.array([0.5, -0.5])
    assert np.allclose(ref.causal_conv(x, w, b)[:, 0], [0.5, 200.5, 420.5, 642.5])
    assert np.allclose(ref.causal_conv(x, w, b)[:, 1], x[:, 1] - 0.5)
    y, z = np.array([[3.0, 4.0, 1.0, 1.0]]), np.array([[1.0, 1.0, 2.0, 2.0]])
    s1, s2 = 1 / (1 + np.exp(-1.0)), 2 / (1 + np.exp(-2.0))
    got = ref.gated_group_norm(y, z, np.array([1.0, 1.0, 1.0, 2.0]), 2, 0.25)
    r1, r2 = np.sqrt(12.5 * s1 ** 2 + 0.25), np.sqrt(s2 ** 2 + 0.25)
    assert np.allclose(got, [[3 * s1 / r1, 4 * s1 / r1, s2 / r2, 2 * s2 / r2]])


def test_a_sequence_is_causal_and_layers_share_weights():
    w = du.as_floats(du.random_weights(CFG, 2))
    m = ref.NumpyDegedra(CFG, w)
    toks = du.tokens(CFG, 30, 1)
    want = m.forward(toks)
    assert np.allclose(want[:20], m.forward(toks[:20]))
    spelled = json.loads(json.dumps(CFG))
    spelled["layers"][2].pop("weights_of")
    f = {**w, **{"l2." + k[3:]: v for k, v in w.items() if k.startswith("l0.")}}
    assert np.allclose(ref.NumpyDegedra(spelled, f).forward(toks), want)
    assert np.abs(want).max() < CFG["logit_softcap"]
