"""Host side of the layered decoder: configuration and checkpoint errors come back as messages before any
device work, and the plain numpy forms used by the device tests agree with independent restatements."""
import json
import os
import struct

import numpy as np
import pytest

import kulurax_util as ku
import np_kulurax as ref
import litenn_amd as ln

CFG = ku.config([ku.linear_attention(), ku.attention(mlp=ku.mlp())])


def load_error(folder):
    with pytest.raises(ln.LiteNNHipError) as e:
        ln.load_model(folder)
    return str(e.value)


def edited(tmp_path, change):
    cfg = json.loads(json.dumps(CFG))
    change(cfg)
    return ku.write_folder(tmp_path, cfg, ku.random_weights(CFG, 1))


@pytest.mark.parametrize("change,text", [
    (lambda c: c.update(architecture="Other"), "unknown architecture 'Other'"),
    (lambda c: c.pop("architecture"), "no 'architecture'"),
    (lambda c: c.pop("vocab"), "no 'vocab'"),
    (lambda c: c.update(width=1.5), "'width' is not a whole number"),
    (lambda c: c.update(layers=[]), "'layers' is not a list"),
    (lambda c: c["layers"][0].update(type="mamba"), "unknown layer type 'mamba'"),
    (lambda c: c["layers"][0]["mixer"].pop("tau"), "no 'tau'"),
    (lambda c: c["layers"][0]["mixer"].update(tau=0), "'tau' must be greater"),
    (lambda c: c["layers"][1]["mixer"].update(kv_rank=5000), "'kv_rank'"),
    (lambda c: c["layers"][1]["mixer"]["mask"].update(size=0), "'size'"),
    (lambda c: c["layers"][1]["mlp"].update(kind="sparse"), "unknown feed-forward kind 'sparse'"),
    (lambda c: c["layers"].append(ku.linear_attention()), "Missing tensor 'l2.mix.a1'"),
])
def test_configuration_errors(tmp_path, change, text):
    assert text in load_error(edited(tmp_path, change))


def test_checkpoint_errors(tmp_path):
    assert "cannot open" in load_error(tmp_path / "nowhere")
    folder = ku.write_folder(tmp_path / "m", CFG, ku.random_weights(CFG, 1))
    path = os.path.join(folder, "model.safetensors")
    whole = open(path, "rb").read()
    size = struct.unpack("<Q", whole[:8])[0]

    def variant(data):
        with open(path, "wb") as f:
            f.write(data)
        return load_error(folder)
    assert "lies outside the file" in variant(whole[:-10])
    assert "header longer than the file" in variant(struct.pack("<Q", 1 << 40) + whole[8:])
    assert "JSON" in variant(whole[:8] + b"[" * size + whole[8 + size:])
    header = json.loads(whole[8:8 + size])
    header["embed"]["shape"][0] += 1
    text = json.dumps(header).encode()
    assert "another size than its shape" in variant(struct.pack("<Q", len(text)) + text + whole[8 + size:])
    os.remove(path)
    assert "cannot open" in load_error(folder)
    ku.write_folder(tmp_path / "n", CFG, ku.random_weights(CFG, 1))
    with open(tmp_path / "n" / "config.json", "w") as f:
        f.write("{\"architecture\": \"Kulurax\"")
    assert "JSON" in load_error(tmp_path / "n")


def test_recurrence_against_the_sum_over_earlier_tokens():
    """o_t as the explicit double sum  sum_s (sum_d q_td k_sd prod_(s < r <= t) a_rd) v_s."""
    rng = np.random.default_rng(3)
    t, h, d, e = 9, 2, 4, 3
    q, k = rng.normal(size=(2, t, h, d))
    v = rng.normal(size=(t, h, e))
    log_a = -rng.uniform(0, 2, (t, h, d))
    o, s = ref.gla_recurrence(q, k, v, log_a)
    total = np.cumsum(log_a, axis=0)
    for i in range(t):
        want = sum(np.einsum("hd,he->he", q[i] * k[j] * np.exp(total[i] - total[j]), v[j]) for j in range(i + 1))
        assert np.allclose(o[i], want)
    want = sum(k[j][:, :, None] * np.exp(total[-1] - total[j])[:, :, None] * v[j][:, None, :] for j in range(t))
    assert np.allclose(s, want)


def test_window_attention_against_one_query_at_a_time():
    rng = np.random.default_rng(4)
    t, h, d, e, window = 11, 2, 5, 3, 4
    q, k = rng.normal(size=(2, t, h, d))
    v = rng.normal(size=(t, h, e))
    sink = rng.normal(size=h)
    got = ref.windowed_sink_attention(q, k, v, 0.7, window, sink)
    for i in range(t):
        for head in range(h):
            seen = [j for j in range(t) if 0 <= i - j < window]
            w = np.array([np.exp(0.7 * q[i, head] @ k[j, head]) for j in seen])
            assert np.allclose(got[i, head], (w[:, None] * v[seen, head]).sum(0) / (w.sum() + np.exp(sink[head])))


def test_position_vectors_and_activations():
    p = ref.sinusoid([0, 3], 6)
    assert np.allclose(p[0], [0, 1, 0, 1, 0, 1])
    angle = 3 * 10000.0 ** (-2 / 6)
    assert np.allclose(p[1][2:4], [np.sin(angle), np.cos(angle)])
    w = {"gate": np.eye(4), "up": np.eye(4), "down": np.eye(4)}
    h = np.array([[-3.0, -0.2, 0.2, 3.0]])
    g, u = np.array([-3.0, -0.2, 0.2, 1.0]), np.array([-1.0, -0.2, 0.2, 1.0])
    assert np.allclose(ref.clamped_glu(h, w, 1.0), g / (1 + np.exp(-1.702 * g)) * (u + 1))


def test_a_sequence_is_causal():
    w = ku.as_floats(ku.random_weights(CFG, 2))
    m = ref.NumpyKulurax(CFG, w)
    toks = ku.tokens(CFG, 30, 1)
    assert np.allclose(m.forward(toks)[:20], m.forward(toks[:20]))
