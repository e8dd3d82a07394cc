"""The layered decoder's mechanisms as single operators against plain numpy (float64) forms."""
import numpy as np
import pytest

import np_kulurax as ref
from conftest import rel_l2
from litenn_amd.formats import DT_BF16, DT_F32
from litenn_amd.model import from_bfloat16, to_bfloat16

pytestmark = pytest.mark.gpu


def pitch(k):
    return -(-k // 64) * 64


def padded_bits(a, fill=0):
    """bfloat16 bits of a [n, k] array in rows of pitch(k), `fill` behind the k-th element."""
    out = np.full((a.shape[0], pitch(a.shape[1])), fill, np.uint16)
    out[:, :a.shape[1]] = to_bfloat16(a)
    return out


def bf16_tensor(hip, bits):
    t = hip.Tensor(bits.shape, DT_BF16)
    hip.DeviceTraits.CopyFromCPU(t.device, DT_BF16, t.ptr, DT_BF16, np.ascontiguousarray(bits, np.uint16), bits.size)
    return t


def bf16_values(hip, t):
    out = np.empty(t.shape, np.uint16)
    hip.DeviceTraits.CopyToCPU(t.device, DT_BF16, t.ptr, t.size, DT_BF16, out)
    return from_bfloat16(out)


NAN16, NAN32 = 0x7FC0, np.float32(np.nan)


@pytest.mark.parametrize("n,k", [(1, 1), (7, 5), (130, 64), (65, 100), (300, 320), (96, 4096), (2049, 513), (4100, 96), (33, 8192)])
@pytest.mark.parametrize("m", [1, 2, 5, 31, 33, 64, 129, 200])
def test_linear_bf16(hip, n, k, m):
    """Every tile form, ragged in all three extents; what lies behind a row's last activation is never used
    (it is NaN here)."""
    rng = np.random.default_rng([n, k, m])
    w = padded_bits(rng.normal(0, 1, (n, k)).astype(np.float32))
    x = rng.normal(0, 1, (m, k)).astype(np.float32)
    wt = bf16_tensor(hip, w)
    wf = from_bfloat16(w)[:, :k].astype(np.float64)
    x32 = np.full((m, pitch(k)), NAN32, np.float32)
    x32[:, :k] = x
    y = hip.linear_bf16(wt, n, k, hip.Tensor.from_numpy(x32), m).numpy()
    assert rel_l2(y, x.astype(np.float64) @ wf.T) <= 5e-6
    xb = padded_bits(x, NAN16)
    y = hip.linear_bf16(wt, n, k, bf16_tensor(hip, xb), m).numpy()
    assert rel_l2(y, from_bfloat16(xb)[:, :k].astype(np.float64) @ wf.T) <= 2e-6


@pytest.mark.parametrize("n,k,m", [(12288, 512, 520), (8192, 256, 700), (2048, 1024, 513), (640, 256, 2000)])
def test_linear_bf16_larger(hip, n, k, m):
    """Sizes at which the large tiles run."""
    rng = np.random.default_rng([n, k, m])
    w = padded_bits(rng.normal(0, 1, (n, k)).astype(np.float32))
    xb = padded_bits(rng.normal(0, 1, (m, k)).astype(np.float32))
    y = hip.linear_bf16(bf16_tensor(hip, w), n, k, bf16_tensor(hip, xb), m).numpy()
    assert rel_l2(y, from_bfloat16(xb).astype(np.float64) @ from_bfloat16(w).astype(np.float64).T) <= 2e-6


def plain_window_attn(q, k, v, q_pos, k_pos, window, scale, sink):
    """Every score, then the mask, then the softmax with the sink; positions are absolute."""
    back = (q_pos + np.arange(q.shape[0]))[:, None] - (k_pos + np.arange(k.shape[0]))[None, :]
    s = np.einsum("ihd,jhd->hij", q, k) * scale
    s = np.where((back >= 0) & (back < window), s, -np.inf)
    top = s.max(axis=-1, keepdims=True)
    if sink is not None:
        top = np.maximum(top, sink[:, None, None])
    e = np.exp(s - top)
    total = e.sum(axis=-1, keepdims=True)
    if sink is not None:
        total = total + np.exp(sink[:, None, None] - top)
    return np.einsum("hij,jhe->ihe", e / total, v)


def window_case(hip, dtype, m, keys, heads, dim, vdim, window, k_pos, q_pos, scale, with_sink=True, with_gate=True, spike=None, seed=0):
    """Runs the operator and the plain form; spike(q, k) may edit the operands first."""
    rng = np.random.default_rng([m, keys, heads, dim, vdim, window, seed])
    q = rng.normal(0, 1, (m, heads, dim)).astype(np.float32)
    k = rng.normal(0, 1, (keys, heads, dim)).astype(np.float32)
    v = rng.normal(0, 1, (keys, heads, vdim)).astype(np.float32)
    if spike:
        spike(q, k)
    q = from_bfloat16(to_bfloat16(q))  # what the matrix-core form multiplies
    sink = rng.normal(0.5, 1, heads).astype(np.float32) if with_sink else None
    gate = rng.normal(0, 1, (m, heads * vdim)).astype(np.float32) if with_gate else None
    kv = np.concatenate([k.reshape(keys, -1), v.reshape(keys, -1)], axis=1)
    if dtype == DT_BF16:
        bits = to_bfloat16(kv)
        kvt, kv = bf16_tensor(hip, bits), from_bfloat16(bits)
    else:
        kvt = hip.Tensor.from_numpy(kv)
    out = hip.window_attn(hip.Tensor.from_numpy(q), kvt, m, keys, heads, dim, vdim, window, scale, k_pos, q_pos,
                          hip.Tensor.from_numpy(sink) if with_sink else None, hip.Tensor.from_numpy(gate) if with_gate else None)
    got = (bf16_values(hip, out) if dtype == DT_BF16 else out.numpy()).reshape(m, heads, vdim)
    kd = kv[:, :heads * dim].reshape(keys, heads, dim).astype(np.float64)
    vd = kv[:, heads * dim:].reshape(keys, heads, vdim).astype(np.float64)

    def plain(win=window, snk=sink):
        o = plain_window_attn(q.astype(np.float64), kd, vd, q_pos, k_pos, win, scale, snk)
        return o * ref.sigmoid(gate.astype(np.float64)).reshape(o.shape) if with_gate else o
    return got, plain


WINDOW_LIMIT = {DT_F32: 2e-6, DT_BF16: 8e-3}


@pytest.mark.parametrize("dtype", [DT_F32, DT_BF16])
@pytest.mark.parametrize("heads,dim,vdim", [(2, 64, 64), (3, 24, 40), (1, 13, 7), (2, 128, 128), (2, 72, 200), (1, 256, 256), (2, 136, 64),
                                            (1, 300, 280)])
@pytest.mark.parametrize("m,keys,k_pos,q_pos,window", [(1, 1, 0, 0, 1), (70, 70, 0, 0, 25), (64, 191, 5, 132, 128), (130, 200, 0, 70, 1000),
                                                       (17, 80, 40, 103, 64)])
def test_window_attention(hip, m, keys, k_pos, q_pos, window, heads, dim, vdim, dtype):
    got, plain = window_case(hip, dtype, m, keys, heads, dim, vdim, window, k_pos, q_pos, dim ** -0.5)
    assert rel_l2(got, plain()) <= WINDOW_LIMIT[dtype]


@pytest.mark.parametrize("dtype", [DT_F32, DT_BF16])
def test_window_attention_without_sink_and_gate(hip, dtype):
    got, plain = window_case(hip, dtype, 90, 90, 2, 64, 64, 33, 0, 0, 0.125, with_sink=False, with_gate=False)
    assert rel_l2(got, plain()) <= WINDOW_LIMIT[dtype]


@pytest.mark.parametrize("dtype", [DT_F32, DT_BF16])
@pytest.mark.parametrize("window", [1, 2, 63, 64, 65, 127, 128, 129])
def test_a_key_at_the_windows_edge(hip, window, dtype):
    """One query's score with the key just inside its window stands far out, another's with the key just
    outside: a window one position off changes those rows completely."""
    m, base = 200, 0
    inside, outside = 150, 170

    def spike(q, k):
        k[inside - (window - 1)] = 3.0 * q[inside]
        k[outside - window] = 3.0 * q[outside]
    got, plain = window_case(hip, dtype, m, m, 2, 64, 64, window, base, 0, 0.5, spike=spike)
    want = plain()
    assert rel_l2(got, want) <= WINDOW_LIMIT[dtype]
    for row in (inside, outside):
        assert rel_l2(got[row], want[row]) <= WINDOW_LIMIT[dtype]
    if window > 1:
        assert rel_l2(plain(win=window - 1)[inside], want[inside]) > 0.2
    assert rel_l2(plain(win=window + 1)[outside], want[outside]) > 0.2


@pytest.mark.parametrize("dtype", [DT_F32, DT_BF16])
def test_a_far_key_among_hundreds(hip, dtype):
    def spike(q, k):
        k[3] = 3.0 * q[699]
    got, plain = window_case(hip, dtype, 700, 700, 1, 64, 32, 5000, 0, 0, 0.5, spike=spike)
    want = plain()
    assert rel_l2(got[699], want[699]) <= WINDOW_LIMIT[dtype]
    assert rel_l2(got, want) <= WINDOW_LIMIT[dtype]


def test_the_sink_outweighs_or_vanishes(hip):
    """Sinks far above and far below every score: the result goes to zero or to the plain softmax, without overflow."""
    for level in (80.0, -200.0):
        rng = np.random.default_rng(4)
        m, heads, dim, vdim = 40, 2, 32, 32
        q, k = (rng.normal(0, 1, (m, heads, dim)).astype(np.float32) for _ in range(2))
        v = rng.normal(0, 1, (m, heads, vdim)).astype(np.float32)
        sink = np.full(heads, level, np.float32)
        kv = np.concatenate([k.reshape(m, -1), v.reshape(m, -1)], axis=1)
        want = plain_window_attn(q.astype(np.float64), k.astype(np.float64), v.astype(np.float64), 0, 0, 16, 1.0, sink)
        got = hip.window_attn(hip.Tensor.from_numpy(q), hip.Tensor.from_numpy(kv), m, m, heads, dim, vdim, 16, 1.0,
                              sinks=hip.Tensor.from_numpy(sink)).numpy().reshape(m, heads, vdim)
        assert np.all(np.isfinite(got)) and np.max(np.abs(got - want)) <= 1e-5


def gla_case(hip, m, heads, dim, vdim, rank, tau, bias, state=None, seed=0):
    rng = np.random.default_rng([m, heads, dim, vdim, rank, seed])
    cols = {"q": heads * dim, "k": heads * dim, "v": heads * vdim, "gate": heads * vdim, "low": rank}
    x = {n: rng.normal(0, 1, (m, c)).astype(np.float32) for n, c in cols.items()}
    a2 = rng.normal(0, rank ** -0.5, (heads * dim, rank)).astype(np.float32)
    bits = padded_bits(a2)
    b = rng.uniform(*bias, heads * dim).astype(np.float32)
    norm = rng.uniform(0.5, 1.5, vdim).astype(np.float32)
    sp = -(-vdim // 4) * 4
    if state is None:
        state = rng.normal(0, 1, (heads, dim, vdim)).astype(np.float32)
    st = np.zeros((heads, dim, sp), np.float32)
    st[..., :vdim] = state
    f = {n: v.astype(np.float64) for n, v in x.items()}
    log_a = ref.log_sigmoid(f["low"] @ from_bfloat16(bits)[:, :rank].astype(np.float64).T + b) / tau
    o, s = ref.gla_recurrence(f["q"].reshape(m, heads, dim) * dim ** -0.5, f["k"].reshape(m, heads, dim),
                              f["v"].reshape(m, heads, vdim), log_a.reshape(m, heads, dim), state.astype(np.float64))
    gated = (ref.rms_norm(o, norm, 1e-5) * ref.silu(f["gate"]).reshape(o.shape)).reshape(m, -1)
    ld = sum(cols.values())
    joined = hip.Tensor.from_numpy(np.concatenate(list(x.values()), axis=1))

    class At:  # a column of the joined buffer
        def __init__(self, first):
            self.ptr = joined.ptr + 4 * first
    first = np.cumsum([0] + list(cols.values()))
    at = {n: At(int(c)) for n, c in zip(cols, first)}
    dev_state = hip.Tensor.from_numpy(st)

    def run(rows_form, out_dtype=DT_F32):
        return hip.gla(at["q"], at["k"], at["v"], at["gate"], at["low"], bf16_tensor(hip, bits), hip.Tensor.from_numpy(b),
                       hip.Tensor.from_numpy(norm) if rows_form else None, dev_state, m, heads, dim, vdim, rank, ld, dim ** -0.5, tau,
                       1e-5, out_dtype)
    return run, dev_state, joined, o, gated, s


@pytest.mark.parametrize("m", [1, 2, 15, 16, 17, 63, 64, 65, 128, 200])
@pytest.mark.parametrize("heads,dim,vdim,rank,tau", [(2, 52, 36, 12, 5.0), (1, 1, 1, 1, 1.0), (3, 70, 100, 5, 2.0), (2, 130, 256, 9, 1.0)])
def test_gla_rows(hip, heads, dim, vdim, rank, tau, m):
    """The chunked form from a given state: outputs and the state it leaves."""
    run, state, _keep, _, gated, s = gla_case(hip, m, heads, dim, vdim, rank, tau, (-1.0, 4.0))
    assert rel_l2(run(True).numpy(), gated) <= 1e-5
    assert rel_l2(state.numpy()[..., :vdim], s) <= 2e-6


@pytest.mark.parametrize("bias", [(-40.0, -20.0), (-300.0, 8.0), (9.0, 12.0)])
def test_gla_rows_extreme_decays(hip, bias):
    run, state, _keep, _, gated, s = gla_case(hip, 150, 2, 40, 24, 6, 1.0, bias)
    assert rel_l2(run(True).numpy(), gated) <= 1e-5
    assert rel_l2(state.numpy()[..., :24], s) <= 2e-6


@pytest.mark.parametrize("heads,dim,vdim,rank", [(2, 52, 36, 12), (1, 1, 1, 1), (3, 65, 33, 5), (2, 129, 100, 9), (1, 512, 40, 64), (2, 200, 256, 3)])
def test_gla_step(hip, heads, dim, vdim, rank):
    run, state, _keep, o, _, s = gla_case(hip, 1, heads, dim, vdim, rank, 3.0, (-1.0, 4.0))
    assert rel_l2(run(False).numpy(), o.reshape(1, -1)) <= 2e-6
    assert rel_l2(state.numpy()[..., :vdim], s) <= 1e-6


def test_gla_bfloat16_output_only_rounds_the_result(hip):
    run, _, _keep, _, gated, _ = gla_case(hip, 80, 2, 44, 32, 11, 6.0, (-1.0, 4.0))
    assert rel_l2(bf16_values(hip, run(True, DT_BF16)), gated) <= 3e-3
