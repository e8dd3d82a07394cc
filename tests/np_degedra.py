"""A plain numpy restatement of the Degedra decoder's mechanisms, one function per mechanism, float64
throughout unless a caller passes another type; the yardstick of the device tests.  Nothing here is
chunked, cached or fused: a recurrence is a loop over positions, attention a full score matrix.

    x += norm(mixer(x)),  x += norm(ff(x))            only what a sublayer returns is normalised
    mixer = a . window_attention(x) + b . state_space(x)
    attention: query heads share key/value heads; q and k are normalised as whole projections and rotated,
               the values are the projected keys themselves
    state space: S_t = exp(-exp(A) dt_t) S_(t-1) + dt_t B_t x_t^T,  y_t = S_t^T C_t + D x_t, inputs behind a
               short causal convolution, y silu(z) normalised in equal parts
"""
from __future__ import annotations

import numpy as np


def rms_norm(x, w, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def silu(z):
    return z * np.exp(-np.logaddexp(0.0, -z))


def softplus(z):
    return np.logaddexp(0.0, z)


def rotate_half(x, positions, dims, base):
    """x [T, H, D]: of the first `dims` entries of a head, entry i and entry i + dims / 2 turn by p base^(-2 i / dims)."""
    half = dims // 2
    angle = np.asarray(positions, np.float64)[:, None] * np.power(float(base), -2.0 * np.arange(half) / dims)[None, :]
    c, s = np.cos(angle)[:, None, :], np.sin(angle)[:, None, :]
    u, v = x[..., :half], x[..., half:dims]
    return np.concatenate([u * c - v * s, v * c + u * s, x[..., dims:]], axis=-1)


def window_softmax(q, k, v, scale, window):
    """q [T, H, D], k [T, G, D], v [T, G, E] -> [T, H, E]; query head h reads key head h // (H / G); causal, the
    last `window` positions."""
    t, heads = q.shape[:2]
    share = heads // k.shape[1]
    i, j = np.arange(t)[:, None], np.arange(t)[None, :]
    seen = (j <= i) & (i - j < window)
    out = np.empty((t, heads, v.shape[2]), q.dtype)
    for h in range(heads):
        s = np.where(seen, q[:, h] @ k[:, h // share].T * scale, -np.inf)
        e = np.exp(s - s.max(axis=-1, keepdims=True))
        out[:, h] = e / e.sum(axis=-1, keepdims=True) @ v[:, h // share]
    return out


def grouped_attention(h, w, cfg, eps):
    heads, groups, dim = cfg["heads"], cfg["kv_heads"], cfg["dim"]
    t = h.shape[0]
    k_raw = h @ w["k"].T
    q = rms_norm(h @ w["q"].T, w["q.norm"], eps).reshape(t, heads, dim)
    k = rms_norm(k_raw, w["k.norm"], eps).reshape(t, groups, dim)
    rot, at = cfg["rot"], np.arange(t)
    o = window_softmax(rotate_half(q, at, rot["dims"], rot["base"]), rotate_half(k, at, rot["dims"], rot["base"]),
                       k_raw.reshape(t, groups, dim), cfg["scale"], cfg["mask"]["size"])
    return o.reshape(t, -1) @ w["o"].T


def causal_conv(x, w, b):
    """x [T, C], w [C, taps]: per channel, the last column meets the current token, zeros before the start."""
    taps = w.shape[1]
    padded = np.concatenate([np.zeros((taps - 1, x.shape[1]), x.dtype), x])
    return sum(padded[i:i + x.shape[0]] * w[:, i] for i in range(taps)) + b


def ssm_recurrence(x, b, c, log_decay, dt, state=None):
    """x [T, H, V], b, c [T, H, N], log_decay, dt [T, H]; returns (S_t^T C_t [T, H, V], final state [H, N, V])."""
    t, heads, n = b.shape
    s = np.zeros((heads, n, x.shape[2]), x.dtype) if state is None else state.copy()
    out = np.zeros(x.shape, x.dtype)
    for i in range(t):
        s = np.exp(log_decay[i])[:, None, None] * s + (dt[i][:, None] * b[i])[:, :, None] * x[i][:, None, :]
        out[i] = np.einsum("hnv,hn->hv", s, c[i])
    return out, s


def gated_group_norm(y, z, w, parts, eps):
    """y silu(z), every one of `parts` equal parts over its own root mean square, times w."""
    g = (y * silu(z)).reshape(y.shape[0], parts, -1)
    return rms_norm(g, 1.0, eps).reshape(y.shape) * w


def state_space(h, w, cfg, eps):
    heads, vdim, n, groups = cfg["heads"], cfg["vdim"], cfg["state"], cfg["groups"]
    t, inner = h.shape[0], heads * vdim
    p = h @ w["in"].T
    z, xbc, dt = p[:, :inner], p[:, inner:2 * inner + 2 * groups * n], p[:, 2 * inner + 2 * groups * n:]
    xbc = silu(causal_conv(xbc, w["conv"], w["conv.b"]))
    x = xbc[:, :inner].reshape(t, heads, vdim)
    spread = np.arange(heads) // (heads // groups)
    b = xbc[:, inner:inner + groups * n].reshape(t, groups, n)[:, spread]
    c = xbc[:, inner + groups * n:].reshape(t, groups, n)[:, spread]
    dt = softplus(dt + w["dt_bias"])
    y, _ = ssm_recurrence(x, b, c, -np.exp(w["A_log"]) * dt, dt)
    y = (y + w["D"][:, None] * x).reshape(t, inner)
    return gated_group_norm(y, p[:, :inner], w["norm"], cfg["norm_groups"], eps) @ w["o"].T


def parallel(h, w, cfg, eps):
    def side(name):
        return {k[len(name) + 1:]: v for k, v in w.items() if k.startswith(name + ".")}
    return cfg["left_scale"] * grouped_attention(h, side("left"), cfg["left"], eps) + \
        cfg["right_scale"] * state_space(h, side("right"), cfg["right"], eps)


def gated_ff(h, w):
    return (silu(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


def owner(layers, i):
    """The layer whose tensors layer i uses."""
    while layers[i].get("weights_of") is not None:
        i = layers[i]["weights_of"]
    return i


class NumpyDegedra:
    """config: the model's dict; weights: {tensor name: array}."""

    def __init__(self, config, weights):
        self.config = config
        self.w = {k: np.asarray(v, np.float64) for k, v in weights.items()}

    def _sub(self, prefix):
        return {k[len(prefix):]: v for k, v in self.w.items() if k.startswith(prefix)}

    def forward(self, tokens, trace=None):
        """Logits [T, vocab] of the whole sequence; `trace` (a list) receives the residual after every layer."""
        cfg, w = self.config, self.w
        eps = cfg["norm"]["eps"]
        x = w["embed"][np.asarray(tokens, np.int64)]
        for i, layer in enumerate(cfg["layers"]):
            p = f"l{owner(cfg['layers'], i)}."
            x = x + rms_norm(parallel(x, self._sub(p + "mix."), layer["mixer"], eps), w[p + "norm1"], eps)
            if layer.get("mlp") is not None:
                x = x + rms_norm(gated_ff(x, self._sub(p + "mlp.")), w[p + "norm2"], eps)
            if trace is not None:
                trace.append(x.copy())
        logits = rms_norm(x, w["final.norm"], eps) @ w["head"].T
        cap = cfg["logit_softcap"]
        return cap * np.tanh(logits / cap)

    def greedy(self, prompt, n_new):
        """Greedy continuation by running the whole sequence anew for every token; also the margins
        between the best and second-best logit, so that a caller can tell a near-tie from a fault."""
        toks, out, margins = list(prompt), [], []
        for _ in range(n_new):
            row = self.forward(toks)[-1]
            top = np.sort(row)[-2:]
            out.append(int(np.argmax(row)))
            margins.append(float(top[1] - top[0]))
            toks.append(out[-1])
        return out, margins
