"""A plain numpy restatement of the Kulurax decoder's mechanisms, one function per mechanism, float64
throughout unless a caller passes another type; the yardstick of the device tests.  Nothing here is
chunked, cached or fused: a recurrence is a loop over positions, attention a full score matrix.

    y = x + norm(mixer(norm(x)))                      each sublayer is normalised on both sides
    latent attention: c = norm(Wdkv h); per head  s_ij = scale * (Wuq cq)_i . (Wuk c)_j,
                      0 <= i - j < window,  weights exp(s_ij) / (exp(sink) + sum_j exp(s_ij))
    gated linear attention: S_t = diag(a_t) S_(t-1) + k_t v_t^T,  o_t = S_t^T q_t
"""
from __future__ import annotations

import json

import numpy as np


def rms_norm(x, w, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def sigmoid(z):
    return np.exp(-np.logaddexp(0.0, -z))


def log_sigmoid(z):
    return -np.logaddexp(0.0, -z)


def silu(z):
    return z * sigmoid(z)


def sinusoid(positions, width):
    """[len(positions), width]: sine on the even entries, cosine on the odd ones."""
    p = np.asarray(positions, np.float64)[:, None]
    j = np.arange(width)
    angle = p * np.power(10000.0, -2.0 * (j // 2) / width)[None, :]
    return np.where(j % 2 == 0, np.sin(angle), np.cos(angle))


def windowed_sink_attention(q, k, v, scale, window, sink):
    """q, k [T, H, D], v [T, H, E], sink [H] -> [T, H, E]; causal, the last `window` positions."""
    t = q.shape[0]
    i, j = np.arange(t)[:, None], np.arange(t)[None, :]
    seen = (j <= i) & (i - j < window)
    s = np.einsum("ihd,jhd->hij", q, k) * scale
    s = np.where(seen[None], s, -np.inf)
    top = np.maximum(s.max(axis=-1, keepdims=True), sink[:, None, None])
    e = np.exp(s - top)
    p = e / (e.sum(axis=-1, keepdims=True) + np.exp(sink[:, None, None] - top))
    return np.einsum("hij,jhe->ihe", p, v)


def latent_attention(h, w, cfg, eps):
    heads, dim, vdim = cfg["heads"], cfg["dim"], cfg["vdim"]
    t = h.shape[0]
    cq = rms_norm(h @ w["dq"].T, w["dq.norm"], eps)
    q = (cq @ w["uq"].T).reshape(t, heads, dim)
    c = rms_norm(h @ w["dkv"].T, w["dkv.norm"], eps)
    k = (c @ w["uk"].T).reshape(t, heads, dim)
    v = (c @ w["uv"].T).reshape(t, heads, vdim)
    o = windowed_sink_attention(q, k, v, cfg["scale"], cfg["mask"]["size"], w["sink"]).reshape(t, heads * vdim)
    return (o * sigmoid(h @ w["g"].T)) @ w["o"].T


def gla_recurrence(q, k, v, log_a, state=None):
    """q, k, log_a [T, H, D], v [T, H, E]; returns (o [T, H, E], final state [H, D, E])."""
    t, heads, dim = q.shape
    s = np.zeros((heads, dim, v.shape[2]), q.dtype) if state is None else state.copy()
    out = np.zeros(v.shape, q.dtype)
    for i in range(t):
        s = np.exp(log_a[i])[:, :, None] * s + k[i][:, :, None] * v[i][:, None, :]
        out[i] = np.einsum("hde,hd->he", s, q[i])
    return out, s


def gla_log_decay(h, w, tau):
    return log_sigmoid(h @ w["a1"].T @ w["a2"].T + w["a2.b"]) / tau


def gla(h, w, cfg, eps):
    heads, dim, vdim = cfg["heads"], cfg["dim"], cfg["vdim"]
    t = h.shape[0]
    q = (h @ w["q"].T).reshape(t, heads, dim) * dim ** -0.5
    k = (h @ w["k"].T).reshape(t, heads, dim)
    v = (h @ w["v"].T).reshape(t, heads, vdim)
    o, _ = gla_recurrence(q, k, v, gla_log_decay(h, w, cfg["tau"]).reshape(t, heads, dim))
    o = rms_norm(o, w["norm"], eps).reshape(t, heads * vdim)
    return (o * silu(h @ w["g"].T)) @ w["o"].T


MIXERS = {"latent_attention": latent_attention, "gla": gla}


def clamped_glu(h, w, limit):
    g = np.minimum(h @ w["gate"].T, limit)
    u = np.clip(h @ w["up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w["down"].T


class NumpyKulurax:
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
        tokens = np.asarray(tokens, np.int64)
        x = w["embed"][tokens] + sinusoid(np.arange(len(tokens)), cfg["width"])
        for i, layer in enumerate(cfg["layers"]):
            p = f"l{i}."
            y = MIXERS[layer["type"]](rms_norm(x, w[p + "norm1"], eps), self._sub(p + "mix."), layer["mixer"], eps)
            x = x + rms_norm(y, w[p + "norm1b"], eps)
            if layer.get("mlp") is not None:
                y = clamped_glu(rms_norm(x, w[p + "norm2"], eps), self._sub(p + "mlp."), layer["mlp"]["limit"])
                x = x + rms_norm(y, w[p + "norm2b"], eps)
            if trace is not None:
                trace.append(x.copy())
        return rms_norm(x, w["final.norm"], eps) @ w["embed"].T

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
