"""Small Kulurax models for the tests: configurations, seeded weights, a safetensors writer."""
from __future__ import annotations

import json
import os
import struct

import numpy as np

from litenn_amd.synth import kulurax_tensor_shapes
from litenn_amd.model import from_bfloat16, to_bfloat16


def attention(heads=3, dim=24, vdim=40, kv_rank=56, q_rank=72, window=9, scale=0.3, mlp=None):
    return {"type": "latent_attention", "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank, "scale": scale,
                      "mask": {"size": window}}}


def linear_attention(heads=2, dim=20, vdim=12, tau=8.0, mlp=None):
    return {"type": "gla", "mlp": mlp, "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}}


def mlp(ff=88, limit=0.75):
    return {"kind": "dense", "ff": ff, "limit": limit}


def config(layers, vocab=131, width=88, eps=3e-5):
    return {"architecture": "Kulurax", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


def random_weights(cfg, seed, decay_rank=7, decay_bias=(-1.0, 4.0), gain=1.0, edit=None):
    """{name: bfloat16 bits}.  Linears have entries of root mean square gain / sqrt(inputs); norms lie around
    one; decay biases are spread over `decay_bias`; edit(weights) may change the Float32 values first."""
    rng = np.random.default_rng(seed)
    w = {}
    for name, shape in kulurax_tensor_shapes(cfg, decay_rank).items():
        if name.endswith("a2.b"):
            v = rng.uniform(*decay_bias, shape)
        elif name.endswith("sink"):
            v = rng.normal(0.5, 1.0, shape)
        elif len(shape) == 1:
            v = rng.uniform(0.5, 1.5, shape)
        elif name == "embed":
            v = rng.normal(0.0, 1.0, shape)
        else:
            v = rng.normal(0.0, gain / np.sqrt(shape[1]), shape)
        w[name] = v.astype(np.float32)
    if edit:
        edit(w)
    return {k: to_bfloat16(v) for k, v in w.items()}


def as_floats(weights):
    return {k: from_bfloat16(v) for k, v in weights.items()}


def tokens(cfg, n, seed):
    return np.random.default_rng([seed, 77]).integers(0, cfg["vocab"], n).astype(np.int32)


def write_folder(path, cfg, weights):
    """config.json and model.safetensors under `path`."""
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    header, blob = {}, b""
    for name, bits in weights.items():
        raw = np.ascontiguousarray(bits, np.uint16).tobytes()
        header[name] = {"dtype": "BF16", "shape": list(bits.shape), "data_offsets": [len(blob), len(blob) + len(raw)]}
        blob += raw
    head = json.dumps(header).encode()
    head += b" " * (-len(head) % 8)
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(head)) + head + blob)
    return str(path)


def row_errors(got, want):
    """Root-mean-square difference of every row of logits, means taken off, over the spread of all logits."""
    d = np.asarray(got, np.float64) - want
    d -= d.mean(axis=-1, keepdims=True)
    spread = want - want.mean(axis=-1, keepdims=True)
    return np.sqrt((d * d).mean(axis=-1)) / np.sqrt((spread * spread).mean())


def error(got, want):
    """The largest of them."""
    return float(row_errors(got, want).max())
