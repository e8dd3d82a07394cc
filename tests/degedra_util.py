"""Small Degedra models for the tests: configurations and seeded weights."""
from __future__ import annotations

import numpy as np

from kulurax_util import as_floats, error, row_errors, tokens, write_folder  # noqa: F401  (the models share them)
from litenn_amd import synth
from litenn_amd.model import to_bfloat16


def attention(heads=6, kv_heads=2, dim=24, window=9, scale=0.3, rot_dims=16, rot_base=700.0):
    return synth.degedra_attention(heads, kv_heads, dim, window, scale, rot_dims, rot_base)


def state_space(heads=6, vdim=20, state=12, groups=3, norm_groups=2, conv=4):
    return synth.degedra_state_space(heads, vdim, state, groups, norm_groups, conv)


def layer(left=None, right=None, ff=None, left_scale=0.8, right_scale=1.3):
    return synth.degedra_layer(left or attention(), right or state_space(), ff, left_scale, right_scale)


def again(layers, of):
    """A layer that uses the weights of layer `of`."""
    return {**layers[of], "weights_of": of}


def config(layers, vocab=131, width=88, eps=3e-5, softcap=20.0):
    return {"architecture": "Degedra", "vocab": vocab, "width": width, "norm": {"eps": eps}, "logit_softcap": softcap,
            "layers": layers}


def random_weights(cfg, seed, rates=(-3.0, 1.0), steps=(-4.0, 1.0), edit=None):
    """{name: bfloat16 bits}.  Linears have entries of root mean square 1 / sqrt(inputs), a convolution's taps of
    1 / sqrt(taps); norms lie around one; 'A_log' is spread over `rates`, 'dt_bias' over `steps`; edit(weights)
    may change the Float32 values first."""
    rng = np.random.default_rng(seed)
    w = {}
    for name, shape in synth.degedra_tensor_shapes(cfg).items():
        leaf = name.rsplit(".", 1)[-1]
        if leaf == "A_log":
            v = rng.uniform(*rates, shape)
        elif leaf == "dt_bias":
            v = rng.uniform(*steps, shape)
        elif leaf == "b":
            v = rng.normal(0.0, 0.3, shape)
        elif leaf == "D":
            v = rng.normal(0.0, 1.0, shape)
        elif len(shape) == 1:
            v = rng.uniform(0.5, 1.5, shape)
        elif name == "embed":
            v = rng.normal(0.0, 1.0, shape)
        else:
            v = rng.normal(0.0, 1.0 / np.sqrt(shape[1]), shape)
        w[name] = v.astype(np.float32)
    if edit:
        edit(w)
    return {k: to_bfloat16(v) for k, v in w.items()}
