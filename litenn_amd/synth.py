"""Seeded synthetic GGUF-layout tensors and LLaMA-shape models.

The laws follow the benchmark configurations: every fp16 scale is
|N(0,1)| * 0.02, every packed quant byte is uniform, activations are N(0,1).
The tensors of a decoder model (llama_tensors) draw their scales with a random
sign, as a quantiser produces them (ggml's Q4_0 scale is the extreme value
/ -8, of either sign): with positive scales only, uniform codes give every
matrix a common offset (Q4_0: -0.5 d per weight) whose rank-one part outweighs
the random part, the hidden state collapses onto the all-ones direction after
a few blocks and greedy decoding repeats one token.  Their spread is
N(0,1) / (CODE_RMS[format] * sqrt(k)), so that a dequantised [n, k] matrix has
entries of root mean square 1/sqrt(k) like an initialised linear layer
whatever its format (0.02 would make a Q4_K weight about 250 times that, the
attention scores of such a model saturate the softmax, and the smallest
rounding difference then picks another key).  The scales of the K-quant
formats land in the fp16 subnormal range, where a trained model's lie too.
Norm weights are drawn from [0.5, 1.5] so that a dropped or misplaced norm
weight changes the result.
Payloads are produced in exactly the byte layout a .gguf file stores
(row-major [n, k/block] blocks), i.e. what LiteNN's importer keeps as a UInt8
variable (tools/gguf/GGUFImporter.cpp:478-491).
"""
from __future__ import annotations

import numpy as np

from .formats import Q4_0, Q4_1, Q5_0, Q5_1, Q8_0, Q2_K, Q3_K, Q4_K, Q5_K, Q6_K, F32, block_layout, row_bytes


def _rng(seed, *stream) -> np.random.Generator:
    return np.random.default_rng([int(seed), *[int(s) for s in stream]])


def _uniform_bytes(rng: np.random.Generator, shape) -> np.ndarray:
    n = int(np.prod(shape))
    return np.frombuffer(rng.bytes(n), np.uint8).reshape(shape)


def _scales_f16(rng: np.random.Generator, shape, signed: bool = False, sigma: float = 0.02) -> np.ndarray:
    d = rng.standard_normal(shape, dtype=np.float32) * np.float32(sigma)
    if not signed:
        d = np.abs(d)
    return d.astype(np.float16).view(np.uint16)


def _put_u16(blocks: np.ndarray, offset: int, values: np.ndarray) -> None:
    blocks[..., offset] = (values & 0xFF).astype(np.uint8)
    blocks[..., offset + 1] = (values >> 8).astype(np.uint8)


def quant_weights(fmt: int, n: int, k: int, seed, *stream, signed_scales: bool = False,
                  scale_sigma: float = 0.02) -> np.ndarray:
    """Random payload of an [n, k] tensor in block format `fmt`: uint8 [n, row_bytes].  Scales are
    |N(0,1)| * scale_sigma, or N(0,1) * scale_sigma with signed_scales."""
    elems, nbytes = block_layout(fmt)
    if k % elems:
        raise ValueError(f"k={k} is not a multiple of the block size {elems}")
    rng = _rng(seed, *stream)
    nb = k // elems
    blocks = np.empty((n, nb, nbytes), np.uint8)
    if fmt == Q8_0:
        _put_u16(blocks, 0, _scales_f16(rng, (n, nb), signed_scales, scale_sigma))
        q = _uniform_bytes(rng, (n, nb, 32)).view(np.int8)
        q = np.where(q == -128, np.int8(-127), q)  # uniform on [-127, 127] up to one remapped code
        blocks[..., 2:] = q.view(np.uint8)
    elif fmt == Q4_0:
        _put_u16(blocks, 0, _scales_f16(rng, (n, nb), signed_scales, scale_sigma))
        blocks[..., 2:] = _uniform_bytes(rng, (n, nb, 16))
    elif fmt == Q4_K:
        _put_u16(blocks, 0, _scales_f16(rng, (n, nb), signed_scales, scale_sigma))
        _put_u16(blocks, 2, _scales_f16(rng, (n, nb), signed_scales, scale_sigma))
        blocks[..., 4:] = _uniform_bytes(rng, (n, nb, 140))
    elif fmt == Q6_K:
        blocks[..., :208] = _uniform_bytes(rng, (n, nb, 208))
        _put_u16(blocks, 208, _scales_f16(rng, (n, nb), signed_scales, scale_sigma))
    elif fmt in (Q4_1, Q5_0, Q5_1, Q5_K):
        # fp16 d [, fp16 m / dmin] first, everything after them uniform bytes
        heads = {Q4_1: 2, Q5_0: 1, Q5_1: 2, Q5_K: 2}[fmt]
        for h in range(heads):
            _put_u16(blocks, 2 * h, _scales_f16(rng, (n, nb), signed_scales, scale_sigma))
        blocks[..., 2 * heads:] = _uniform_bytes(rng, (n, nb, nbytes - 2 * heads))
    elif fmt == Q2_K:
        blocks[..., :80] = _uniform_bytes(rng, (n, nb, 80))
        _put_u16(blocks, 80, _scales_f16(rng, (n, nb), signed_scales, scale_sigma))
        _put_u16(blocks, 82, _scales_f16(rng, (n, nb), signed_scales, scale_sigma))
    elif fmt == Q3_K:
        blocks[..., :108] = _uniform_bytes(rng, (n, nb, 108))
        _put_u16(blocks, 108, _scales_f16(rng, (n, nb), signed_scales, scale_sigma))
    else:
        raise ValueError(f"unsupported format {fmt}")
    return blocks.reshape(n, nb * nbytes)


def activations(m: int, k: int, seed, *stream) -> np.ndarray:
    return _rng(seed, *stream).standard_normal((m, k), dtype=np.float32)


class LLaMAConfig:
    """Shape of a LLaMA-family decoder (tools/gguf/GGUFImporter.cpp:505-642 field names)."""

    def __init__(self, name, block_count, embedding_length, head_count, head_count_kv, feed_forward_length,
                 vocab, context_length, rms_eps=float(np.float32(1e-5)), rope_freq_base=1e4, formats=None,
                 rope_freq_scale=1.0, rope_dimension_count=0):
        self.name = name
        self.block_count = block_count
        self.embedding_length = embedding_length
        self.head_count = head_count
        self.head_count_kv = head_count_kv
        self.feed_forward_length = feed_forward_length
        self.vocab = vocab
        self.context_length = context_length
        self.rms_eps = rms_eps
        self.rope_freq_base = rope_freq_base
        self.rope_freq_scale = rope_freq_scale            # 1 / factor of linear scaling
        self.rope_dimension_count = rope_dimension_count  # 0: the whole head
        # tensor-kind -> block format
        self.formats = formats or {}

    @property
    def head_dim(self) -> int:
        return self.embedding_length // self.head_count

    def fmt(self, kind: str) -> int:
        return self.formats.get(kind, self.formats.get("default", Q4_0))

    def tensor_shapes(self):
        d, hd = self.embedding_length, self.head_dim
        qw, kvw, ff = self.head_count * hd, self.head_count_kv * hd, self.feed_forward_length
        return {
            "attn_q": (qw, d), "attn_k": (kvw, d), "attn_v": (kvw, d), "attn_output": (d, qw),
            "ffn_gate": (ff, d), "ffn_up": (ff, d), "ffn_down": (d, ff),
            "token_embd": (self.vocab, d), "output": (self.vocab, d),
        }

    def matmul_weight_bytes_per_token(self) -> int:
        shapes = self.tensor_shapes()
        per_layer = sum(shapes[k][0] * row_bytes(self.fmt(k), shapes[k][1])
                        for k in ("attn_q", "attn_k", "attn_v", "attn_output", "ffn_gate", "ffn_up", "ffn_down"))
        out = shapes["output"][0] * row_bytes(self.fmt("output"), shapes["output"][1])
        return per_layer * self.block_count + out


def llama_7b_q4_0(context_length: int = 512) -> LLaMAConfig:
    return LLaMAConfig("llama-7b-shape-q4_0", 32, 4096, 32, 32, 11008, 32000, context_length,
                       rope_freq_base=1e4, formats={"default": Q4_0})


def llama_8b_gqa_mixed(context_length: int = 4096) -> LLaMAConfig:
    return LLaMAConfig("llama-8b-gqa-shape-q4_k-q6_k", 32, 4096, 32, 8, 14336, 128256, context_length,
                       rope_freq_base=5e5,
                       formats={"default": Q4_K, "attn_v": Q6_K, "ffn_down": Q6_K, "output": Q6_K})


def tiny_llama(fmt: int = Q4_0, block_count: int = 2, d_model: int = 256, heads: int = 4, kv_heads: int = 2,
               ff: int = 512, vocab: int = 320, context_length: int = 64, formats=None) -> LLaMAConfig:
    return LLaMAConfig("tiny", block_count, d_model, heads, kv_heads, ff, vocab, context_length,
                       formats=formats or {"default": fmt})


TENSOR_KINDS = ("attn_q", "attn_k", "attn_v", "attn_output", "ffn_gate", "ffn_up", "ffn_down")


# root mean square of a dequantised weight at unit scales and uniform code bytes
CODE_RMS = {Q4_0: 4.64, Q4_1: 8.9, Q5_0: 9.3, Q5_1: 18.2, Q8_0: 74.0, Q2_K: 18.7, Q3_K: 43.5, Q4_K: 325.0, Q5_K: 670.0,
            Q6_K: 1355.0}


def model_weights(fmt: int, n: int, k: int, seed, *stream) -> np.ndarray:
    """Payload of a decoder matrix: signed scales sized so that its entries have rms 1/sqrt(k)."""
    return quant_weights(fmt, n, k, seed, *stream, signed_scales=True,
                         scale_sigma=1.0 / (CODE_RMS[fmt] * float(np.sqrt(k))))


def norm_weights(d: int, seed, *stream) -> np.ndarray:
    """f32 [d], uniform on [0.5, 1.5]."""
    return (_rng(seed, *stream).random(d, dtype=np.float32) + np.float32(0.5)).astype(np.float32)


def llama_tensors(cfg: LLaMAConfig, seed: int):
    """Yield (kind, layer, fmt, payload, n, k); matrices follow model_weights, norm weights are f32
    drawn from [0.5, 1.5]."""
    shapes = cfg.tensor_shapes()
    d = cfg.embedding_length
    for kind_id, kind in enumerate(("token_embd", "output")):
        n, k = shapes[kind]
        f = cfg.fmt(kind)
        yield kind, -1, f, model_weights(f, n, k, seed, 1000 + kind_id), n, k
    yield "output_norm", -1, F32, norm_weights(d, seed, 2000), 1, d
    for layer in range(cfg.block_count):
        for kind_id, kind in enumerate(TENSOR_KINDS):
            n, k = shapes[kind]
            f = cfg.fmt(kind)
            yield kind, layer, f, model_weights(f, n, k, seed, layer, kind_id), n, k
        yield "attn_norm", layer, F32, norm_weights(d, seed, 2001, layer), 1, d
        yield "ffn_norm", layer, F32, norm_weights(d, seed, 2002, layer), 1, d


def prompt_tokens(cfg: LLaMAConfig, n: int, seed: int) -> np.ndarray:
    return _rng(seed, 777).integers(0, cfg.vocab, size=n, dtype=np.int32)


# ---- layered decoders --------------------------------------------------------------------------------

def kulurax_config(width: int, ff: int, layers: int, heads: int, vocab: int, window: int, kv_rank: int, q_rank: int,
                   dim: int = 128, gla_heads: int = 16, gla_dim: int = 128, gla_vdim: int = 256) -> dict:
    """A Kulurax decoder in which linear and latent attention alternate, every layer with a feed-forward."""
    mlp = {"kind": "dense", "ff": ff, "limit": 7.0}
    linear = {"type": "gla", "mlp": mlp, "mixer": {"heads": gla_heads, "dim": gla_dim, "vdim": gla_vdim, "tau": 16.0}}
    latent = {"type": "latent_attention", "mlp": mlp,
              "mixer": {"heads": heads, "dim": dim, "vdim": dim, "kv_rank": kv_rank, "q_rank": q_rank,
                        "scale": dim ** -0.5, "mask": {"size": window}}}
    return {"architecture": "Kulurax", "vocab": vocab, "width": width, "norm": {"eps": 1e-5},
            "layers": [linear if i % 2 == 0 else latent for i in range(layers)]}


def kulurax_tensor_shapes(cfg: dict, decay_rank: int = 16) -> dict:
    w = cfg["width"]
    out = {"embed": (cfg["vocab"], w), "final.norm": (w,)}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        keys, values = m["heads"] * m["dim"], m["heads"] * m["vdim"]
        out[p + "norm1"] = out[p + "norm1b"] = (w,)
        if layer["type"] == "gla":
            parts = {"q": (keys, w), "k": (keys, w), "v": (values, w), "g": (values, w), "o": (w, values),
                     "norm": (m["vdim"],), "a1": (decay_rank, w), "a2": (keys, decay_rank), "a2.b": (keys,)}
        else:
            parts = {"dq": (m["q_rank"], w), "dq.norm": (m["q_rank"],), "uq": (keys, m["q_rank"]),
                     "dkv": (m["kv_rank"], w), "dkv.norm": (m["kv_rank"],), "uk": (keys, m["kv_rank"]),
                     "uv": (values, m["kv_rank"]), "sink": (m["heads"],), "g": (values, w), "o": (w, values)}
        out.update({p + "mix." + k: s for k, s in parts.items()})
        if layer["mlp"]:
            ff = layer["mlp"]["ff"]
            out[p + "norm2"] = out[p + "norm2b"] = (w,)
            out.update({p + "mlp.gate": (ff, w), p + "mlp.up": (ff, w), p + "mlp.down": (w, ff)})
    return out


def degedra_attention(heads: int, kv_heads: int, dim: int, window: int, scale: float | None = None, rot_dims: int | None = None,
                      rot_base: float = 10000.0) -> dict:
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5 if scale is None else scale,
            "mask": {"size": window}, "rot": {"dims": dim if rot_dims is None else rot_dims, "base": rot_base}}


def degedra_state_space(heads: int, vdim: int, state: int, groups: int = 1, norm_groups: int = 1, conv: int = 4) -> dict:
    return {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "norm_groups": norm_groups, "conv": conv}


def degedra_layer(left: dict, right: dict, ff: int | None, left_scale: float = 1.0, right_scale: float = 1.0) -> dict:
    return {"type": "parallel", "mlp": None if ff is None else {"kind": "dense", "ff": ff},
            "mixer": {"left": left, "right": right, "left_scale": left_scale, "right_scale": right_scale}}


def degedra_config(width: int, ff: int, layers: int, heads: int, kv_heads: int, vocab: int, window: int, dim: int = 128,
                   ssm_heads: int = 64, ssm_vdim: int = 64, state: int = 128, groups: int = 2) -> dict:
    """A Degedra decoder of equal layers, every one with a feed-forward."""
    layer = degedra_layer(degedra_attention(heads, kv_heads, dim, window),
                          degedra_state_space(ssm_heads, ssm_vdim, state, groups, groups), ff)
    return {"architecture": "Degedra", "vocab": vocab, "width": width, "norm": {"eps": 1e-5}, "logit_softcap": 30.0,
            "layers": [layer] * layers}


def degedra_tensor_shapes(cfg: dict) -> dict:
    w = cfg["width"]
    out = {"embed": (cfg["vocab"], w), "head": (cfg["vocab"], w), "final.norm": (w,)}
    for i, layer in enumerate(cfg["layers"]):
        if layer.get("weights_of") is not None:
            continue
        p, a, r = f"l{i}.", layer["mixer"]["left"], layer["mixer"]["right"]
        keys, cached, inner = a["heads"] * a["dim"], a["kv_heads"] * a["dim"], r["heads"] * r["vdim"]
        channels = inner + 2 * r["groups"] * r["state"]
        left = {"q": (keys, w), "k": (cached, w), "q.norm": (keys,), "k.norm": (cached,), "o": (w, keys)}
        right = {"in": (inner + channels + r["heads"], w), "conv": (channels, r["conv"]), "conv.b": (channels,),
                 "dt_bias": (r["heads"],), "A_log": (r["heads"],), "D": (r["heads"],), "norm": (inner,), "o": (w, inner)}
        out[p + "norm1"] = (w,)
        out.update({p + "mix.left." + k: s for k, s in left.items()})
        out.update({p + "mix.right." + k: s for k, s in right.items()})
        if layer["mlp"]:
            ff = layer["mlp"]["ff"]
            out[p + "norm2"] = (w,)
            out.update({p + "mlp.gate": (ff, w), p + "mlp.up": (ff, w), p + "mlp.down": (w, ff)})
    return out


TENSOR_SHAPES = {"Kulurax": kulurax_tensor_shapes, "Degedra": degedra_tensor_shapes}


def layered_large_tensors(cfg: dict, seed) -> dict:
    """bfloat16 bits for a large model: every matrix is a window into one pool of N(0, 1/64) values, so that
    gigabytes of weights take a second to make and little host memory."""
    rng = _rng(seed)
    shapes = TENSOR_SHAPES[cfg["architecture"]](cfg)
    size = max(int(np.prod(s)) for s in shapes.values()) + 65536
    pool = (rng.standard_normal(size, dtype=np.float32) * np.float32(1.0 / 64.0)).view(np.uint32)
    pool = ((pool + 0x8000) >> 16).astype(np.uint16)
    out = {}
    for name, s in shapes.items():
        n = int(np.prod(s))
        if len(s) == 1:
            out[name] = rng.uniform(0.5, 1.5, s).astype(np.float32)
        else:
            at = int(rng.integers(0, 65536))
            out[name] = pool[at:at + n].reshape(s)
    return out


def layered_decode_weight_bytes(cfg: dict) -> int:
    """Weight bytes a single-token step reads: every matrix once (an embedding table only where it is the head)."""
    shapes = TENSOR_SHAPES[cfg["architecture"]](cfg)
    return 2 * sum(int(np.prod(s)) for n, s in shapes.items() if len(s) == 2 and not (n == "embed" and "head" in shapes))


def window_pairs(rows: int, window: int) -> float:
    """Query-key pairs of `rows` tokens from an empty sequence."""
    return rows * (rows + 1) / 2 if rows <= window else window * (window + 1) / 2 + (rows - window) * window


def layered_prefill_flops(cfg: dict, rows: int) -> float:
    """Matrix-product operations of a prompt pass of `rows` tokens from an empty sequence: linears, window attention's
    visible scores and values, the recurrence (state update and read)."""
    shapes = TENSOR_SHAPES[cfg["architecture"]](cfg)
    total = sum(2.0 * rows * np.prod(s) for n, s in shapes.items() if len(s) == 2 and n not in ("embed", "head"))
    for layer in cfg["layers"]:
        m = layer["mixer"]
        if layer["type"] == "gla":
            total += 4.0 * rows * m["heads"] * m["dim"] * m["vdim"]
        elif layer["type"] == "parallel":
            r, m = m["right"], m["left"]
            total += 4.0 * rows * r["heads"] * r["state"] * r["vdim"]
        if "mask" in m:
            total += 2.0 * window_pairs(rows, m["mask"]["size"]) * m["heads"] * (m["dim"] + m["vdim"])
    return float(total + 2.0 * cfg["vocab"] * cfg["width"])
