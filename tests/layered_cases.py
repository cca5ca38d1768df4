"""Small random models described layer by layer, for the tests: configurations, bf16 weights, comparison with the oracle."""
import json
import os

import numpy as np


def attn(heads=3, dim=24, rot=8, vdim=20, rank=40, scale=None, base=10000.0, dims=None, scaling=None, ff=72, rotate=True):
    mx = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "scale": scale or (dim + rot) ** -0.5}
    if rotate:
        mx["rot"] = {"base": base, "dims": rot if dims is None else dims}
        if scaling:
            mx["rot"]["scaling"] = scaling
    return {"type": "latent_attention", "mixer": mx, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def mem(heads=2, dim=20, vdim=28, cap=10.0, ff=0):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}, "mlp": {"kind": "dense", "ff": ff} if ff else None}


YARN = {"factor": 4.0, "original": 64, "fast": 8.0, "slow": 1.0}


def config(layers, width=88, vocab=150, eps=1e-5, mult=0.4, bigram=(61, 13, 5)):
    c = {"architecture": "Zamelix", "width": width, "vocab": vocab, "norm": {"eps": eps}, "residual_mult": mult, "layers": layers}
    if bigram:
        c["embedding"] = {"bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))}
    return c


def bf16(x):
    """Round to bf16 (nearest even), as f32."""
    u = np.ascontiguousarray(x, np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) & 0xFFFF0000).view(np.float32)


class Weights(dict):
    """name -> f32 array of bf16 values; `get(name, shape)` is what the loader asks a source for."""

    def __init__(self, parsed, seed=0):
        super().__init__()
        rng = np.random.default_rng(seed)
        for name, shape in parsed.tensor_shapes():
            if "norm" in name.split(".")[-1] or name.endswith(("norm1", "norm2")):
                v = 1.0 + 0.2 * rng.standard_normal(shape)
            elif name.endswith(".f.b"):
                v = 3.0 + rng.standard_normal(shape)          # a memory that lasts
            elif len(shape) == 1:
                v = 0.5 * rng.standard_normal(shape)
            elif name in ("embed", "bigram"):
                v = rng.standard_normal(shape)
            else:
                v = rng.standard_normal(shape) / np.sqrt(shape[1])
            self[name] = bf16(v)

    def get(self, name, shape=None):
        if shape is None:
            return super().get(name)
        v = self[name]
        assert tuple(v.shape) == tuple(shape), name
        return 30, (np.ascontiguousarray(v).view(np.uint32) >> 16).astype(np.uint16).reshape(-1)


def write_dir(path, cfg, weights):
    """config.json + model.safetensors as a checkpoint folder holds them."""
    head, blobs, at = {}, [], 0
    for name, v in weights.items():
        raw = (np.ascontiguousarray(v).view(np.uint32) >> 16).astype("<u2").tobytes()
        head[name] = {"dtype": "BF16", "shape": list(v.shape), "data_offsets": [at, at + len(raw)]}
        at += len(raw)
        blobs.append(raw)
    h = json.dumps(head).encode()
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(len(h).to_bytes(8, "little") + h + b"".join(blobs))
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)


def tokens(n, vocab, seed=1):
    return np.random.default_rng(seed).integers(0, vocab, n).tolist()


def row_error(got, want):
    """Per row: rms over the vocabulary of the difference (mean taken off), over the rms of the expected logits."""
    d = np.asarray(got, np.float64) - want
    d -= d.mean(-1, keepdims=True)
    return np.sqrt((d * d).mean(-1)) / np.sqrt((want * want).mean())
