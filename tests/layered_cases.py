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


def tied(heads=6, kv_heads=2, dim=24, window=40, keep=3, scale=None, cap=20.0, mlp=None):
    """Attention whose values are its keys; window 0: no mask."""
    mx = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale or dim ** -0.5}
    if window:
        mx["mask"] = {"size": window, "keep_first": keep}
    if cap:
        mx["softcap"] = cap
    return {"type": "attention", "mixer": mx, "mlp": mlp}


def moe(experts=6, top=2, ff=40, shared=56):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}, "shared": {"ff": shared} if shared else None}


def sandwich(layers, width=88, vocab=150, eps=1e-5, taps=3):
    return {"architecture": "Pubopel", "width": width, "vocab": vocab, "norm": {"eps": eps}, "canon": {"taps": taps}, "layers": layers}


def rglru(width=96, blocks=3, taps=4, mlp=None):
    return {"type": "rglru", "mixer": {"width": width, "blocks": blocks, "conv": taps}, "mlp": mlp}


def gated(heads=6, kv_heads=2, dim=20, vdim=28, chunk=40, rot=8, base=10000.0, scale=None, mlp=None):
    """Attention with gated values; chunk 0: no chunks, rot 0: nothing is rotated."""
    mx = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale or dim ** -0.5}
    if chunk:
        mx["mask"] = {"size": chunk}
    if rot:
        mx["rot"] = {"base": base, "dims": rot}
    return {"type": "gated_attention", "mixer": mx, "mlp": mlp}


def gla(heads=3, dim=24, vdim=20, tau=16.0, rank=12, mlp=None):
    """rank is told by a tensor's shape, not by the configuration: the tests keep it beside the layer."""
    return {"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}, "mlp": mlp, "rank": rank}


def parallel(left=None, right=None, scales=(0.8, 1.3), mlp=None):
    left, right = left or gated(), right or gla()
    return {"type": "parallel", "mixer": {"left": left["mixer"], "right": right["mixer"], "left_scale": scales[0], "right_scale": scales[1]}, "mlp": mlp, "rank": right["rank"]}


def dense(ff=72):
    return {"kind": "dense", "ff": ff}


def grouped(experts=9, identity=3, top=3, ff=40, groups=(4, 2), limit=1.1):
    router = {"experts": experts, "top": top, "identity": identity}
    if groups:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": router}


def prenorm(layers, width=88, vocab=150, eps=1e-6, logit_scale=1.7):
    return {"architecture": "Sumevik", "width": width, "vocab": vocab, "norm": {"eps": eps}, "logit_scale": logit_scale, "layers": layers}


def grouped_attn(heads=6, kv_heads=2, dim=24, vdim=20, window=40, rot=8, base=10000.0, scaling=None, scale=None, source=None, mlp=None):
    """Grouped attention with a sink; window 0: no mask, rot 0: nothing is rotated; source: the layer whose keys and values it reads."""
    mx = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale or dim ** -0.5}
    if window:
        mx["mask"] = {"size": window}
    if rot:
        mx["rot"] = dict({"base": base, "dims": rot}, **({"scaling": scaling} if scaling else {}))
    if source is not None:
        mx["kv_from"] = source
    return {"type": "attention", "mixer": mx, "mlp": mlp}


def latent2(heads=3, dim=24, rot=8, vdim=20, rank=40, q_rank=28, window=40, scale=None, base=10000.0, dims=None, scaling=None, rotate=True, mlp=None):
    """Latent attention with a query latent and a gate per value; window 0: no mask."""
    lay = attn(heads, dim, rot, vdim, rank, scale, base, dims, scaling, 0, rotate)
    lay["mixer"]["q_rank"] = q_rank
    if window:
        lay["mixer"]["mask"] = {"size": window}
    return dict(lay, mlp=mlp)


def delta(heads=4, kv_heads=2, dim=24, vdim=20, taps=4, mlp=None):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": taps}, "mlp": mlp}


def sandwich_ln(layers, width=88, vocab=150, eps=1e-5, cap=2.5):
    return {"architecture": "Tarudra", "width": width, "vocab": vocab, "norm": {"eps": eps}, "logit_softcap": cap, "layers": layers}


def parse(pkg, cfg):
    def shape_of(name):
        return cfg["layers"][int(name[1:].split(".")[0])].get("rank"), cfg["width"]
    return pkg.layered_model.parse_config(cfg).resolve(shape_of)


def bf16(x):
    """Round to bf16 (nearest even), as f32."""
    u = np.ascontiguousarray(x, np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) & 0xFFFF0000).view(np.float32).reshape(np.shape(x))


class Weights(dict):
    """name -> f32 array of bf16 values; `get(name, shape)` is what the loader asks a source for."""

    def __init__(self, parsed, seed=0):
        super().__init__()
        rng = np.random.default_rng(seed)
        for name, shape in parsed.tensor_shapes():
            last = name.split(".")[-1]
            if getattr(parsed, "residual", 0) == 2 and last in ("norm1", "norm2") or getattr(parsed, "tied_head", False) and name == "final.norm":
                v = 0.2 * rng.standard_normal(shape)           # stored around zero
            elif last in ("ls1", "ls2"):
                v = 0.7 + 0.2 * rng.standard_normal(shape)
            elif last == "dt_bias":
                v = -4.0 + 1.5 * rng.standard_normal(shape)    # a state that lasts
            elif last == "lam":
                v = -5.0 + 1.5 * rng.standard_normal(shape)    # a state that lasts
            elif last == "conv":
                v = 0.5 * rng.standard_normal(shape)
            elif last == "correction":
                v = 0.1 * rng.standard_normal(shape)
            elif name.endswith(".a2.b"):
                v = 2.0 + rng.standard_normal(shape)
            elif len(shape) == 3:
                v = rng.standard_normal(shape) / np.sqrt(shape[-1])
            elif last == "b" and not name.endswith("mix.b"):
                v = (3.0 if name.endswith(".f.b") else 0.0) + (1.0 if name.endswith(".f.b") else 0.5) * rng.standard_normal(shape)
            elif name.endswith(".alpha"):
                v = np.asarray(0.4 + 0.4 * rng.random())
            elif name.endswith(".temp"):
                v = 1.0 + 0.3 * rng.standard_normal(shape)
            elif name.endswith(".sink"):
                v = rng.standard_normal(shape)
            elif "canon" in name:
                v = 0.4 * rng.standard_normal(shape)
            elif "norm" in last or name.endswith(("norm1", "norm2")):
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


def clear_calls(W, cfg, seed=77):
    """Routing without close calls, whatever the number format: every token carries a ranking of the experts in channels that no sublayer
    changes, and the routers read those channels alone.  In bf16 a close call may fall to either side, which says nothing."""
    E = max(lay["mlp"]["router"]["experts"] for lay in cfg["layers"] if lay["mlp"] and lay["mlp"]["kind"] == "moe")
    rng = np.random.default_rng(seed)
    for t in range(cfg["vocab"]):
        W["embed"][t, :E] = bf16((rng.permutation(E) - (E - 1) / 2) * (4.0 / E))
    for i, lay in enumerate(cfg["layers"]):
        for n in ("1", "2") if lay["mlp"] else ("1",):
            for part in ("b", "b.b"):
                W[f"l{i}.norm{n}{part}"][:E] = 0.0
        if lay["mlp"]:
            W[f"l{i}.norm2"][:E], W[f"l{i}.norm2.b"][:E] = 1.0, 0.0
            W[f"l{i}.canon2"][:E] = 0.0
            if lay["mlp"]["kind"] == "moe":
                W[f"l{i}.mlp.router"][:] = 3.0 * np.eye(lay["mlp"]["router"]["experts"], cfg["width"])
    return W


def clear_calls_prenorm(W, cfg, seed=77):
    """The same where sublayers add to the stream: nothing is added to the channels that carry the ranking (an identity expert scales them all)."""
    moes = [lay["mlp"]["router"] for lay in cfg["layers"] if lay["mlp"] and lay["mlp"]["kind"] == "moe"]
    if not moes:
        return W
    E = max(r["experts"] + r.get("identity", 0) for r in moes)
    rng = np.random.default_rng(seed)
    for t in range(cfg["vocab"]):
        W["embed"][t, :E] = bf16((rng.permutation(E) - (E - 1) / 2) * (6.0 / E))
    for name, v in W.items():
        if name.endswith((".o", ".down")):
            v[:E] = 0.0
    for i, lay in enumerate(cfg["layers"]):
        if lay["mlp"] and lay["mlp"]["kind"] == "moe":
            W[f"l{i}.norm2"][:E] = 0.0
            n = W[f"l{i}.mlp.router"].shape[0]
            W[f"l{i}.mlp.router"][:] = 2.0 * np.eye(n, cfg["width"])
            W[f"l{i}.mlp.correction"][:] = bf16(0.003 * rng.standard_normal(n))
    return W


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


TOL = {"f32": 2e-5, "bf16": 3e-2}
DTYPES = ("f32", "bf16")


def make(pkg, cfg, dtype, max_seq=256, seed=0, weights=None, **kw):
    parsed = parse(pkg, cfg)
    W = weights if weights is not None else Weights(parsed, seed)
    hb = pkg.hip_backend
    eng = pkg.HipGpuInference.from_layered(pkg.LayeredModel(parsed, W), max_seq, compute=hb.COMPUTE_F32 if dtype == "f32" else hb.COMPUTE_BF16, **kw)
    return eng, W


def check(got, want, dtype, what=""):
    """f32: every row.  bf16: every row but the few whose read-out nearly cancels before its RMS norm, which magnifies the rounding of the
    operands (the same rows are the worst of the f32 run, 20 times above the rest)."""
    err = row_error(got, want)
    if dtype == "bf16" and len(err) >= 40:
        assert err.max() <= 0.4, f"{what}: row {int(err.argmax())} off by {err.max():.2e}"
        err = np.sort(err)[: int(0.96 * len(err))]
    assert err.max() <= TOL[dtype], f"{what}: row {int(err.argmax())} of {len(err)} off by {err.max():.2e} (limit {TOL[dtype]:.0e})"


def stepwise(eng, toks):
    return np.array([eng.forward(int(t)) for t in toks])
