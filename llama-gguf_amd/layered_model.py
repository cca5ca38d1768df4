"""Models described layer by layer: the registry of architectures, config.json, safetensors weights.

A model folder holds ``config.json`` (its ``architecture`` picks the parser here) and ``model.safetensors``.  A parser turns the
configuration into ``LayeredConfig``; every layer is a mixer (``MIXERS``) and an optional feed-forward (``FEED_FORWARDS``), each read
by a function of its own, so another architecture made of the same parts adds one entry.  The engine takes the result through
``HipGpuInference.from_layered``; nothing here computes.
"""
from __future__ import annotations

import json
import os
from dataclasses import dataclass, field
from typing import Iterator, List, Optional, Tuple

import numpy as np

from . import hip_backend as hb

BF16, F32 = 30, 0        # ggml type ids
_SAFETENSORS_TYPES = {"BF16": (BF16, 2), "F32": (F32, 4)}


class ConfigError(ValueError):
    """config.json asks for something no part of the engine computes, or lacks a value."""


def _need(d: dict, key: str, where: str):
    if not isinstance(d, dict) or key not in d:
        raise ConfigError(f"{where}: '{key}' is missing")
    return d[key]


def _sizes(layer: hb.LayerDesc, mixer: dict, where: str, **fields) -> None:
    for name, key in fields.items():
        setattr(layer, name, int(_need(mixer, key, where)))


def _rotation(layer: hb.LayerDesc, mx: dict, where: str) -> None:
    """Leading values of a head (of its rotated part) that are rotated, with the frequencies' scaling; without an entry nothing is."""
    rot = mx.get("rot")
    if not rot:
        return
    layer.rot_dims, layer.rot_base = int(_need(rot, "dims", where)), float(_need(rot, "base", where))
    sc = rot.get("scaling")
    if sc:
        for f in ("factor", "original", "fast", "slow"):
            setattr(layer, "yarn_" + f, float(_need(sc, f, where)))
        if layer.yarn_factor <= 0.0:
            raise ConfigError(f"{where}: a scaling of {layer.yarn_factor}")


def _rotated_of(layer: hb.LayerDesc, size: int, where: str) -> None:
    if layer.rot_dims % 2 or layer.rot_dims > size:
        raise ConfigError(f"{where}: {layer.rot_dims} rotated values of {size}")


def _window(layer: hb.LayerDesc, mx: dict, where: str) -> None:
    """The last positions that a position sees; without an entry all of them."""
    mask = mx.get("mask")
    if mask is not None:
        layer.window = int(_need(mask, "size", where))
        if layer.window < 1:
            raise ConfigError(f"{where}: a window of {layer.window} positions")


def _head_groups(layer: hb.LayerDesc, where: str) -> None:
    if layer.kv_heads < 1 or layer.heads % layer.kv_heads:
        raise ConfigError(f"{where}: {layer.heads} heads do not divide into {layer.kv_heads} key heads")


def _latent_attention(layer: hb.LayerDesc, mx: dict, where: str) -> None:
    layer.mixer = hb.MIXER_LATENT_ATTENTION
    _sizes(layer, mx, where, heads="heads", dim="dim", vdim="vdim", kv_rank="kv_rank", rot_dim="rot_dim")
    layer.scale = float(_need(mx, "scale", where))
    _rotation(layer, mx, where)


def _windowed_latent_attention(layer: hb.LayerDesc, mx: dict, where: str) -> None:
    """Queries through a latent of their own, halves rotated, a window, every value gated."""
    _latent_attention(layer, mx, where)
    _sizes(layer, mx, where, q_rank="q_rank")
    if layer.q_rank < 1:
        raise ConfigError(f"{where}: a query latent of {layer.q_rank}")
    _rotated_of(layer, layer.rot_dim, where)
    layer.rot_form, layer.gate_form = hb.ROT_HALVES, hb.GATE_VALUES
    _window(layer, mx, where)


def _grouped_attention(layer: hb.LayerDesc, mx: dict, where: str) -> None:
    layer.mixer = hb.MIXER_GROUPED_ATTENTION
    _sizes(layer, mx, where, heads="heads", kv_heads="kv_heads", dim="dim", vdim="vdim")
    _head_groups(layer, where)
    layer.scale, layer.sink_one = float(_need(mx, "scale", where)), 1
    _rotation(layer, mx, where)
    _rotated_of(layer, layer.dim, where)
    _window(layer, mx, where)
    if mx.get("kv_from") is not None:
        layer.kv_from = int(mx["kv_from"]) + 1
        if layer.kv_from < 1:
            raise ConfigError(f"{where}: keys and values of layer {mx['kv_from']}")


def _delta(layer: hb.LayerDesc, mx: dict, where: str) -> None:
    layer.mixer = hb.MIXER_DELTA
    _sizes(layer, mx, where, heads="heads", kv_heads="kv_heads", dim="dim", vdim="vdim", taps="conv")
    _head_groups(layer, where)
    if layer.taps < 1:
        raise ConfigError(f"{where}: a convolution of {layer.taps} taps")


def _mlstm(layer: hb.LayerDesc, mx: dict, where: str) -> None:
    layer.mixer = hb.MIXER_MLSTM
    _sizes(layer, mx, where, heads="heads", dim="dim", vdim="vdim")
    layer.gate_cap = float(_need(mx, "gate_cap", where))


def _tied_attention(layer: hb.LayerDesc, mx: dict, where: str) -> None:
    layer.mixer = hb.MIXER_TIED_ATTENTION
    _sizes(layer, mx, where, heads="heads", kv_heads="kv_heads", dim="dim")
    layer.vdim = int(mx.get("vdim") or layer.dim)
    if layer.vdim != layer.dim:
        raise ConfigError(f"{where}: values are keys, 'vdim' {layer.vdim} differs from 'dim' {layer.dim}")
    _head_groups(layer, where)
    layer.scale = float(_need(mx, "scale", where))
    layer.score_cap = float(mx.get("softcap") or 0.0)
    _window(layer, mx, where)
    if mx.get("mask"):
        layer.keep_first = int(mx["mask"].get("keep_first") or 0)


def _gated_attention(layer: hb.LayerDesc, mx: dict, where: str) -> None:
    layer.mixer = hb.MIXER_GATED_ATTENTION
    _sizes(layer, mx, where, heads="heads", kv_heads="kv_heads", dim="dim", vdim="vdim")
    _head_groups(layer, where)
    layer.scale = float(_need(mx, "scale", where))
    _rotation(layer, mx, where)
    _rotated_of(layer, layer.dim, where)
    mask = mx.get("mask")
    if mask:
        layer.chunk = int(_need(mask, "size", where))
        if layer.chunk < 1:
            raise ConfigError(f"{where}: chunks of {layer.chunk} positions")


def _gla(layer: hb.LayerDesc, mx: dict, where: str) -> None:
    layer.mixer = hb.MIXER_GLA
    _sizes(layer, mx, where, gla_heads="heads", gla_dim="dim", gla_vdim="vdim")
    layer.gla_tau = float(_need(mx, "tau", where))


def _parallel(layer: hb.LayerDesc, mx: dict, where: str) -> None:
    _gated_attention(layer, _need(mx, "left", where), where + " left")
    _gla(layer, _need(mx, "right", where), where + " right")
    layer.mixer = hb.MIXER_PARALLEL
    layer.left_scale, layer.right_scale = float(_need(mx, "left_scale", where)), float(_need(mx, "right_scale", where))


def _rglru(layer: hb.LayerDesc, mx: dict, where: str) -> None:
    layer.mixer = hb.MIXER_GLRU
    width, layer.heads, layer.taps = (int(_need(mx, k, where)) for k in ("width", "blocks", "conv"))
    if layer.heads < 1 or width % layer.heads or layer.taps < 1:
        raise ConfigError(f"{where}: {width} channels, {layer.heads} blocks, {layer.taps} taps")
    layer.dim = layer.vdim = width // layer.heads


def _dense(layer: hb.LayerDesc, mlp: dict, where: str) -> None:
    layer.ff_kind, layer.ff = hb.FF_GEGLU, int(_need(mlp, "ff", where))


def _squared_relu(layer: hb.LayerDesc, mlp: dict, where: str) -> None:
    layer.ff_kind, layer.ff = hb.FF_RELU2, int(_need(mlp, "ff", where))


def _moe(layer: hb.LayerDesc, mlp: dict, where: str) -> None:
    layer.ff_kind, layer.ff = hb.FF_MOE, int(_need(_need(mlp, "expert", where), "ff", where))
    router = _need(mlp, "router", where)
    layer.experts, layer.top = int(_need(router, "experts", where)), int(_need(router, "top", where))
    if mlp.get("shared"):
        layer.shared_ff = int(_need(mlp["shared"], "ff", where))


def _grouped_moe(layer: hb.LayerDesc, mlp: dict, where: str) -> None:
    """Clamped experts, chosen by corrected softmax scores among the best groups; router outputs without tensors hand the input back."""
    _moe(layer, mlp, where)
    layer.router_form, layer.expert_form = hb.ROUTER_SOFTMAX_GROUPS, hb.EXPERT_CLAMPED
    layer.expert_limit = float(_need(mlp["expert"], "limit", where))
    router = mlp["router"]
    groups = router.get("groups") or {"count": 1, "keep": 1}
    layer.groups, layer.keep_groups = int(_need(groups, "count", where)), int(_need(groups, "keep", where))
    layer.identity = int(router.get("identity") or 0)
    n = layer.experts + layer.identity
    if layer.groups < 1 or n % layer.groups or not 1 <= layer.keep_groups <= layer.groups or layer.keep_groups * (n // layer.groups) < layer.top:
        raise ConfigError(f"{where}: {n} router outputs, {layer.groups} groups of which {layer.keep_groups} stay open, {layer.top} per token")


MIXERS = {"latent_attention": _latent_attention, "mlstm": _mlstm, "attention": _tied_attention, "gated_attention": _gated_attention, "gla": _gla,
          "parallel": _parallel, "rglru": _rglru, "grouped_attention": _grouped_attention, "windowed_latent_attention": _windowed_latent_attention,
          "delta": _delta}
FEED_FORWARDS = {"dense": _dense, "moe": _moe, "grouped_moe": _grouped_moe, "squared_relu": _squared_relu}


@dataclass
class LayeredConfig:
    name: str
    hidden_size: int
    vocab_size: int
    norm_eps: float
    residual_mult: float
    layers: List[hb.LayerDesc] = field(default_factory=list)
    bigram: Optional[Tuple[int, int, int]] = None      # buckets, factor of the previous token, factor of the token
    residual: int = hb.RESIDUAL_POST_LN
    conv_taps: int = 0
    tied_head: bool = False                            # the output projection is the embedding table
    logit_scale: float = 1.0
    logit_cap: float = 0.0                             # logits = cap * tanh(logits / cap); 0: none

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    def desc(self) -> hb.LayeredDesc:
        d = hb.LayeredDesc()
        d.struct_size = hb.C.sizeof(hb.LayeredDesc)
        d.width, d.vocab_size, d.num_layers = self.hidden_size, self.vocab_size, self.num_layers
        d.norm_eps, d.residual_mult = self.norm_eps, self.residual_mult
        d.residual, d.conv_taps = self.residual, self.conv_taps
        d.tied_head, d.logit_scale, d.logit_cap = int(self.tied_head), self.logit_scale, self.logit_cap
        if self.bigram:
            d.bigram_buckets, d.bigram_mul_prev, d.bigram_mul_cur = self.bigram
        return d

    def layer_descs(self):
        return (hb.LayerDesc * self.num_layers)(*self.layers)

    def _norm_shapes(self, name: str) -> Iterator[Tuple[str, Tuple[int, ...]]]:
        yield name, (self.hidden_size,)
        if self.residual == hb.RESIDUAL_SANDWICH_DYT:
            yield name + ".b", (self.hidden_size,)
            yield name + ".alpha", ()

    def _sublayer_shapes(self, p: str, which: int) -> Iterator[Tuple[str, Tuple[int, ...]]]:
        """What surrounds a layer's mixer (1) or feed-forward (2)."""
        yield from self._norm_shapes(f"{p}norm{which}")
        if self.residual == hb.RESIDUAL_SANDWICH_DYT:
            yield from self._norm_shapes(f"{p}norm{which}b")
        if self.residual == hb.RESIDUAL_SANDWICH_LN:
            yield f"{p}norm{which}b", (self.hidden_size,)
            yield f"{p}ls{which}", (self.hidden_size,)
        if self.conv_taps:
            yield f"{p}canon{which}", (self.hidden_size, self.conv_taps)

    def resolve(self, shape_of) -> "LayeredConfig":
        """Sizes that only a tensor's shape tells; shape_of(name) -> shape or None."""
        for i, l in enumerate(self.layers):
            if l.mixer in (hb.MIXER_GLA, hb.MIXER_PARALLEL):
                name = f"l{i}.mix.{'right.' if l.mixer == hb.MIXER_PARALLEL else ''}a1"
                shape = shape_of(name)
                if shape is None or len(shape) != 2 or shape[0] < 1:
                    raise ConfigError(f"tensor '{name}': shape {shape} does not tell the decay's inner size")
                l.gla_rank = int(shape[0])
        return self

    def _gated_shapes(self, p: str, l) -> Iterator[Tuple[str, Tuple[int, ...]]]:
        W = self.hidden_size
        for n, rows in (("q", l.heads * l.dim), ("k", l.kv_heads * l.dim), ("v", l.kv_heads * l.vdim)):
            yield p + n, (rows, W)
            yield p + n + ".b", (rows,)
        yield p + "q.norm", (l.dim,)
        yield p + "k.norm", (l.dim,)
        yield p + "g", (l.heads * l.vdim, W)
        yield p + "o", (W, l.heads * l.vdim)

    def _gla_shapes(self, p: str, l) -> Iterator[Tuple[str, Tuple[int, ...]]]:
        W, hd, vd = self.hidden_size, l.gla_heads * l.gla_dim, l.gla_heads * l.gla_vdim
        for n, rows in (("q", hd), ("k", hd), ("v", vd), ("g", vd)):
            yield p + n, (rows, W)
        yield p + "o", (W, vd)
        yield p + "norm", (l.gla_vdim,)
        yield p + "a1", (l.gla_rank, W)
        yield p + "a2", (hd, l.gla_rank)
        yield p + "a2.b", (hd,)

    def _rglru_shapes(self, p: str, l) -> Iterator[Tuple[str, Tuple[int, ...]]]:
        W, n = self.hidden_size, l.heads * l.dim
        for b in ("y", "x"):
            yield p + b, (n, W)
            yield p + b + ".b", (n,)
        yield p + "conv", (n, l.taps)
        yield p + "conv.b", (n,)
        for g in ("ra", "ri"):
            yield p + g, (l.heads, l.dim, l.dim)
            yield p + g + ".b", (l.heads, l.dim)
        yield p + "lam", (n,)
        yield p + "o", (W, n)

    def _latent_shapes(self, p: str, l) -> Iterator[Tuple[str, Tuple[int, ...]]]:
        W, rows, vd = self.hidden_size, l.heads * (l.dim + l.rot_dim), l.heads * l.vdim
        if l.q_rank:
            yield p + "dq", (l.q_rank, W)
            yield p + "dq.norm", (l.q_rank,)
            yield p + "uq", (rows, l.q_rank)
        else:
            yield p + "q", (rows, W)
        yield p + "dkv", (l.kv_rank + l.rot_dim, W)
        yield p + "dkv.norm", (l.kv_rank,)
        yield p + "uk", (l.heads * l.dim, l.kv_rank)
        yield p + "uv", (vd, l.kv_rank)
        yield p + "g", (vd if l.gate_form == hb.GATE_VALUES else l.heads, W)
        yield p + "o", (W, vd)

    def _grouped_shapes(self, p: str, l) -> Iterator[Tuple[str, Tuple[int, ...]]]:
        W = self.hidden_size
        for n, rows in (("q", l.heads * l.dim), ("k", l.kv_heads * l.dim), ("v", l.kv_heads * l.vdim)):
            if n == "q" or not l.kv_from:
                yield p + n, (rows, W)
                yield p + n + ".b", (rows,)
        yield p + "o", (W, l.heads * l.vdim)
        yield p + "o.b", (W,)

    def _delta_shapes(self, p: str, l) -> Iterator[Tuple[str, Tuple[int, ...]]]:
        W, vd = self.hidden_size, l.heads * l.vdim
        for n, rows in (("q", l.kv_heads * l.dim), ("k", l.kv_heads * l.dim), ("v", vd)):
            yield p + n, (rows, W)
            yield p + n + ".conv", (rows, l.taps)
        for n, rows in (("b", l.heads), ("a", l.heads), ("g", vd)):
            yield p + n, (rows, W)
        yield p + "A_log", (l.heads,)
        yield p + "dt_bias", (l.heads,)
        yield p + "norm", (l.vdim,)
        yield p + "o", (W, vd)

    def tensor_shapes(self) -> Iterator[Tuple[str, Tuple[int, ...]]]:
        """(name, shape) of every tensor the model needs, [out, in]."""
        W = self.hidden_size
        ff = lambda p, n: ((p + "gate", (n, W)), (p + "up", (n, W)), (p + "down", (W, n)))
        yield "embed", (self.vocab_size, W)
        if self.bigram:
            yield "bigram", (self.bigram[0] + 1, W)
        for i, l in enumerate(self.layers):
            p, vd = f"l{i}.", l.heads * l.vdim
            yield from self._sublayer_shapes(p, 1)
            if l.mixer == hb.MIXER_LATENT_ATTENTION:
                yield from self._latent_shapes(p + "mix.", l)
            elif l.mixer == hb.MIXER_GROUPED_ATTENTION:
                yield from self._grouped_shapes(p + "mix.", l)
            elif l.mixer == hb.MIXER_DELTA:
                yield from self._delta_shapes(p + "mix.", l)
            elif l.mixer == hb.MIXER_TIED_ATTENTION:
                for n, rows in (("q", vd), ("k", l.kv_heads * l.dim)):
                    yield p + "mix." + n, (rows, W)
                    yield p + "mix." + n + ".norm", (rows,)
                yield p + "mix.temp", (l.heads,)
                yield p + "mix.sink", (l.heads,)
            elif l.mixer == hb.MIXER_GATED_ATTENTION:
                yield from self._gated_shapes(p + "mix.", l)
            elif l.mixer == hb.MIXER_GLA:
                yield from self._gla_shapes(p + "mix.", l)
            elif l.mixer == hb.MIXER_PARALLEL:
                yield from self._gated_shapes(p + "mix.left.", l)
                yield from self._gla_shapes(p + "mix.right.", l)
            elif l.mixer == hb.MIXER_GLRU:
                yield from self._rglru_shapes(p + "mix.", l)
            else:
                yield p + "mix.q", (l.heads * l.dim, W)
                yield p + "mix.k", (l.heads * l.dim, W)
                yield p + "mix.v", (vd, W)
                yield p + "mix.g", (vd, W)
                yield p + "mix.norm", (vd,)
                for g in ("i", "f"):
                    yield p + "mix." + g, (l.heads, W)
                    yield p + "mix." + g + ".b", (l.heads,)
            if l.mixer in (hb.MIXER_TIED_ATTENTION, hb.MIXER_MLSTM):
                yield p + "mix.o", (W, vd)
            if l.ff_kind:
                yield from self._sublayer_shapes(p, 2)
            if l.ff_kind == hb.FF_MOE:
                yield p + "mlp.router", (l.experts + l.identity, W)
                if l.router_form == hb.ROUTER_SOFTMAX_GROUPS:
                    yield p + "mlp.correction", (l.experts + l.identity,)
                for e in range(l.experts):
                    yield from ff(f"{p}mlp.e{e}.", l.ff)
                if l.shared_ff:
                    yield from ff(p + "mlp.shared.", l.shared_ff)
            elif l.ff_kind == hb.FF_RELU2:
                yield p + "mlp.up", (l.ff, W)
                yield p + "mlp.down", (W, l.ff)
            elif l.ff_kind:
                yield from ff(p + "mlp.", l.ff)
        yield from self._norm_shapes("final.norm")
        if not self.tied_head:
            yield "head", (self.vocab_size, W)


def _zamelix(cfg: dict) -> LayeredConfig:
    """Latent attention and matrix-memory layers in any order, gated feed-forwards, layer norm on every sublayer's output, a hashed
    pair embedding."""
    where = "Zamelix"
    out = LayeredConfig(where, int(_need(cfg, "width", where)), int(_need(cfg, "vocab", where)),
                        float(_need(_need(cfg, "norm", where), "eps", where)), float(_need(cfg, "residual_mult", where)))
    big = (cfg.get("embedding") or {}).get("bigram")
    if big:
        out.bigram = tuple(int(_need(big, k, where)) for k in ("buckets", "mul_prev", "mul_cur"))
    _layers(out, cfg, where)
    return out


def _pubopel(cfg: dict) -> LayeredConfig:
    """Windowed attention whose values are its keys, mixtures of experts, squashing norms before and after every sublayer, a short causal
    convolution in front of it."""
    where = "Pubopel"
    out = LayeredConfig(where, int(_need(cfg, "width", where)), int(_need(cfg, "vocab", where)),
                        float(_need(_need(cfg, "norm", where), "eps", where)), 1.0, residual=hb.RESIDUAL_SANDWICH_DYT)
    out.conv_taps = int(_need(_need(cfg, "canon", where), "taps", where))
    if out.conv_taps < 1:
        raise ConfigError(f"{where}: a convolution of {out.conv_taps} taps")
    _layers(out, cfg, where)
    return out


def _sumevik(cfg: dict) -> LayeredConfig:
    """Gated linear recurrences, and gated chunked attention beside gated linear attention, in any order; dense feed-forwards or grouped mixtures;
    RMS norms in front of the sublayers; the embedding table as output projection."""
    where = "Sumevik"
    out = LayeredConfig(where, int(_need(cfg, "width", where)), int(_need(cfg, "vocab", where)),
                        float(_need(_need(cfg, "norm", where), "eps", where)), 1.0, residual=hb.RESIDUAL_PRE_RMS, tied_head=True)
    out.logit_scale = float(_need(cfg, "logit_scale", where))
    if not out.logit_scale:
        raise ConfigError(f"{where}: logit_scale is 0")
    _layers(out, cfg, where, dict(FEED_FORWARDS, moe=_grouped_moe))
    return out


def _tarudra(cfg: dict) -> LayeredConfig:
    """Windowed grouped attention (some layers on another layer's keys and values), windowed latent attention with query latents and gated delta rules,
    in any order; squared-relu feed-forwards; layer norms before and after every sublayer with a scale per channel; squashed logits."""
    where = "Tarudra"
    out = LayeredConfig(where, int(_need(cfg, "width", where)), int(_need(cfg, "vocab", where)),
                        float(_need(_need(cfg, "norm", where), "eps", where)), 1.0, residual=hb.RESIDUAL_SANDWICH_LN)
    out.logit_cap = float(_need(cfg, "logit_softcap", where))
    if not out.logit_cap > 0.0:
        raise ConfigError(f"{where}: logits capped at {out.logit_cap}")
    _layers(out, cfg, where, dict(FEED_FORWARDS, dense=_squared_relu), dict(MIXERS, attention=_grouped_attention, latent_attention=_windowed_latent_attention))
    for i, l in enumerate(out.layers):
        src = out.layers[l.kv_from - 1] if 0 < l.kv_from <= i else None
        if l.kv_from and (src is None or src.mixer != l.mixer or src.kv_from):
            raise ConfigError(f"{where} layer {i}: no keys and values in layer {l.kv_from - 1}")
        if src and any(getattr(l, f) != getattr(src, f) for f in ("heads", "kv_heads", "dim", "vdim", "rot_dims", "rot_base", "yarn_factor", "yarn_original", "yarn_fast", "yarn_slow")):
            raise ConfigError(f"{where} layer {i}: sizes or rotation differ from layer {l.kv_from - 1}, whose keys it reads")
    return out


def _layers(out: LayeredConfig, cfg: dict, where: str, feed_forwards: dict = FEED_FORWARDS, mixers: dict = MIXERS) -> None:
    """The 'layers' list: a mixer and an optional feed-forward each; feed_forwards, mixers: what a design calls its own."""
    for i, entry in enumerate(_need(cfg, "layers", where)):
        at = f"{where} layer {i}"
        layer = hb.LayerDesc()
        layer.struct_size = hb.C.sizeof(hb.LayerDesc)
        kind = _need(entry, "type", at)
        if kind not in mixers:
            raise ConfigError(f"{at}: unknown mixer '{kind}'")
        mixers[kind](layer, _need(entry, "mixer", at), at)
        mlp = entry.get("mlp")
        if mlp:
            if _need(mlp, "kind", at) not in feed_forwards:
                raise ConfigError(f"{at}: unknown feed-forward '{mlp['kind']}'")
            feed_forwards[mlp["kind"]](layer, mlp, at)
        out.layers.append(layer)


ARCHITECTURES = {"Zamelix": _zamelix, "Pubopel": _pubopel, "Sumevik": _sumevik, "Tarudra": _tarudra}      # config.json "architecture" -> parser


def parse_config(cfg: dict) -> LayeredConfig:
    arch = _need(cfg, "architecture", "config.json")
    if arch not in ARCHITECTURES:
        raise ConfigError(f"config.json: unknown architecture '{arch}' (known: {', '.join(sorted(ARCHITECTURES))})")
    return ARCHITECTURES[arch](cfg)


class SafetensorsFile:
    """The tensors of a .safetensors file, mapped: an 8-byte little-endian header length, a JSON header, then the data."""

    def __init__(self, path: str):
        size = os.path.getsize(path)
        with open(path, "rb") as f:
            n = int.from_bytes(f.read(8), "little")
            if n > size - 8:
                raise ConfigError(f"{path}: header longer than the file")
            self.header = json.loads(f.read(n))
        self.header.pop("__metadata__", None)
        self._data = np.memmap(path, dtype=np.uint8, mode="r", offset=8 + n) if size > 8 + n else np.zeros(0, np.uint8)

    def shape(self, name: str) -> Optional[Tuple[int, ...]]:
        h = self.header.get(name)
        return None if h is None else tuple(h["shape"])

    def get(self, name: str, shape: Tuple[int, ...]) -> Tuple[int, np.ndarray]:
        """(ggml type, bytes) of a tensor, checked against the shape the model needs."""
        h = self.header.get(name)
        if h is None:
            raise ConfigError(f"tensor '{name}' is missing")
        if h["dtype"] not in _SAFETENSORS_TYPES:
            raise ConfigError(f"tensor '{name}': type {h['dtype']} is not supported")
        t, el = _SAFETENSORS_TYPES[h["dtype"]]
        a, b = h["data_offsets"]
        if tuple(h["shape"]) != tuple(shape) or b - a != el * int(np.prod(shape)) or a < 0 or b > self._data.size:
            raise ConfigError(f"tensor '{name}': shape {h['shape']}, expected {list(shape)}")
        return t, self._data[a:b]


class LayeredModel:
    """A configuration with its weights; `tensors()` is what `HipGpuInference.from_layered` uploads."""

    def __init__(self, config: LayeredConfig, source):
        self.config, self._source = config, source       # source.get(name, shape) -> (ggml type, bytes)

    @classmethod
    def from_dir(cls, path: str) -> "LayeredModel":
        with open(os.path.join(path, "config.json")) as f:
            cfg = parse_config(json.load(f))
        source = SafetensorsFile(os.path.join(path, "model.safetensors"))
        return cls(cfg.resolve(source.shape), source)

    def tensors(self):
        for name, shape in self.config.tensor_shapes():
            t, data = self._source.get(name, shape)
            yield name, t, tuple(reversed(shape)) or (1,), data

    def weight_bytes(self) -> int:
        return sum(2 * int(np.prod(s)) for _, s in self.config.tensor_shapes())


def load_model(path: str, max_seq_len: int, device: int = 0, compute: int = hb.COMPUTE_BF16, flags: int = 0) -> hb.HipGpuInference:
    """A model folder (config.json + model.safetensors) or a .gguf file -> a ready context."""
    if os.path.isdir(path):
        return hb.HipGpuInference.from_layered(LayeredModel.from_dir(path), max_seq_len, device, compute, flags)
    if compute == hb.COMPUTE_F32:
        raise hb.BackendError(5, "GGUF models run with quantized weights and f32 activations; there is no separate 32-bit mode")
    return hb.HipGpuInference.from_gguf(path, max_seq_len, device, flags=flags)
