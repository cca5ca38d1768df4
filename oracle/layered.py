"""Plain numpy (float64) restatement of models whose layers are described one by one (mixer + optional feed-forward): TEST
INFRASTRUCTURE only, slow on purpose, one function per mechanism, no code shared with the product.

Weights are a dict name -> array ([out, in] for linear maps); ``cfg`` is the parsed config.json.  Every function takes whole
sequences; ``forward`` runs a prompt from nothing, and ``forward(..., cache=...)`` is deliberately NOT offered: a test that needs
"prompt then decode" compares the product's steps against rows of one whole-sequence run.
"""
from __future__ import annotations

import math

import numpy as np

F = np.float64


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def log_sigmoid(z):
    return -np.logaddexp(0.0, -z)


def rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def layer_norm(x, w, eps):
    mu = np.mean(x, axis=-1, keepdims=True)
    d = x - mu
    return d / np.sqrt(np.mean(d * d, axis=-1, keepdims=True) + eps) * w


def bigram_rows(tokens, buckets, mul_prev, mul_cur):
    """Row of the pair table for every position: a hash of (previous, current); the extra last row opens a sequence."""
    return [buckets if p == 0 else (int(tokens[p - 1]) * mul_prev + int(tokens[p]) * mul_cur) % buckets for p in range(len(tokens))]


def rope_frequencies(rot):
    """(frequency of each pair, factor on cos and sin) with the YaRN blend when ``rot`` has a scaling entry."""
    n, base = int(rot["dims"]), float(rot["base"])
    f = np.array([base ** (-2.0 * i / n) for i in range(n // 2)], dtype=F)
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0
    turn = lambda t: n * math.log(sc["original"] / (2 * math.pi * t)) / (2 * math.log(base))
    lo, hi = max(math.floor(turn(sc["fast"])), 0), min(math.ceil(turn(sc["slow"])), n - 1)
    ramp = np.clip((np.arange(n // 2) - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / sc["factor"] * ramp + f * (1.0 - ramp), 0.1 * math.log(sc["factor"]) + 1.0


def rotate_pairs(x, positions, rot):
    """x [T, ..., d]: neighbouring pairs (2i, 2i+1) of the first rot.dims values turned by position * frequency."""
    f, mag = rope_frequencies(rot)
    n = int(rot["dims"])
    out = np.array(x, dtype=F)
    ang = np.asarray(positions, dtype=F).reshape((-1,) + (1,) * (x.ndim - 1)) * f
    c, s = np.cos(ang) * mag, np.sin(ang) * mag
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    out[..., 0:n:2] = u * c - v * s
    out[..., 1:n:2] = v * c + u * s
    return out


def rotate_halves(x, positions, rot):
    """x [T, ..., d]: value i of the first rot.dims paired with value i + dims / 2."""
    f, mag = rope_frequencies(rot)
    n = int(rot["dims"])
    out = np.array(x, dtype=F)
    ang = np.asarray(positions, dtype=F).reshape((-1,) + (1,) * (x.ndim - 1)) * f
    c, s = np.cos(ang) * mag, np.sin(ang) * mag
    u, v = x[..., : n // 2], x[..., n // 2: n]
    out[..., : n // 2] = u * c - v * s
    out[..., n // 2: n] = v * c + u * s
    return out


def latent_attention(h, w, mx, eps):
    """h [T, width] -> [T, width]; w: the layer's mixer tensors by short name."""
    T, H, d, r, dv, kr = len(h), mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"], mx["kv_rank"]
    pos = np.arange(T)
    q = (h @ w["q"].T).reshape(T, H, d + r)
    dkv = h @ w["dkv"].T
    c = rms(dkv[:, :kr], eps) * w["dkv.norm"]
    turn = lambda x: rotate_pairs(x, pos, mx["rot"]) if mx.get("rot") else x
    k_rot, q_rot = turn(dkv[:, kr:]), turn(q[..., d:])
    k = (c @ w["uk"].T).reshape(T, H, d)
    v = (c @ w["uv"].T).reshape(T, H, dv)
    gate = sigmoid(h @ w["g"].T)
    out = np.zeros((T, H, dv), dtype=F)
    for i in range(T):
        for n in range(H):
            s = (k[: i + 1, n] @ q[i, n, :d] + k_rot[: i + 1] @ q_rot[i, n]) * mx["scale"]
            p = np.exp(s - s.max())
            out[i, n] = (p / p.sum()) @ v[: i + 1, n] * gate[i, n]
    return out.reshape(T, H * dv) @ w["o"].T


def mlstm(h, w, mx, eps):
    """The matrix memory, one token after the other, from an empty state."""
    T, H, d, dv, cap = len(h), mx["heads"], mx["dim"], mx["vdim"], mx["gate_cap"]
    q = (h @ w["q"].T).reshape(T, H, d) * d ** -0.5
    k = (h @ w["k"].T).reshape(T, H, d)
    v = (h @ w["v"].T).reshape(T, H, dv)
    li = cap * np.tanh((h @ w["i"].T + w["i.b"]) / cap)
    lf = log_sigmoid(cap * np.tanh((h @ w["f"].T + w["f.b"]) / cap))
    out = np.zeros((T, H, dv), dtype=F)
    for n in range(H):
        S, nv, m = np.zeros((d, dv), dtype=F), np.zeros(d, dtype=F), 0.0
        for t in range(T):
            m2 = max(lf[t, n] + m, li[t, n])
            a, b = math.exp(lf[t, n] + m - m2), math.exp(li[t, n] - m2)
            m = m2
            S = a * S + b * np.outer(k[t, n], v[t, n])
            nv = a * nv + b * k[t, n]
            out[t, n] = (S.T @ q[t, n]) / (max(abs(nv @ q[t, n]), math.exp(-m)) + 1e-6)
    out = rms(out, eps).reshape(T, H * dv) * w["norm"] * sigmoid(h @ w["g"].T)
    return out @ w["o"].T


def query_latent(h, w, eps):
    """Queries through a latent of their own, which is normed between its two projections."""
    return (rms(h @ w["dq"].T, eps) * w["dq.norm"]) @ w["uq"].T


def windowed_latent_attention(h, w, mx, eps):
    """Attention over a shared latent whose queries have a latent too; the last `size` positions are visible; halves rotated; every value gated."""
    T, H, d, r, dv, kr = len(h), mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"], mx["kv_rank"]
    pos = np.arange(T)
    q = query_latent(h, w, eps).reshape(T, H, d + r)
    dkv = h @ w["dkv"].T
    c = rms(dkv[:, :kr], eps) * w["dkv.norm"]
    turn = lambda x: rotate_halves(x, pos, mx["rot"]) if mx.get("rot") else x
    k_rot, q_rot = turn(dkv[:, kr:]), turn(q[..., d:])
    k = (c @ w["uk"].T).reshape(T, H, d)
    v = (c @ w["uv"].T).reshape(T, H, dv)
    out = np.zeros((T, H, dv), dtype=F)
    for i in range(T):
        seen = visible_keys(i, mx.get("mask"))
        for n in range(H):
            s = (k[seen, n] @ q[i, n, :d] + k_rot[seen] @ q_rot[i, n]) * mx["scale"]
            p = np.exp(s - s.max())
            out[i, n] = (p / p.sum()) @ v[seen, n]
    return (out.reshape(T, H * dv) * sigmoid(h @ w["g"].T)) @ w["o"].T


def grouped_keys_values(h, w, mx):
    """What a grouped attention layer caches: rotated keys [T, G, d] and values [T, G, dv]."""
    T, G = len(h), mx["kv_heads"]
    k, v = linear(h, w, "k").reshape(T, G, mx["dim"]), linear(h, w, "v").reshape(T, G, mx["vdim"])
    return (rotate_pairs(k, np.arange(T), mx["rot"]) if mx.get("rot") else k), v


def grouped_attention(h, w, mx, kv):
    """Grouped attention on given keys and values (its own or another layer's): rotated queries, a window, one more in the softmax's denominator."""
    T, H, G = len(h), mx["heads"], mx["kv_heads"]
    k, v = kv
    q = linear(h, w, "q").reshape(T, H, mx["dim"])
    if mx.get("rot"):
        q = rotate_pairs(q, np.arange(T), mx["rot"])
    out = np.zeros((T, H, mx["vdim"]), dtype=F)
    for i in range(T):
        seen = visible_keys(i, mx.get("mask"))
        for n in range(H):
            g = n // (H // G)
            out[i, n] = sink_softmax((k[seen, g] @ q[i, n]) * mx["scale"], 0.0) @ v[seen, g]
    return linear(out.reshape(T, -1), w, "o")


def unit(x):
    """Vectors of length one along the last axis."""
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + 1e-6)


def delta_rule(h, w, mx, eps):
    """A matrix state per head that decays as a whole and is corrected towards each value, one token after the other."""
    T, H, G, d, dv = len(h), mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    short = lambda name: silu(causal_conv(h @ w[name].T, w[name + ".conv"]))
    q = unit(short("q").reshape(T, G, d)) * d ** -0.5
    k = unit(short("k").reshape(T, G, d))
    v = short("v").reshape(T, H, dv)
    beta = sigmoid(h @ w["b"].T)
    g = np.exp(-np.exp(w["A_log"]) * softplus(h @ w["a"].T + w["dt_bias"]))
    out = np.zeros((T, H, dv), dtype=F)
    for n in range(H):
        S = np.zeros((d, dv), dtype=F)
        m = n // (H // G)
        for t in range(T):
            S = g[t, n] * S
            u = beta[t, n] * (v[t, n] - S.T @ k[t, m])
            S = S + np.outer(k[t, m], u)
            out[t, n] = S.T @ q[t, m]
    o = rms(out, eps) * w["norm"]
    return (o.reshape(T, H * dv) * silu(h @ w["g"].T)) @ w["o"].T


def squared_relu_ff(x, w):
    return (np.maximum(x @ w["up"].T, 0.0) ** 2) @ w["down"].T


def visible_keys(i, mask):
    """Positions that position i sees: all up to itself, or the last ``size`` of them and the sequence's first ``keep_first``."""
    if not mask:
        return list(range(i + 1))
    return [j for j in range(i + 1) if i - j < mask["size"] or j < mask.get("keep_first", 0)]


def head_slope(h, heads):
    """What a unit of distance costs head h."""
    return 2.0 ** (-8.0 * (h + 1) / heads)


def soft_cap(s, cap):
    return cap * np.tanh(s / cap) if cap else s


def sink_softmax(s, sink):
    """Weights of the scores s when the denominator has one more term, exp(sink)."""
    m = max(s.max(), sink)
    p = np.exp(s - m)
    return p / (p.sum() + math.exp(sink - m))


def tied_attention(h, w, mx, eps):
    """Grouped attention whose values are its keys as they were projected; queries and keys are normed over all heads at once."""
    T, H, G, d = len(h), mx["heads"], mx["kv_heads"], mx["dim"]
    q = (rms(h @ w["q"].T, eps) * w["q.norm"]).reshape(T, H, d)
    v = (h @ w["k"].T).reshape(T, G, d)
    k = (rms(h @ w["k"].T, eps) * w["k.norm"]).reshape(T, G, d)
    out = np.zeros((T, H, d), dtype=F)
    for i in range(T):
        seen = visible_keys(i, mx.get("mask"))
        for n in range(H):
            g = n // (H // G)
            s = soft_cap((k[seen, g] @ q[i, n]) * mx["scale"] * w["temp"][n], mx.get("softcap"))
            s = s - head_slope(n, H) * (i - np.array(seen, dtype=F))
            out[i, n] = sink_softmax(s, w["sink"][n]) @ v[seen, g]
    return out.reshape(T, H * d) @ w["o"].T


def silu(z):
    return z * sigmoid(z)


def dense_ff(x, w):
    return (gelu_tanh(x @ w["gate"].T) * (x @ w["up"].T)) @ w["down"].T


def expert(x, w, name):
    return (silu(x @ w[name + ".gate"].T) * (x @ w[name + ".up"].T)) @ w[name + ".down"].T


def route(z, top):
    """(expert, weight) of the ``top`` largest scores, largest first; the weights are the scores."""
    s = sigmoid(z)
    order = sorted(range(len(z)), key=lambda e: (-z[e], e))[:top]
    return [(e, s[e]) for e in order]


def moe_ff(x, w, mlp):
    """Every token through its experts, each of which reads the token times its weight; a shared expert beside them."""
    out = np.zeros_like(x)
    for t, z in enumerate(x @ w["router"].T):
        for e, g in route(z, mlp["router"]["top"]):
            out[t] += expert(g * x[t], w, f"e{e}")
    return out + expert(x, w, "shared") if mlp.get("shared") else out


def dyt(x, w, b, alpha):
    """A norm without statistics: a squashed multiple of every value."""
    return np.tanh(alpha * x) * w + b


def causal_conv(h, w):
    """Every channel's own filter over time, w [width, taps], the last tap at the token itself; nothing before the first token."""
    out = np.zeros_like(h)
    taps = w.shape[1]
    for t in range(len(h)):
        for j in range(taps):
            if t - taps + 1 + j >= 0:
                out[t] += w[:, j] * h[t - taps + 1 + j]
    return out


def softplus(z):
    return np.logaddexp(0.0, z)


def linear(x, w, name):
    """A projection, with its bias where there is one."""
    y = x @ w[name].T
    return y + w[name + ".b"] if name + ".b" in w else y


def block_diagonal(u, m, b):
    """u [T, n * s] in n parts, each through its own square matrix m [n, s, s] with bias b [n, s]."""
    n, s = m.shape[0], m.shape[1]
    parts = [u[:, i * s:(i + 1) * s] @ m[i].T + b[i] for i in range(n)]
    return np.concatenate(parts, axis=1)


def linear_recurrence(a, x):
    """S_t = a_t S_(t-1) + x_t per channel, from nothing; all S [T, channels]."""
    S, out = np.zeros(a.shape[1], dtype=F), np.zeros_like(a)
    for t in range(len(a)):
        S = a[t] * S + x[t]
        out[t] = S
    return out


def rglru(h, w, mx, eps):
    """A gated linear recurrence per channel behind a short convolution, beside a gelu branch."""
    y = gelu_tanh(linear(h, w, "y"))
    u = causal_conv(linear(h, w, "x"), w["conv"]) + w["conv.b"]
    r = sigmoid(block_diagonal(u, w["ra"], w["ra.b"]))
    i = sigmoid(block_diagonal(u, w["ri"], w["ri.b"]))
    log_a = -8.0 * r * softplus(w["lam"])
    S = linear_recurrence(np.exp(log_a), np.sqrt(-np.expm1(2.0 * log_a)) * i * u)
    return (S * y) @ w["o"].T


def chunk_keys(i, size):
    """Positions that position i sees when the sequence is cut into chunks of `size` (0: not cut) from position 0 on."""
    return list(range(i // size * size if size else 0, i + 1))


def gated_attention(h, w, mx, eps):
    """Grouped attention with its own values; queries and keys normed per head and then rotated; keys of the own chunk; the output gated element
    by element before its projection."""
    T, H, G, d, dv = len(h), mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    pos = np.arange(T)
    q = rms(linear(h, w, "q").reshape(T, H, d), eps) * w["q.norm"]
    k = rms(linear(h, w, "k").reshape(T, G, d), eps) * w["k.norm"]
    v = linear(h, w, "v").reshape(T, G, dv)
    if mx.get("rot"):
        q, k = rotate_pairs(q, pos, mx["rot"]), rotate_pairs(k, pos, mx["rot"])
    size = mx["mask"]["size"] if mx.get("mask") else 0
    out = np.zeros((T, H, dv), dtype=F)
    for i in range(T):
        seen = chunk_keys(i, size)
        for n in range(H):
            g = n // (H // G)
            s = (k[seen, g] @ q[i, n]) * mx["scale"]
            p = np.exp(s - s.max())
            out[i, n] = (p / p.sum()) @ v[seen, g]
    return (out.reshape(T, H * dv) * sigmoid(h @ w["g"].T)) @ w["o"].T


def gated_linear_attention(h, w, mx, eps):
    """A matrix state per head whose rows (key channels) decay each at its own rate, one token after the other."""
    T, H, d, dv = len(h), mx["heads"], mx["dim"], mx["vdim"]
    q = (h @ w["q"].T).reshape(T, H, d) * d ** -0.5
    k = (h @ w["k"].T).reshape(T, H, d)
    v = (h @ w["v"].T).reshape(T, H, dv)
    z = (h @ w["a1"].T) @ w["a2"].T + w["a2.b"]
    alpha = np.exp(log_sigmoid(z) / mx["tau"]).reshape(T, H, d)
    out = np.zeros((T, H, dv), dtype=F)
    for n in range(H):
        S = np.zeros((d, dv), dtype=F)
        for t in range(T):
            S = alpha[t, n][:, None] * S + np.outer(k[t, n], v[t, n])
            out[t, n] = S.T @ q[t, n]
    o = rms(out, eps) * w["norm"]
    return (o.reshape(T, H * dv) * silu(h @ w["g"].T)) @ w["o"].T


def parallel(h, w, mx, eps):
    """Attention and linear attention side by side on the same input."""
    side = lambda s: {k[len(s):]: v for k, v in w.items() if k.startswith(s)}
    return (mx["left_scale"] * gated_attention(h, side("left."), mx["left"], eps)
            + mx["right_scale"] * gated_linear_attention(h, side("right."), mx["right"], eps))


def clamped_expert(x, w, name, limit):
    g = np.minimum(x @ w[name + ".gate"].T, limit)
    u = np.clip(x @ w[name + ".up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w[name + ".down"].T


def route_groups(z, correction, router):
    """(expert, weight) of a token: softmax scores; the choice by corrected scores among the best groups of neighbours; the weights are the plain
    scores of the chosen ones, divided by their sum."""
    s = np.exp(z - z.max())
    s = s / s.sum()
    c = s + correction
    groups = router.get("groups") or {"count": 1, "keep": 1}
    n, keep = groups["count"], groups["keep"]
    size = len(z) // n
    best = sorted(range(n), key=lambda g: (-c[g * size:(g + 1) * size].max(), g))[:keep]
    open_ = [e for e in range(len(z)) if e // size in best]
    chosen = sorted(open_, key=lambda e: (-c[e], e))[: router["top"]]
    total = sum(s[e] for e in chosen) + 1e-20
    return [(e, s[e] / total) for e in chosen]


def grouped_moe_ff(x, w, mlp):
    """Weighted sum of the chosen experts' outputs; the last `identity` router outputs hand the input back."""
    out = np.zeros_like(x)
    for t, z in enumerate(x @ w["router"].T):
        for e, g in route_groups(z, w["correction"], mlp["router"]):
            out[t] += g * (x[t] if e >= mlp["router"]["experts"] else clamped_expert(x[t], w, f"e{e}", mlp["expert"]["limit"]))
    return out


MIXERS = {"latent_attention": latent_attention, "mlstm": mlstm, "attention": tied_attention, "rglru": rglru, "parallel": parallel,
          "gated_attention": gated_attention, "gla": gated_linear_attention}


def feed_forward(x, w, mlp):
    if mlp["kind"] != "moe":
        return dense_ff(x, w)
    return grouped_moe_ff(x, w, mlp) if "limit" in mlp["expert"] else moe_ff(x, w, mlp)


def forward_pre_norm(cfg, weights, tokens, layers_out=None):
    """Sublayers read the RMS-normed stream and add to it; the output projection is the embedding table."""
    W = {k: np.asarray(v, dtype=F) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    norm = lambda v, name: rms(v, eps) * (1.0 + W[name])
    x = W["embed"][list(tokens)]
    for i, lay in enumerate(cfg["layers"]):
        p = f"l{i}."
        sub = lambda g: {k[len(p + g):]: v for k, v in W.items() if k.startswith(p + g)}
        x = x + MIXERS[lay["type"]](norm(x, p + "norm1"), sub("mix."), lay["mixer"], eps)
        if lay["mlp"]:
            x = x + feed_forward(norm(x, p + "norm2"), sub("mlp."), lay["mlp"])
        if layers_out is not None:
            layers_out.append(x.copy())
    return norm(x, "final.norm") @ W["embed"].T * cfg["logit_scale"]


def forward_sandwich(cfg, weights, tokens, layers_out=None):
    """Squashing norms before and after every sublayer, whose input is the normed stream plus a short causal convolution of it."""
    W = {k: np.asarray(v, dtype=F) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    norm = lambda v, name: dyt(v, W[name], W[name + ".b"], W[name + ".alpha"])
    x = W["embed"][list(tokens)]
    for i, lay in enumerate(cfg["layers"]):
        p = f"l{i}."
        sub = lambda g: {k[len(p + g):]: v for k, v in W.items() if k.startswith(p + g)}

        def read(n):
            h = norm(x, f"{p}norm{n}")
            return h + causal_conv(h, W[f"{p}canon{n}"])
        x = x + norm(MIXERS[lay["type"]](read(1), sub("mix."), lay["mixer"], eps), p + "norm1b")
        if lay["mlp"]:
            x = x + norm(feed_forward(read(2), sub("mlp."), lay["mlp"]), p + "norm2b")
        if layers_out is not None:
            layers_out.append(x.copy())
    return norm(x, "final.norm") @ W["head"].T


def forward_sandwich_ln(cfg, weights, tokens, layers_out=None):
    """Layer norms before and after every sublayer, whose result is scaled channel by channel; layers may read another layer's keys and values;
    logits are squashed."""
    W = {k: np.asarray(v, dtype=F) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    norm = lambda v, name: layer_norm(v, W[name], eps)
    x = W["embed"][list(tokens)]
    kvs = {}
    for i, lay in enumerate(cfg["layers"]):
        p, mx = f"l{i}.", lay["mixer"]
        sub = lambda g: {k[len(p + g):]: v for k, v in W.items() if k.startswith(p + g)}
        h, w = norm(x, p + "norm1"), sub("mix.")
        if lay["type"] == "attention":
            src = mx.get("kv_from")
            kvs[i] = grouped_keys_values(h, w, mx) if src is None else kvs[src]
            y = grouped_attention(h, w, mx, kvs[i])
        else:
            y = {"latent_attention": windowed_latent_attention, "delta": delta_rule}[lay["type"]](h, w, mx, eps)
        x = x + norm(y, p + "norm1b") * W[p + "ls1"]
        if lay["mlp"]:
            x = x + norm(squared_relu_ff(norm(x, p + "norm2"), sub("mlp.")), p + "norm2b") * W[p + "ls2"]
        if layers_out is not None:
            layers_out.append(x.copy())
    return soft_cap(norm(x, "final.norm") @ W["head"].T, cfg["logit_softcap"])


def forward(cfg, weights, tokens, layers_out=None):
    """Logits [T, vocab] of a whole sequence; layers_out (a list) receives the residual stream after every layer."""
    if "canon" in cfg:
        return forward_sandwich(cfg, weights, tokens, layers_out)
    if "logit_softcap" in cfg:
        return forward_sandwich_ln(cfg, weights, tokens, layers_out)
    if "logit_scale" in cfg:
        return forward_pre_norm(cfg, weights, tokens, layers_out)
    W = {k: np.asarray(v, dtype=F) for k, v in weights.items()}
    eps, m = cfg["norm"]["eps"], cfg["residual_mult"]
    x = W["embed"][list(tokens)]
    big = (cfg.get("embedding") or {}).get("bigram")
    if big:
        x = x + W["bigram"][bigram_rows(tokens, big["buckets"], big["mul_prev"], big["mul_cur"])]
    for i, lay in enumerate(cfg["layers"]):
        p = f"l{i}."
        sub = lambda g: {k[len(p + g):]: v for k, v in W.items() if k.startswith(p + g)}
        x = x + m * layer_norm(MIXERS[lay["type"]](x, sub("mix."), lay["mixer"], eps), W[p + "norm1"], eps)
        if lay["mlp"]:
            x = x + m * layer_norm(feed_forward(x, sub("mlp."), lay["mlp"]), W[p + "norm2"], eps)
        if layers_out is not None:
            layers_out.append(x.copy())
    return layer_norm(x, W["final.norm"], eps) @ W["head"].T
