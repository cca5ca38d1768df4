"""CPU: the plain restatement of the layer-by-layer models (oracle/layered.py) against independent identities, the registry and
configuration parsing, the safetensors reader, and how the product answers what it cannot run."""
import math

import numpy as np
import pytest

import layered_cases as lc
from oracle import layered as lo


# ---- mechanisms ----
def test_gelu_and_log_sigmoid_known_values():
    assert lo.gelu_tanh(np.array([0.0, 1.0, -1.0])) == pytest.approx([0.0, 0.841192, -0.158808], abs=1e-6)
    assert lo.log_sigmoid(np.array([0.0, 800.0, -800.0])) == pytest.approx([-math.log(2), 0.0, -800.0])


def test_layer_norm_is_shift_and_scale_free():
    x = np.random.default_rng(0).standard_normal((3, 17))
    w = np.linspace(0.5, 1.5, 17)
    a, b = lo.layer_norm(x, w, 0.0), lo.layer_norm(7.0 * x + 3.0, w, 0.0)
    assert np.allclose(a, b) and np.allclose((a / w).mean(-1), 0) and np.allclose(((a / w) ** 2).mean(-1), 1)


def test_bigram_rows():
    assert lo.bigram_rows([5, 7, 7], 11, 3, 2) == [11, (15 + 14) % 11, (21 + 14) % 11]


def test_rotation_is_relative_and_pairs_are_neighbours():
    rot = {"dims": 6, "base": 100.0}
    x = np.random.default_rng(1).standard_normal((1, 8))
    y = np.random.default_rng(2).standard_normal((1, 8))
    dot = lambda p, q: float((lo.rotate_pairs(x, [p], rot) @ lo.rotate_pairs(y, [q], rot).T).item())
    assert dot(9, 4) == pytest.approx(dot(105, 100)) and dot(0, 0) == pytest.approx(float((x @ y.T).item()))
    r = lo.rotate_pairs(x, [3], rot)
    assert np.hypot(r[0, 0], r[0, 1]) == pytest.approx(np.hypot(x[0, 0], x[0, 1])) and np.array_equal(r[0, 6:], x[0, 6:])


def test_yarn_keeps_fast_pairs_and_stretches_slow_ones():
    rot = {"dims": 32, "base": 10000.0, "scaling": {"factor": 8.0, "original": 256, "fast": 16.0, "slow": 1.0}}
    f, mag = lo.rope_frequencies(rot)
    plain, one = lo.rope_frequencies({"dims": 32, "base": 10000.0})
    assert one == 1.0 and mag == pytest.approx(0.1 * math.log(8) + 1)
    assert f[0] == pytest.approx(plain[0]) and f[-1] == pytest.approx(plain[-1] / 8)
    assert np.all(f <= plain + 1e-15) and np.all(f >= plain / 8 - 1e-15)


def test_matrix_memory_recurrence_equals_its_explicit_sum():
    rng = np.random.default_rng(3)
    T, W, mx = 9, 11, {"heads": 2, "dim": 5, "vdim": 4, "gate_cap": 6.0}
    shapes = {"q": (10, W), "k": (10, W), "v": (8, W), "g": (8, W), "i": (2, W), "f": (2, W), "i.b": (2,), "f.b": (2,), "norm": (8,), "o": (W, 8)}
    w = {k: rng.standard_normal(s) for k, s in shapes.items()}
    h = rng.standard_normal((T, W))
    li = 6 * np.tanh((h @ w["i"].T + w["i.b"]) / 6)
    lf = lo.log_sigmoid(6 * np.tanh((h @ w["f"].T + w["f.b"]) / 6))
    q, k, v = ((h @ w[n].T).reshape(T, 2, -1) for n in "qkv")
    out = np.zeros((T, 2, 4))
    for n in range(2):
        for t in range(T):
            wt = np.array([math.exp(li[s, n] + lf[s + 1: t + 1, n].sum()) for s in range(t + 1)])   # unnormalised weights
            m = 0.0
            for s in range(t + 1):
                m = max(lf[s, n] + m, li[s, n])
            a = wt * (k[: t + 1, n] @ q[t, n]) / math.sqrt(5) * math.exp(-m)
            out[t, n] = a @ v[: t + 1, n] / (max(abs(a.sum()), math.exp(-m)) + 1e-6)
    want = (lo.rms(out, 1e-5).reshape(T, 8) * w["norm"] * lo.sigmoid(h @ w["g"].T)) @ w["o"].T
    assert np.allclose(lo.mlstm(h, w, mx, 1e-5), want, rtol=1e-9, atol=1e-12)


def test_latent_attention_equals_the_absorbed_form():
    rng = np.random.default_rng(4)
    mx = lc.attn(ff=0)["mixer"]
    H, d, r, dv, kr, W, T = mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"], mx["kv_rank"], 30, 7
    w = {"q": (H * (d + r), W), "dkv": (kr + r, W), "dkv.norm": (kr,), "uk": (H * d, kr), "uv": (H * dv, kr), "g": (H, W), "o": (W, H * dv)}
    w = {k: rng.standard_normal(s) for k, s in w.items()}
    h = rng.standard_normal((T, W))
    dkv = h @ w["dkv"].T
    c = lo.rms(dkv[:, :kr], 1e-5) * w["dkv.norm"]
    kr_ = lo.rotate_pairs(dkv[:, kr:], np.arange(T), mx["rot"])
    q = (h @ w["q"].T).reshape(T, H, d + r)
    qr = lo.rotate_pairs(q[..., d:], np.arange(T), mx["rot"])
    out = np.zeros((T, H, dv))
    for n in range(H):
        s = (q[:, n, :d] @ w["uk"][n * d:(n + 1) * d] @ c.T + qr[:, n] @ kr_.T) * mx["scale"]
        s[np.triu_indices(T, 1)] = -np.inf
        p = np.exp(s - s.max(1, keepdims=True))
        out[:, n] = p / p.sum(1, keepdims=True) @ c @ w["uv"][n * dv:(n + 1) * dv].T * lo.sigmoid(h @ w["g"].T)[:, n:n + 1]
    assert np.allclose(lo.latent_attention(h, w, mx, 1e-5), out.reshape(T, -1) @ w["o"].T)


def test_a_sequence_does_not_see_its_future():
    cfg = lc.config([lc.attn(), lc.mem()])
    import __graft_entry__ as graft
    W = lc.Weights(graft.load_package().layered_model.parse_config(cfg))
    t = lc.tokens(12, cfg["vocab"])
    a, b = lo.forward(cfg, W, t), lo.forward(cfg, W, t[:8])
    assert np.allclose(a[:8], b)


# ---- registry, configuration, weights ----
def test_parse_config_reads_every_size_and_constant(pkg):
    hb = pkg.hip_backend
    cfg = lc.config([lc.attn(scaling=lc.YARN, dims=6), lc.mem(cap=7.5, ff=40)], eps=3e-6, mult=0.7)
    p = pkg.layered_model.parse_config(cfg)
    a, m = p.layers
    assert (a.mixer, a.heads, a.dim, a.rot_dim, a.rot_dims, a.vdim, a.kv_rank, a.ff_kind, a.ff) == (hb.MIXER_LATENT_ATTENTION, 3, 24, 8, 6, 20, 40, hb.FF_GEGLU, 72)
    assert (a.yarn_factor, a.yarn_original, a.yarn_fast, a.yarn_slow, a.rot_base) == (4.0, 64.0, 8.0, 1.0, 10000.0)
    assert (m.mixer, m.heads, m.dim, m.vdim, m.gate_cap, m.ff) == (hb.MIXER_MLSTM, 2, 20, 28, 7.5, 40)
    d = p.desc()
    assert (d.width, d.vocab_size, d.norm_eps, d.residual_mult, d.bigram_buckets, d.bigram_mul_prev, d.bigram_mul_cur) == (88, 150, 3e-6, 0.7, 61, 13, 5)
    assert pkg.layered_model.parse_config(lc.config([lc.mem()], bigram=None)).desc().bigram_buckets == 0


@pytest.mark.parametrize("break_it", [
    lambda c: c.update(architecture="Unheard"), lambda c: c.pop("residual_mult"), lambda c: c["layers"][0].update(type="conv"),
    lambda c: c["layers"][0]["mlp"].update(kind="routed"), lambda c: c["layers"][0]["mixer"].pop("kv_rank"),
    lambda c: c["layers"][1]["mixer"].pop("gate_cap")])
def test_unknown_or_incomplete_configurations_are_refused(pkg, break_it):
    c = lc.config([lc.attn(), lc.mem()])
    break_it(c)
    with pytest.raises(pkg.layered_model.ConfigError):
        pkg.layered_model.parse_config(c)


def test_safetensors_folder_round_trip(pkg, tmp_path):
    cfg = lc.config([lc.attn(), lc.mem()])
    W = lc.Weights(pkg.layered_model.parse_config(cfg))
    lc.write_dir(tmp_path, cfg, W)
    model = pkg.LayeredModel.from_dir(str(tmp_path))
    seen = {}
    for name, t, ne, data in model.tensors():
        assert t == 30
        seen[name] = (np.frombuffer(data.tobytes(), "<u2").astype(np.uint32) << 16).view(np.float32).reshape(tuple(reversed(ne)))
    assert seen.keys() == W.keys() and all(np.array_equal(seen[k], W[k]) for k in W)
    del W["l0.mix.uk"]
    lc.write_dir(tmp_path, cfg, W)
    with pytest.raises(pkg.layered_model.ConfigError, match="l0.mix.uk"):
        list(pkg.LayeredModel.from_dir(str(tmp_path)).tensors())


def test_layered_descriptors_match_the_header(pkg):
    import os
    import re
    text = open(os.path.join(os.path.dirname(os.path.dirname(os.path.abspath(__file__))), "include", "llama_gguf_hip.h")).read()
    for struct, cls in (("lgh_layer_desc", pkg.hip_backend.LayerDesc), ("lgh_layered_desc", pkg.hip_backend.LayeredDesc)):
        body = re.search(r"typedef struct %s \{(.*?)\} %s;" % (struct, struct), text, re.S).group(1)
        body = re.sub(r"/\*.*?\*/", "", body, flags=re.S)
        fields = [n.strip() for decl in re.findall(r"(?:uint32_t|uint64_t|int32_t|double)\s+([^;]+);", body) for n in decl.split(",")]
        assert fields == [n for n, _ in cls._fields_]


def test_create_refuses_before_it_touches_a_device(pkg):
    """Sizes no kernel holds and malformed descriptors answer with the reason's status; without a device a good one is NotAvailable."""
    hb = pkg.hip_backend
    parse = pkg.layered_model.parse_config

    def status(cfg, **kw):
        with pytest.raises(pkg.BackendError) as ei:
            hb.HipGpuInference.from_layered(pkg.LayeredModel(parse(cfg), lc.Weights(parse(cfg))), 16, **kw)
        return ei.value.variant
    assert status(lc.config([lc.attn(dims=5)])) == "InvalidArgument"             # an odd number of rotated values
    assert status(lc.config([lc.mem(cap=0.0)])) == "InvalidArgument"
    assert status(lc.config([lc.attn()]), flags=2) == "Unsupported"
    assert status(lc.config([lc.attn(rank=4000, heads=1, dim=1, vdim=1)], width=8)) == "Unsupported"
    if hb.device_count() == 0:
        assert status(lc.config([lc.attn(), lc.mem()])) == "NotAvailable"


def test_trace_steps_reset_between_requests(pkg):
    """The runner's bookkeeping, with a stand-in for the engine: one live request, state given back at its end."""
    class Fake:
        vocab_size = 4

        def __init__(self):
            self.calls = []

        def reset(self):
            self.calls.append("reset")

        def eval(self, toks, want):
            self.calls.append((list(toks), list(want)))
            return np.zeros((len(want), 4), np.float32)
    fake = Fake()
    run = pkg.trace.TraceRunner(fake)
    assert run.step([{"id": "a", "tokens": [1, 2], "want": [1]}], []).shape == (1, 4)
    assert run.step([{"id": "a", "tokens": [3], "want": []}], ["a"]).shape == (0, 4)
    assert run.step([{"id": "a", "tokens": [1], "want": [0]}], []).shape == (1, 4)
    assert fake.calls == ["reset", ([1, 2], [1]), ([3], []), "reset", ([1], [0])]
    with pytest.raises(pkg.BackendError):
        run.step([{"id": "b", "tokens": [1], "want": []}], [])


def test_trace_run_command_line():
    import os
    import subprocess
    import sys
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    exe = os.path.join(root, "bin", "trace_run")
    assert os.access(exe, os.X_OK)
    p = subprocess.run([sys.executable, exe, "--help"], capture_output=True, text=True)
    assert p.returncode == 0 and "--dtype" in p.stdout


def test_bench_sizes_are_models_the_registry_takes(pkg):
    import bench
    for name, sz in bench.LAYERED_SIZES.items():
        cfg = bench.layered_config(sz)
        p = pkg.layered_model.parse_config(cfg).resolve(lambda _: (16, sz["width"]))
        assert p.num_layers == sz["layers"] and {l.mixer for l in p.layers} == {"p": {3}, "w": {1, 2}, "s": {6, 7}, "t": {1, 8, 9}}[name[0]], name
        shapes = dict(p.tensor_shapes())
        t, data = bench.RandomBf16().get("l0.mix.o", (8, 16))
        assert t == 30 and data.size == 128 and shapes["embed" if p.tied_head else "head"] == (sz["vocab"], sz["width"])


# ---- the Pubopel design ----
def test_visible_keys_and_slopes():
    assert lo.visible_keys(3, None) == [0, 1, 2, 3]
    assert lo.visible_keys(9, {"size": 3, "keep_first": 2}) == [0, 1, 7, 8, 9]
    assert lo.visible_keys(2, {"size": 3, "keep_first": 5}) == [0, 1, 2] and lo.visible_keys(4, {"size": 1}) == [4]
    assert lo.head_slope(7, 8) == pytest.approx(2.0 ** -8) and lo.head_slope(0, 8) == 0.5 and lo.head_slope(2, 3) == pytest.approx(2.0 ** -8)


def test_sink_is_one_more_key_without_a_value():
    s = np.array([0.3, -1.0, 2.0])
    e = np.exp(np.append(s, 0.7))
    assert lo.sink_softmax(s, 0.7) == pytest.approx(e[:3] / e.sum())
    assert lo.sink_softmax(s, -np.inf).sum() == pytest.approx(1.0) and lo.sink_softmax(s, 900.0).sum() == pytest.approx(0.0)


def test_soft_cap():
    s = np.array([-1e4, -0.01, 0.0, 0.01, 1e4])
    assert lo.soft_cap(s, 5.0) == pytest.approx([-5.0, -0.01, 0.0, 0.01, 5.0], rel=1e-5) and np.array_equal(lo.soft_cap(s, None), s)


def test_tied_attention_equals_an_explicit_matrix_form():
    """All positions at once with mask matrices, keys normed beforehand, heads repeated over their group."""
    rng = np.random.default_rng(6)
    T, Wd, H, G, d, mx = 13, 21, 6, 2, 5, None
    mx = lc.tied(heads=H, kv_heads=G, dim=d, window=4, keep=2, cap=2.5, scale=0.8)["mixer"]
    shapes = {"q": (H * d, Wd), "k": (G * d, Wd), "q.norm": (H * d,), "k.norm": (G * d,), "temp": (H,), "sink": (H,), "o": (Wd, H * d)}
    w = {k: rng.standard_normal(s) for k, s in shapes.items()}
    h = rng.standard_normal((T, Wd))
    q, k = h @ w["q"].T, h @ w["k"].T
    v = np.repeat(k.reshape(T, G, d), H // G, axis=1)
    n = lambda x, g: x / np.sqrt((x * x).mean(-1, keepdims=True) + 1e-5) * g
    q, kn = n(q, w["q.norm"]).reshape(T, H, d), np.repeat(n(k, w["k.norm"]).reshape(T, G, d), H // G, axis=1)
    s = 2.5 * np.tanh(np.einsum("ihd,jhd->hij", q, kn) * 0.8 * w["temp"][:, None, None] / 2.5)
    dist = np.arange(T)[:, None] - np.arange(T)[None]
    s = s - (2.0 ** (-8.0 * np.arange(1, H + 1) / H))[:, None, None] * dist
    s[:, (dist < 0) | ((dist >= 4) & (np.arange(T)[None] >= 2))] = -np.inf
    e = np.exp(s)
    out = np.einsum("hij,jhd->ihd", e / (e.sum(-1, keepdims=True) + np.exp(w["sink"])[:, None, None]), v)
    assert np.allclose(lo.tied_attention(h, w, mx, 1e-5), out.reshape(T, -1) @ w["o"].T)


def test_mixture_weights_the_experts_input():
    rng = np.random.default_rng(7)
    mlp = lc.moe(experts=5, top=2, ff=6, shared=4)
    w = {"router": rng.standard_normal((5, 8))}
    for n, f in [(f"e{i}", 6) for i in range(5)] + [("shared", 4)]:
        w.update({n + ".gate": rng.standard_normal((f, 8)), n + ".up": rng.standard_normal((f, 8)), n + ".down": rng.standard_normal((8, f))})
    x = rng.standard_normal((3, 8))
    ex = lambda n, v: w[n + ".down"] @ ((w[n + ".gate"] @ v) / (1 + np.exp(-(w[n + ".gate"] @ v))) * (w[n + ".up"] @ v))
    for t in range(3):
        s = 1 / (1 + np.exp(-(w["router"] @ x[t])))
        best = np.argsort(-s)[:2]
        assert np.allclose(lo.moe_ff(x, w, mlp)[t], sum(ex(f"e{e}", s[e] * x[t]) for e in best) + ex("shared", x[t]))
    assert [e for e, _ in lo.route(np.array([1.0, 3.0, 3.0, 2.0]), 3)] == [1, 2, 3]


def test_convolution_and_squashing_norm():
    h = np.array([[1.0, 10.0], [2.0, 20.0], [3.0, 30.0]])
    w = np.array([[1.0, 2.0, 3.0], [0.0, 0.0, 1.0]])
    assert lo.causal_conv(h, w).tolist() == [[3.0, 10.0], [8.0, 20.0], [14.0, 30.0]]
    assert lo.dyt(np.array([0.0, 1e3]), np.array([2.0, 2.0]), np.array([0.5, 0.5]), 0.7).tolist() == [0.5, 2.5]


def test_a_pubopel_sequence_does_not_see_its_future(pkg):
    cfg = lc.sandwich([lc.tied(window=5, mlp=lc.moe()), lc.tied(window=0)], taps=4)
    W = lc.Weights(pkg.layered_model.parse_config(cfg))
    t = lc.tokens(14, cfg["vocab"])
    assert np.allclose(lo.forward(cfg, W, t)[:9], lo.forward(cfg, W, t[:9]))


def test_parse_pubopel_reads_every_size_and_constant(pkg):
    hb = pkg.hip_backend
    cfg = lc.sandwich([lc.tied(heads=9, kv_heads=3, dim=17, window=21, keep=5, scale=0.3, cap=11.0, mlp=lc.moe(7, 3, 19, 23)), lc.tied(window=0, cap=0)], eps=2e-6, taps=5)
    p = pkg.layered_model.parse_config(cfg)
    a, b = p.layers
    assert (a.mixer, a.heads, a.kv_heads, a.dim, a.vdim, a.window, a.keep_first, a.scale, a.score_cap) == (hb.MIXER_TIED_ATTENTION, 9, 3, 17, 17, 21, 5, 0.3, 11.0)
    assert (a.ff_kind, a.experts, a.top, a.ff, a.shared_ff) == (hb.FF_MOE, 7, 3, 19, 23)
    assert (b.window, b.keep_first, b.score_cap, b.ff_kind) == (0, 0, 0.0, hb.FF_NONE)
    d = p.desc()
    assert (d.width, d.vocab_size, d.norm_eps, d.residual_mult, d.residual, d.conv_taps) == (88, 150, 2e-6, 1.0, hb.RESIDUAL_SANDWICH_DYT, 5)
    shapes = dict(p.tensor_shapes())
    assert shapes["l0.norm2b.alpha"] == () and shapes["l0.canon2"] == (88, 5) and shapes["l0.mlp.e6.down"] == (88, 19) and shapes["l0.mix.k.norm"] == (51,)
    assert "l1.norm2" not in shapes and "l1.canon2" not in shapes and "l0.mlp.e7.up" not in shapes and shapes["final.norm.b"] == (88,)


@pytest.mark.parametrize("break_it", [
    lambda c: c.pop("canon"), lambda c: c["canon"].update(taps=0), lambda c: c["layers"][0]["mixer"].pop("kv_heads"), lambda c: c["layers"][0]["mixer"].update(vdim=8),
    lambda c: c["layers"][0]["mixer"].update(kv_heads=4), lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), lambda c: c["layers"][0]["mixer"].pop("scale"),
    lambda c: c["layers"][0]["mlp"].pop("expert"), lambda c: c["layers"][0]["mlp"]["router"].pop("top"), lambda c: c["norm"].pop("eps")])
def test_unusable_pubopel_configurations_are_refused(pkg, break_it):
    c = lc.sandwich([lc.tied(mlp=lc.moe())])
    break_it(c)
    with pytest.raises(pkg.layered_model.ConfigError):
        pkg.layered_model.parse_config(c)


def test_scalars_in_a_model_folder(pkg, tmp_path):
    cfg = lc.sandwich([lc.tied(mlp=lc.moe())])
    W = lc.Weights(pkg.layered_model.parse_config(cfg))
    lc.write_dir(tmp_path, cfg, W)
    got = {name: (ne, data.tobytes()) for name, _, ne, data in pkg.LayeredModel.from_dir(str(tmp_path)).tensors()}
    assert got.keys() == W.keys()
    ne, raw = got["l0.norm1.alpha"]
    assert ne == (1,) and (np.frombuffer(raw, "<u2").astype(np.uint32) << 16).view(np.float32)[0] == W["l0.norm1.alpha"]


def test_create_refuses_unusable_experts_and_heads(pkg):
    hb, parse = pkg.hip_backend, pkg.layered_model.parse_config

    def status(cfg):
        with pytest.raises(pkg.BackendError) as ei:
            hb.HipGpuInference.from_layered(pkg.LayeredModel(parse(cfg), lc.Weights(parse(cfg))), 16)
        return ei.value.variant
    assert status(lc.sandwich([lc.tied(mlp=lc.moe(experts=2, top=3))])) == "InvalidArgument"
    assert status(lc.sandwich([lc.tied(heads=1, kv_heads=1, dim=300)])) == "Unsupported"
    assert status(lc.sandwich([lc.tied(mlp=lc.moe(experts=1, top=1, ff=8, shared=40000))], width=4, vocab=8)) == "Unsupported"
    assert status(lc.sandwich([lc.tied()], taps=65)) == "Unsupported"


# ---- the Sumevik design ----
def _random(shapes, seed):
    rng = np.random.default_rng(seed)
    return {k: rng.standard_normal(s) for k, s in shapes.items()}, rng


def test_linear_recurrence_equals_its_explicit_sum():
    rng = np.random.default_rng(11)
    a, x = rng.random((12, 5)), rng.standard_normal((12, 5))
    S = lo.linear_recurrence(a, x)
    for t in range(12):
        assert np.allclose(S[t], sum(np.prod(a[s + 1: t + 1], axis=0) * x[s] for s in range(t + 1)))


def test_gated_recurrence_step_by_step():
    """One channel block at a time with plain loops: gates, decay, convolution with nothing before the first token."""
    T, W, n, nb, taps = 7, 9, 6, 2, 3
    s = n // nb
    w, rng = _random({"y": (n, W), "y.b": (n,), "x": (n, W), "x.b": (n,), "conv": (n, taps), "conv.b": (n,), "ra": (nb, s, s), "ra.b": (nb, s), "ri": (nb, s, s), "ri.b": (nb, s),
                      "lam": (n,), "o": (W, n)}, 12)
    h = rng.standard_normal((T, W))
    got = lo.rglru(h, w, {"width": n, "blocks": nb, "conv": taps}, 1e-6)
    x = h @ w["x"].T + w["x.b"]
    S, out = np.zeros(n), []
    for t in range(T):
        u = np.array([w["conv.b"][c] + sum(w["conv"][c, taps - 1 - j] * x[t - j, c] for j in range(taps) if t >= j) for c in range(n)])
        for c in range(n):
            k = c // s
            r = 1 / (1 + math.exp(-(w["ra"][k, c % s] @ u[k * s:(k + 1) * s] + w["ra.b"][k, c % s])))
            i = 1 / (1 + math.exp(-(w["ri"][k, c % s] @ u[k * s:(k + 1) * s] + w["ri.b"][k, c % s])))
            a = math.exp(-8 * r * math.log1p(math.exp(w["lam"][c])))
            S[c] = a * S[c] + math.sqrt(1 - a * a) * i * u[c]
        out.append(w["o"] @ (S * lo.gelu_tanh(w["y"] @ h[t] + w["y.b"])))
    assert np.allclose(got, out)


def test_chunks_are_counted_from_the_start():
    assert lo.chunk_keys(7, 4) == [4, 5, 6, 7] and lo.chunk_keys(8, 4) == [8] and lo.chunk_keys(3, 0) == [0, 1, 2, 3] and lo.chunk_keys(5, 1) == [5]


def test_gated_attention_equals_an_explicit_matrix_form():
    T, Wd, H, G, d, dv, size = 11, 17, 4, 2, 6, 5, 4
    mx = lc.gated(heads=H, kv_heads=G, dim=d, vdim=dv, chunk=size, rot=4, base=50.0, scale=0.7)["mixer"]
    w, rng = _random({"q": (H * d, Wd), "q.b": (H * d,), "k": (G * d, Wd), "k.b": (G * d,), "v": (G * dv, Wd), "v.b": (G * dv,), "q.norm": (d,), "k.norm": (d,), "g": (H * dv, Wd),
                      "o": (Wd, H * dv)}, 13)
    h = rng.standard_normal((T, Wd))
    n = lambda x, g: x / np.sqrt((x * x).mean(-1, keepdims=True) + 1e-6) * g
    q = n((h @ w["q"].T + w["q.b"]).reshape(T, H, d), w["q.norm"])
    k = np.repeat(n((h @ w["k"].T + w["k.b"]).reshape(T, G, d), w["k.norm"]), H // G, axis=1)
    v = np.repeat((h @ w["v"].T + w["v.b"]).reshape(T, G, dv), H // G, axis=1)
    turn = np.exp(1j * np.arange(T)[:, None, None] * 50.0 ** (-np.arange(2) / 2.0))          # neighbouring pairs as complex numbers
    rot = lambda x: np.concatenate([np.stack([((x[..., 0:4:2] + 1j * x[..., 1:4:2]) * turn).real, ((x[..., 0:4:2] + 1j * x[..., 1:4:2]) * turn).imag], -1).reshape(T, H, 4), x[..., 4:]], -1)
    s = np.einsum("ihd,jhd->hij", rot(q), rot(k)) * 0.7
    i = np.arange(T)
    s[:, (i[None] > i[:, None]) | (i[None] // size != i[:, None] // size)] = -np.inf
    e = np.exp(s)
    out = np.einsum("hij,jhd->ihd", e / e.sum(-1, keepdims=True), v).reshape(T, -1) / (1 + np.exp(-(h @ w["g"].T)))
    assert np.allclose(lo.gated_attention(h, w, mx, 1e-6), out @ w["o"].T)


def test_gated_linear_attention_equals_its_explicit_sum():
    T, Wd, H, d, dv, rank = 8, 10, 2, 4, 3, 2
    w, rng = _random({"q": (H * d, Wd), "k": (H * d, Wd), "v": (H * dv, Wd), "g": (H * dv, Wd), "o": (Wd, H * dv), "norm": (dv,), "a1": (rank, Wd), "a2": (H * d, rank), "a2.b": (H * d,)}, 14)
    h = rng.standard_normal((T, Wd))
    z = (h @ w["a1"].T @ w["a2"].T + w["a2.b"]).reshape(T, H, d)
    alpha = (1 / (1 + np.exp(-z))) ** (1 / 5.0)
    q, k, v = ((h @ w[n].T).reshape(T, H, -1) for n in "qkv")
    out = np.zeros((T, H, dv))
    for t in range(T):
        for n in range(H):
            for s in range(t + 1):
                out[t, n] += (q[t, n] / 2.0 * np.prod(alpha[s + 1: t + 1, n], axis=0)) @ k[s, n] * v[s, n]
    out = out / np.sqrt((out * out).mean(-1, keepdims=True) + 1e-6) * w["norm"]
    g = h @ w["g"].T
    assert np.allclose(lo.gated_linear_attention(h, w, {"heads": H, "dim": d, "vdim": dv, "tau": 5.0}, 1e-6), (out.reshape(T, -1) * g / (1 + np.exp(-g))) @ w["o"].T)


def test_routing_by_groups():
    s = np.array([0.30, 0.02, 0.25, 0.03, 0.05, 0.35])
    route = lambda c, n, keep, top: lo.route_groups(np.log(s), np.array(c), {"groups": {"count": n, "keep": keep}, "top": top})
    assert [e for e, _ in route([0] * 6, 3, 3, 2)] == [5, 0] and [e for e, _ in route([0] * 6, 3, 1, 2)] == [5, 4]       # the second best lies in a closed group
    assert [e for e, _ in route([-9.0, -9.0, -9.0, -9.0, -8.5, -8.0], 3, 2, 3)] == [5, 4, 0]                              # all negative: closed ones stay out
    (a, wa), (b, wb) = route([0, 0, 0, 5.0, 0, 0], 2, 2, 2)
    assert (a, b) == (3, 5) and wa == pytest.approx(0.03 / 0.38) and wb == pytest.approx(0.35 / 0.38)                     # weights without the correction


def test_identity_experts_and_clamped_experts():
    w, rng = _random({"router": (3, 6), "correction": (3,), "e0.gate": (4, 6), "e0.up": (4, 6), "e0.down": (6, 4)}, 15)
    mlp = {"kind": "moe", "expert": {"ff": 4, "limit": 0.6}, "router": {"experts": 1, "identity": 2, "top": 3, "groups": {"count": 3, "keep": 3}}}
    x = rng.standard_normal((2, 6))
    for t in range(2):
        e = np.exp(w["router"] @ x[t])
        e /= e.sum()
        g, u = np.minimum(w["e0.gate"] @ x[t], 0.6), np.clip(w["e0.up"] @ x[t], -0.6, 0.6)
        assert np.allclose(lo.feed_forward(x, w, mlp)[t], (e[1] + e[2]) * x[t] + e[0] * (w["e0.down"] @ (g / (1 + np.exp(-1.702 * g)) * (u + 1))))


def test_a_sumevik_sequence_does_not_see_its_future(pkg):
    cfg = lc.prenorm([lc.rglru(mlp=lc.grouped()), lc.parallel(mlp=lc.dense())])
    W = lc.Weights(lc.parse(pkg, cfg))
    t = lc.tokens(14, cfg["vocab"])
    assert np.allclose(lo.forward(cfg, W, t)[:9], lo.forward(cfg, W, t[:9]))


def test_parse_sumevik_reads_every_size_and_constant(pkg):
    hb = pkg.hip_backend
    cfg = lc.prenorm([lc.rglru(width=90, blocks=5, taps=3, mlp=lc.grouped(10, 2, 3, 19, (6, 2), 0.7)),
                      lc.parallel(lc.gated(9, 3, 18, 7, 21, 6, 77.0, 0.3), lc.gla(2, 11, 13, 4.0, 5), (0.3, 0.6), lc.dense(31)), lc.rglru()], eps=3e-6, logit_scale=0.25)
    p = lc.parse(pkg, cfg)
    a, b, c = p.layers
    assert (a.mixer, a.heads, a.dim, a.vdim, a.taps) == (hb.MIXER_GLRU, 5, 18, 18, 3)
    assert (a.ff_kind, a.ff, a.experts, a.identity, a.top, a.groups, a.keep_groups, a.expert_limit) == (hb.FF_MOE, 19, 10, 2, 3, 6, 2, 0.7)
    assert (a.router_form, a.expert_form, a.shared_ff) == (hb.ROUTER_SOFTMAX_GROUPS, hb.EXPERT_CLAMPED, 0)
    assert (b.mixer, b.heads, b.kv_heads, b.dim, b.vdim, b.chunk, b.rot_dims, b.rot_base, b.scale) == (hb.MIXER_PARALLEL, 9, 3, 18, 7, 21, 6, 77.0, 0.3)
    assert (b.gla_heads, b.gla_dim, b.gla_vdim, b.gla_tau, b.gla_rank, b.left_scale, b.right_scale, b.ff_kind, b.ff) == (2, 11, 13, 4.0, 5, 0.3, 0.6, hb.FF_GEGLU, 31)
    assert c.ff_kind == hb.FF_NONE
    d = p.desc()
    assert (d.width, d.vocab_size, d.norm_eps, d.residual_mult, d.residual, d.conv_taps, d.tied_head, d.logit_scale) == (88, 150, 3e-6, 1.0, hb.RESIDUAL_PRE_RMS, 0, 1, 0.25)
    s = dict(p.tensor_shapes())
    assert s["l0.mix.ra"] == (5, 18, 18) and s["l0.mix.ri.b"] == (5, 18) and s["l0.mix.conv"] == (90, 3) and s["l0.mlp.router"] == (12, 88) and s["l0.mlp.correction"] == (12,)
    assert s["l0.mlp.e9.down"] == (88, 19) and "l0.mlp.e10.down" not in s and s["l1.mix.left.v.b"] == (21,) and s["l1.mix.left.q.norm"] == (18,) and s["l1.mix.right.a2"] == (22, 5)
    assert s["l1.mix.right.norm"] == (13,) and s["l1.mix.left.o"] == (88, 63) and "head" not in s and "l2.norm2" not in s and "l1.mix.o" not in s
    # the parts of a mixture that another design leaves out
    q = pkg.layered_model.parse_config(lc.prenorm([lc.rglru(mlp={"kind": "moe", "expert": {"ff": 8, "limit": 1.0}, "router": {"experts": 4, "top": 2}})]))
    assert (q.layers[0].groups, q.layers[0].keep_groups, q.layers[0].identity) == (1, 1, 0)


@pytest.mark.parametrize("break_it", [
    lambda c: c.pop("logit_scale"), lambda c: c["norm"].pop("eps"), lambda c: c["layers"][0]["mixer"].update(blocks=7), lambda c: c["layers"][0]["mixer"].update(conv=0),
    lambda c: c["layers"][0]["mixer"].pop("width"), lambda c: c["layers"][1]["mixer"].pop("left_scale"), lambda c: c["layers"][1]["mixer"]["left"].update(kv_heads=4),
    lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=7), lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=40),
    lambda c: c["layers"][1]["mixer"]["left"]["mask"].update(size=0), lambda c: c["layers"][1]["mixer"]["right"].pop("tau"), lambda c: c["layers"][1].update(rank=0),
    lambda c: c["layers"][0]["mlp"]["expert"].pop("limit"), lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(count=5),
    lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(keep=5), lambda c: c["layers"][0]["mlp"]["router"].update(top=7)])
def test_unusable_sumevik_configurations_are_refused(pkg, break_it):
    c = lc.prenorm([lc.rglru(mlp=lc.grouped()), lc.parallel()])
    lc.parse(pkg, c)
    break_it(c)
    with pytest.raises(pkg.layered_model.ConfigError):
        lc.parse(pkg, c)


def test_a_size_that_only_a_tensor_tells(pkg, tmp_path):
    cfg = lc.prenorm([lc.rglru(), lc.parallel(right=lc.gla(rank=7), mlp=lc.grouped())])
    W = lc.Weights(lc.parse(pkg, cfg))
    lc.write_dir(tmp_path, cfg, W)
    m = pkg.LayeredModel.from_dir(str(tmp_path))
    assert m.config.layers[1].gla_rank == 7 and {t[0]: t[2] for t in m.tensors()}["l0.mix.ra"] == (32, 32, 3)
    del W["l1.mix.right.a1"]
    lc.write_dir(tmp_path, cfg, W)
    with pytest.raises(pkg.layered_model.ConfigError, match="right.a1"):
        pkg.LayeredModel.from_dir(str(tmp_path))


def test_create_refuses_unusable_recurrences_and_routers(pkg):
    hb = pkg.hip_backend

    def status(cfg, **change):
        p = lc.parse(pkg, cfg)
        for k, v in change.items():
            setattr(p.layers[0], k, v)
        with pytest.raises(pkg.BackendError) as ei:
            hb.HipGpuInference.from_layered(pkg.LayeredModel(p, {}), 16)
        return ei.value.variant
    assert status(lc.prenorm([lc.rglru(taps=65)])) == "Unsupported"
    assert status(lc.prenorm([lc.rglru()]), vdim=31) == "InvalidArgument"
    assert status(lc.prenorm([lc.gated(heads=1, kv_heads=1, dim=520)])) == "Unsupported"
    assert status(lc.prenorm([lc.gla()]), gla_tau=0.0) == "InvalidArgument"
    assert status(lc.prenorm([lc.rglru(mlp=lc.grouped())]), groups=5) == "InvalidArgument"
    assert status(lc.prenorm([lc.rglru(mlp=lc.grouped())]), router_form=7) == "Unsupported"
    assert status(lc.prenorm([lc.rglru(mlp=lc.grouped(600, 8, 2, 8, None))])) == "Unsupported"
    assert status(lc.config([lc.mem(ff=0) | {"mlp": None}]), ff_kind=2, ff=8, experts=2, top=1, router_form=1, expert_form=1, groups=1, keep_groups=1, identity=1) == "Unsupported"


# ---- the Tarudra design ----
def test_halves_turn_as_complex_numbers():
    rng = np.random.default_rng(21)
    x, rot = rng.standard_normal((5, 2, 9)), {"dims": 6, "base": 30.0}
    got = lo.rotate_halves(x, np.arange(5), rot)
    z = (x[..., :3] + 1j * x[..., 3:6]) * np.exp(1j * np.arange(5)[:, None, None] * 30.0 ** (-np.arange(3) / 3.0))
    assert np.allclose(got[..., :3], z.real) and np.allclose(got[..., 3:6], z.imag) and np.array_equal(got[..., 6:], x[..., 6:])
    assert np.allclose(lo.rotate_pairs(x[..., [0, 3, 1, 4, 2, 5]], np.arange(5), rot)[..., 0::2], z.real)       # the same rotation, other neighbours


def test_grouped_attention_equals_an_explicit_matrix_form():
    T, Wd, H, G, d, dv, size = 11, 17, 4, 2, 6, 5, 4
    mx = lc.grouped_attn(H, G, d, dv, size, 4, 50.0, scale=0.7)["mixer"]
    w, rng = _random({"q": (H * d, Wd), "q.b": (H * d,), "k": (G * d, Wd), "k.b": (G * d,), "v": (G * dv, Wd), "v.b": (G * dv,), "o": (Wd, H * dv), "o.b": (Wd,)}, 22)
    h, other = rng.standard_normal((T, Wd)), rng.standard_normal((T, Wd))
    turn = np.exp(1j * np.arange(T)[:, None, None] * 50.0 ** (-np.arange(2) / 2.0))

    def rot(x):
        z = (x[..., 0:4:2] + 1j * x[..., 1:4:2]) * turn
        return np.concatenate([np.stack([z.real, z.imag], -1).reshape(T, x.shape[1], 4), x[..., 4:]], -1)
    for src in (h, other):                       # its own keys and values, and another layer's
        k = np.repeat(rot((src @ w["k"].T + w["k.b"]).reshape(T, G, d)), H // G, axis=1)
        v = np.repeat((src @ w["v"].T + w["v.b"]).reshape(T, G, dv), H // G, axis=1)
        s = np.einsum("ihd,jhd->hij", rot((h @ w["q"].T + w["q.b"]).reshape(T, H, d)), k) * 0.7
        i = np.arange(T)
        e = np.where((i[None] <= i[:, None]) & (i[:, None] - i[None] < size), np.exp(s), 0.0)
        out = np.einsum("hij,jhd->ihd", e / (1.0 + e.sum(-1, keepdims=True)), v).reshape(T, -1)
        assert np.allclose(lo.grouped_attention(h, w, mx, lo.grouped_keys_values(src, w, mx)), out @ w["o"].T + w["o.b"])


def test_windowed_latent_attention_equals_an_explicit_matrix_form():
    T, Wd, H, d, r, dv, kr, qr, size = 10, 13, 3, 4, 4, 5, 6, 7, 3
    mx = lc.latent2(H, d, r, dv, kr, qr, size, 0.6, 40.0)["mixer"]
    w, rng = _random({"dq": (qr, Wd), "dq.norm": (qr,), "uq": (H * (d + r), qr), "dkv": (kr + r, Wd), "dkv.norm": (kr,), "uk": (H * d, kr), "uv": (H * dv, kr), "g": (H * dv, Wd),
                      "o": (Wd, H * dv)}, 23)
    h = rng.standard_normal((T, Wd))
    n = lambda x, g: x / np.sqrt((x * x).mean(-1, keepdims=True) + 1e-6) * g
    q = (n(h @ w["dq"].T, w["dq.norm"]) @ w["uq"].T).reshape(T, H, d + r)
    c, kr_part = n(h @ w["dkv"][:kr].T, w["dkv.norm"]), h @ w["dkv"][kr:].T
    turn = np.exp(1j * np.arange(T)[:, None] * 40.0 ** (-np.arange(2) / 2.0))
    rot = lambda x: (x[..., :2] + 1j * x[..., 2:]) * (turn if x.ndim == 2 else turn[:, None])
    s = np.einsum("ihd,jhd->hij", q[..., :d], (c @ w["uk"].T).reshape(T, H, d)) + np.einsum("ihd,jd->hij", rot(q[..., d:]), rot(kr_part).conj()).real
    i = np.arange(T)
    e = np.where((i[None] <= i[:, None]) & (i[:, None] - i[None] < size), np.exp(0.6 * s), 0.0)
    out = np.einsum("hij,jhd->ihd", e / e.sum(-1, keepdims=True), (c @ w["uv"].T).reshape(T, H, dv)).reshape(T, -1) / (1 + np.exp(-(h @ w["g"].T)))
    assert np.allclose(lo.windowed_latent_attention(h, w, mx, 1e-6), out @ w["o"].T)


def test_delta_rule_equals_one_linear_system():
    """The written rows solve (I + L) U = B V for the whole sequence; outputs are decayed scores times them."""
    T, Wd, H, G, d, dv, taps = 9, 12, 4, 2, 5, 3, 3
    w, rng = _random({"q": (G * d, Wd), "k": (G * d, Wd), "v": (H * dv, Wd), "q.conv": (G * d, taps), "k.conv": (G * d, taps), "v.conv": (H * dv, taps), "b": (H, Wd), "a": (H, Wd),
                      "A_log": (H,), "dt_bias": (H,), "norm": (dv,), "g": (H * dv, Wd), "o": (Wd, H * dv)}, 24)
    h = rng.standard_normal((T, Wd))

    def short(n):
        x = np.concatenate([np.zeros((taps - 1, w[n].shape[0])), h @ w[n].T])
        y = sum(x[j:j + T] * w[n + ".conv"][:, j] for j in range(taps))
        return y / (1 + np.exp(-y))
    unit = lambda x: x / np.sqrt((x * x).sum(-1, keepdims=True) + 1e-6)
    q, k, v = unit(short("q").reshape(T, G, d)) / math.sqrt(d), unit(short("k").reshape(T, G, d)), short("v").reshape(T, H, dv)
    beta = 1 / (1 + np.exp(-(h @ w["b"].T)))
    ld = np.cumsum(-np.exp(w["A_log"]) * np.log1p(np.exp(h @ w["a"].T + w["dt_bias"])), axis=0)
    out = np.zeros((T, H, dv))
    for n in range(H):
        dec = np.tril(np.exp(np.minimum(ld[:, None, n] - ld[None, :, n], 0.0)))
        kn, qn = k[:, n // 2], q[:, n // 2]
        U = np.linalg.solve(np.eye(T) + beta[:, n, None] * np.tril(dec * (kn @ kn.T), -1), beta[:, n, None] * v[:, n])
        out[:, n] = (dec * (qn @ kn.T)) @ U
    out = out / np.sqrt((out * out).mean(-1, keepdims=True) + 1e-5) * w["norm"]
    g = h @ w["g"].T
    mx = {"heads": H, "kv_heads": G, "dim": d, "vdim": dv}
    assert np.allclose(lo.delta_rule(h, w, mx, 1e-5), (out.reshape(T, -1) * g / (1 + np.exp(-g))) @ w["o"].T)


def test_squared_relu_and_capped_logits(pkg):
    w, rng = _random({"up": (5, 4), "down": (4, 5)}, 25)
    x = rng.standard_normal((3, 4))
    z = x @ w["up"].T
    assert np.allclose(lo.squared_relu_ff(x, w), np.where(z > 0, z * z, 0) @ w["down"].T)
    cfg = lc.sandwich_ln([lc.grouped_attn()], cap=0.7)
    W = lc.Weights(lc.parse(pkg, cfg))
    o = lo.forward(cfg, W, lc.tokens(5, cfg["vocab"]))
    wide = lo.forward(dict(cfg, logit_softcap=1e9), W, lc.tokens(5, cfg["vocab"]))
    assert np.abs(o).max() < 0.7 and np.allclose(o, 0.7 * np.tanh(wide / 0.7))


def test_a_tarudra_sequence_does_not_see_its_future(pkg):
    cfg = lc.sandwich_ln([lc.grouped_attn(window=4, mlp=lc.dense()), lc.delta(), lc.latent2(window=5), lc.grouped_attn(window=6, source=0)])
    W = lc.Weights(lc.parse(pkg, cfg))
    t = lc.tokens(14, cfg["vocab"])
    assert np.allclose(lo.forward(cfg, W, t)[:9], lo.forward(cfg, W, t[:9]))


def test_a_reader_sees_the_cache_of_its_source(pkg):
    """The source's keys and values decide, not the reader's input; the reader's window is its own."""
    cfg = lc.sandwich_ln([lc.grouped_attn(window=2), lc.grouped_attn(window=5, source=0)])
    W = lc.Weights(lc.parse(pkg, cfg))
    assert "l1.mix.k" not in W and "l1.mix.v.b" not in W and "l1.mix.o.b" in W
    t = lc.tokens(9, cfg["vocab"])
    base = lo.forward(cfg, W, t)[-1]
    for far, seen in ((4, True), (3, False)):              # the last token is 8: its widest window is 4 .. 8
        u = list(t)
        u[far] = (u[far] + 1) % cfg["vocab"]
        assert np.allclose(lo.forward(cfg, W, u)[-1], base) != seen


def test_parse_tarudra_reads_every_size_and_constant(pkg):
    hb = pkg.hip_backend
    cfg = lc.sandwich_ln([lc.grouped_attn(9, 3, 18, 7, 21, 6, 77.0, dict(factor=3.0, original=50, fast=9.0, slow=2.0), 0.3, mlp=lc.dense(31)), lc.delta(6, 2, 11, 13, 3),
                          lc.grouped_attn(9, 3, 18, 7, 40, 6, 77.0, dict(factor=3.0, original=50, fast=9.0, slow=2.0), 0.2, source=0), lc.latent2(5, 12, 6, 9, 17, 23, 33, 0.4, 88.0, 4, mlp=lc.dense(8)),
                          lc.latent2(window=0, rotate=False), lc.grouped_attn(window=0, rot=0)], eps=3e-6, cap=12.5)
    p = pkg.layered_model.parse_config(cfg)
    a, b, c, e, f, g = p.layers
    assert (a.mixer, a.heads, a.kv_heads, a.dim, a.vdim, a.window, a.rot_dims, a.rot_base, a.scale, a.sink_one, a.kv_from) == (hb.MIXER_GROUPED_ATTENTION, 9, 3, 18, 7, 21, 6, 77.0, 0.3, 1, 0)
    assert (a.yarn_factor, a.yarn_original, a.yarn_fast, a.yarn_slow, a.ff_kind, a.ff) == (3.0, 50.0, 9.0, 2.0, hb.FF_RELU2, 31)
    assert (b.mixer, b.heads, b.kv_heads, b.dim, b.vdim, b.taps, b.ff_kind) == (hb.MIXER_DELTA, 6, 2, 11, 13, 3, hb.FF_NONE)
    assert (c.kv_from, c.window, c.scale) == (1, 40, 0.2)
    assert (e.mixer, e.heads, e.dim, e.rot_dim, e.vdim, e.kv_rank, e.q_rank, e.window, e.scale, e.rot_base, e.rot_dims) == (hb.MIXER_LATENT_ATTENTION, 5, 12, 6, 9, 17, 23, 33, 0.4, 88.0, 4)
    assert (e.rot_form, e.gate_form, e.yarn_factor) == (hb.ROT_HALVES, hb.GATE_VALUES, 0.0) and (f.window, f.rot_dims, g.window, g.rot_dims) == (0, 0, 0, 0)
    d = p.desc()
    assert (d.width, d.vocab_size, d.norm_eps, d.residual_mult, d.residual, d.tied_head, d.logit_cap) == (88, 150, 3e-6, 1.0, hb.RESIDUAL_SANDWICH_LN, 0, 12.5)
    s = dict(p.tensor_shapes())
    assert s["l0.mix.v.b"] == (21,) and s["l0.mix.o"] == (88, 63) and s["l0.mix.o.b"] == (88,) and s["l0.mlp.up"] == (31, 88) and "l0.mlp.gate" not in s and s["l0.ls2"] == (88,)
    assert s["l1.mix.v.conv"] == (78, 3) and s["l1.mix.q"] == (22, 88) and s["l1.mix.b"] == (6, 88) and s["l1.mix.dt_bias"] == (6,) and s["l1.mix.norm"] == (13,) and "l1.ls2" not in s
    assert "l2.mix.k" not in s and s["l2.mix.q"] == (162, 88) and s["l3.mix.uq"] == (90, 23) and s["l3.mix.dkv"] == (23, 88) and s["l3.mix.g"] == (45, 88) and s["l3.norm2b"] == (88,)
    assert "l3.mix.q" not in s and "head" in s


@pytest.mark.parametrize("break_it", [
    lambda c: c.pop("logit_softcap"), lambda c: c.update(logit_softcap=0.0), lambda c: c["norm"].pop("eps"), lambda c: c["layers"][0]["mixer"].pop("kv_heads"),
    lambda c: c["layers"][0]["mixer"].update(kv_heads=4), lambda c: c["layers"][0]["mixer"].pop("scale"), lambda c: c["layers"][0]["mixer"]["mask"].update(size=0),
    lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7), lambda c: c["layers"][0]["mixer"]["rot"].update(dims=40), lambda c: c["layers"][0]["mixer"]["rot"].update(scaling={"factor": 2.0}),
    lambda c: c["layers"][1]["mixer"].pop("conv"), lambda c: c["layers"][1]["mixer"].update(conv=0), lambda c: c["layers"][1]["mixer"].update(kv_heads=3),
    lambda c: c["layers"][2]["mixer"].update(kv_from=1), lambda c: c["layers"][2]["mixer"].update(kv_from=2), lambda c: c["layers"][2]["mixer"].update(kv_from=3),
    lambda c: c["layers"][2]["mixer"].update(kv_from=-1), lambda c: c["layers"][2]["mixer"].update(dim=30), lambda c: c["layers"][2]["mixer"]["rot"].update(base=5.0),
    lambda c: c["layers"][3]["mixer"].pop("q_rank"), lambda c: c["layers"][3]["mixer"].update(q_rank=0), lambda c: c["layers"][3]["mixer"]["rot"].update(dims=10),
    lambda c: c["layers"][3]["mixer"]["mask"].pop("size"), lambda c: c["layers"][0].update(type="mamba"), lambda c: c["layers"][0]["mlp"].update(kind="moe")])
def test_unusable_tarudra_configurations_are_refused(pkg, break_it):
    c = lc.sandwich_ln([lc.grouped_attn(mlp=lc.dense()), lc.delta(), lc.grouped_attn(source=0), lc.latent2()])
    pkg.layered_model.parse_config(c)
    break_it(c)
    with pytest.raises(pkg.layered_model.ConfigError):
        pkg.layered_model.parse_config(c)


def test_create_refuses_unusable_delta_rules_and_shared_keys(pkg):
    hb, parse = pkg.hip_backend, pkg.layered_model.parse_config

    def status(cfg, layer=0, **change):
        p = parse(cfg)
        for k, v in change.items():
            setattr(p.layers[layer], k, v)
        with pytest.raises(pkg.BackendError) as ei:
            hb.HipGpuInference.from_layered(pkg.LayeredModel(p, {}), 16)
        return ei.value.variant
    two = lc.sandwich_ln([lc.grouped_attn(), lc.grouped_attn(source=0)])
    assert status(lc.sandwich_ln([lc.delta(taps=65)])) == "Unsupported"
    assert status(lc.sandwich_ln([lc.delta()]), kv_heads=3) == "InvalidArgument"
    assert status(lc.sandwich_ln([lc.delta()]), taps=0) == "InvalidArgument"
    assert status(lc.sandwich_ln([lc.grouped_attn(heads=1, kv_heads=1, dim=520)])) == "Unsupported"
    assert status(two, 1, kv_from=2) == "InvalidArgument" and status(two, 1, kv_from=9) == "InvalidArgument" and status(two, 1, dim=16) == "InvalidArgument"
    assert status(lc.prenorm([lc.gated()]), sink_one=1) == "Unsupported" and status(lc.prenorm([lc.gated(), lc.gated()]), 1, kv_from=1) == "Unsupported"
    assert status(lc.sandwich_ln([lc.latent2()]), rot_form=2) == "Unsupported" and status(lc.sandwich_ln([lc.latent2()]), gate_form=2) == "Unsupported"
    assert status(lc.sandwich_ln([lc.grouped_attn(mlp=lc.dense())]), ff_kind=2, experts=2, top=1) == "Unsupported"
