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
        p = pkg.layered_model.parse_config(cfg)
        assert p.num_layers == sz["layers"] and {l.mixer for l in p.layers} == {1, 2}, name
        shapes = dict(p.tensor_shapes())
        t, data = bench.RandomBf16().get("l0.mix.o", (8, 16))
        assert t == 30 and data.size == 128 and shapes["head"] == (sz["vocab"], sz["width"])
