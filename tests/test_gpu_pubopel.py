"""GPU: the Pubopel design (windowed attention whose values are its keys, mixtures of experts, squashing norms around every sublayer, a short
causal convolution in front of it) against the plain restatement (oracle/layered.py), through the C ABI.

f32 contexts are the sharp test; bf16 contexts are held to bf16 rounding of operands, with routing that rests on no close call.  Prompts,
single tokens, portions and resets must all agree with ONE whole-sequence run of the oracle."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import layered_cases as lc
from oracle import layered as lo

pytestmark = pytest.mark.gpu
DTYPES, make, check, stepwise = lc.DTYPES, lc.make, lc.check, lc.stepwise


def engine(pkg, cfg, dtype, **kw):
    """bf16: routing without close calls where the model routes."""
    W = kw.pop("weights", None)
    if W is None:
        W = lc.Weights(pkg.layered_model.parse_config(cfg), kw.pop("seed", 0))
        if dtype == "bf16" and any(lay["mlp"] for lay in cfg["layers"]):
            lc.clear_calls(W, cfg)
    return make(pkg, cfg, dtype, weights=W, **kw)


# every mechanism alone, sizes at and around the kernels' granules, and sizes that another model of the design might have
CASES = {
    "attention": dict(layers=[lc.tied()]),
    "attention, no mask": dict(layers=[lc.tied(window=0)]),
    "attention, no cap": dict(layers=[lc.tied(cap=0)]),
    "attention, nothing kept": dict(layers=[lc.tied(keep=0, window=17)]),
    "attention, tight cap": dict(layers=[lc.tied(cap=0.7, scale=1.5)]),
    "window of one": dict(layers=[lc.tied(window=1, keep=1)]),
    "window of two, none kept": dict(layers=[lc.tied(window=2, keep=0)]),
    "kept beyond the window": dict(layers=[lc.tied(window=20, keep=70)]),
    "one head of one value": dict(layers=[lc.tied(heads=1, kv_heads=1, dim=1)]),
    "as many key heads as heads": dict(layers=[lc.tied(heads=5, kv_heads=5, dim=40)]),
    "eleven heads on one": dict(layers=[lc.tied(heads=11, kv_heads=1, dim=72)]),
    "groups of seven": dict(layers=[lc.tied(heads=14, kv_heads=2, dim=33)]),
    "heads of 64": dict(layers=[lc.tied(heads=4, kv_heads=1, dim=64)]),
    "heads of 128": dict(layers=[lc.tied(heads=4, kv_heads=4, dim=128, window=100, keep=9)]),
    "heads of 136": dict(layers=[lc.tied(heads=2, kv_heads=1, dim=136)]),
    "heads of 256": dict(layers=[lc.tied(heads=2, kv_heads=2, dim=256)]),
    "one tap": dict(layers=[lc.tied()], taps=1),
    "two taps": dict(layers=[lc.tied()], taps=2),
    "four taps": dict(layers=[lc.tied()], taps=4),
    "nine taps": dict(layers=[lc.tied()], taps=9),
    "twenty taps": dict(layers=[lc.tied()], taps=20),
    "odd width": dict(layers=[lc.tied(mlp=lc.moe(ff=33, shared=17))], width=301, vocab=77),
    "mixture": dict(layers=[lc.tied(mlp=lc.moe())]),
    "one expert": dict(layers=[lc.tied(mlp=lc.moe(experts=1, top=1))]),
    "top one, nothing shared": dict(layers=[lc.tied(mlp=lc.moe(experts=7, top=1, shared=0))]),
    "every expert": dict(layers=[lc.tied(mlp=lc.moe(experts=5, top=5, ff=65))]),
    "many experts": dict(layers=[lc.tied(mlp=lc.moe(experts=70, top=6, ff=16, shared=130))]),
    "wide": dict(layers=[lc.tied(heads=10, kv_heads=2, dim=64, mlp=lc.moe(experts=4, top=2, ff=200, shared=300))], width=640),
    "mixed": dict(layers=[lc.tied(mlp=lc.moe()), lc.tied(heads=3, kv_heads=1, dim=20, window=9, keep=0, cap=5.0),
                          lc.tied(heads=4, kv_heads=4, dim=70, window=0, mlp=lc.moe(experts=9, top=3, ff=20, shared=0)),
                          lc.tied(window=64, keep=64, mlp=lc.moe(top=1))], taps=4),
}


def case(name):
    return lc.sandwich(**CASES[name])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(CASES))
def test_prompt_and_decode_match_the_oracle(pkg, gpu, name, dtype):
    print(name, dtype, flush=True)
    cfg = case(name)
    eng, W = engine(pkg, cfg, dtype)
    toks = lc.tokens(150, cfg["vocab"])
    layers = []
    want = lo.forward(cfg, W, toks, layers)
    eng.set_layer_tap(True)
    got = eng.eval(toks, range(len(toks)))
    tap = eng.read_layers(len(toks))
    eng.set_layer_tap(False)
    for i, x in enumerate(layers):   # the residual stream after every layer
        d = np.sort(np.abs(tap[i] - x).max(1) / np.abs(x).max())
        assert (d[-1] <= 1e-5 if dtype == "f32" else d[-7] <= 3e-2), f"layer {i}: {d[-7:]}"
    check(got, want, dtype, "whole prompt")
    eng.reset()
    check(stepwise(eng, toks[:60]), want[:60], dtype, "token by token")
    eng.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_portions_of_any_size_agree(pkg, gpu, dtype):
    """Cuts at and around multiples of the kernels' tiles (16 tokens: the decode kernel's portions; 32 / 64 keys; 64 / 128 queries), down to two
    tokens, and single tokens between them: the convolutions' inputs cross every border."""
    cfg = case("mixed")
    eng, W = engine(pkg, cfg, dtype, max_seq=400)
    toks = lc.tokens(330, cfg["vocab"], 5)
    want = lo.forward(cfg, W, toks)
    for cuts in ([2] * 20, [3, 1, 2, 1, 5], [16, 17, 15, 2, 16], [63, 1, 64, 2], [64, 64, 64], [65, 63, 129], [31, 33, 2, 30], [200, 2, 100],
                 [1, 2, 127, 3, 128, 2]):
        eng.reset()
        at, rows = 0, []
        for n in list(cuts) + [330]:
            n = min(n, 330 - at)
            if n:
                rows.append(eng.eval(toks[at:at + n], range(n)))
                at += n
        check(np.concatenate(rows), want, dtype, f"portions {cuts}")
    # prompt, then decoding through the replayed graph, then another portion
    eng.reset()
    rows = [eng.eval(toks[:100], range(100)), stepwise(eng, toks[100:170]), eng.eval(toks[170:174], range(4)), stepwise(eng, toks[174:180]),
            eng.eval(toks[180:300], range(120)), stepwise(eng, toks[300:330])]
    check(np.concatenate(rows), want, dtype, "portions and decoding in turn")
    eng.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window,keep,n", [(50, 3, 140), (64, 64, 200), (63, 1, 130), (129, 5, 300), (40, 33, 75), (1, 2, 20), (200, 0, 260)])
def test_a_key_just_inside_and_just_outside(pkg, gpu, dtype, window, keep, n):
    """One key stands out for the last token's query.  Where it is visible (inside the window, among the kept ones) its value must decide the
    logits, one position further it must not matter at all, in a prompt and in decoding; the oracle says which is which."""
    cfg = lc.sandwich([lc.tied(heads=2, kv_heads=1, dim=16, window=window, keep=keep, scale=1.0, cap=60.0)], width=96, vocab=120)
    W = lc.Weights(pkg.layered_model.parse_config(cfg), 3)
    Q, KA, KB = 117, 118, 119                       # the asking token, and two keys that answer differently
    for t in (Q, KA, KB):
        W["embed"][t] = 0.0
    W["embed"][:, :3] = 0.0
    W["embed"][Q, 0] = 3.0                          # the question's direction, the keys' direction, and what they answer
    W["embed"][[KA, KB], 2] = 3.0
    W["embed"][KA, 1], W["embed"][KB, 1] = 3.0, -3.0
    W["l0.norm1"][:3], W["l0.norm1.b"][:3], W["l0.canon1"][:3] = 1.0, 0.0, 0.0
    W["l0.norm1.b"][:] = lc.bf16(W["l0.norm1.b"] * 0.1)   # (what all tokens share would drown the question)
    W["l0.mix.q"][:, 0] = 0.0
    W["l0.mix.q"][16, :] = 0.0
    W["l0.mix.q"][16, 0] = 8.0                      # head 1 (the one that minds distance least) asks in its first value
    W["l0.mix.q.norm"][16] = 4.0
    W["l0.mix.k"][0, :] = 0.0
    W["l0.mix.k"][0, 2] = 8.0                       # the key's first value carries the direction, its second the answer
    W["l0.mix.k"][1, :] = 0.0
    W["l0.mix.k"][1, 1] = 8.0
    W["l0.mix.k.norm"][:2] = 4.0, 0.0
    W["l0.mix.temp"][:] = 1.0
    W["l0.mix.sink"][:] = 0.5
    eng, _ = make(pkg, cfg, dtype, max_seq=320, weights=W)
    base = [t % 110 for t in lc.tokens(n, 110, 9)]
    last = n - 1
    places = {0, keep - 1, keep, last - window + 1, last - window, last - window - 1, last - 1, 31, 32, 63, 64}
    seen_some = hidden_some = False
    for far in sorted(p for p in places if 0 <= p < last):
        ends = []
        for key in (KA, KB):
            toks = list(base)
            toks[far], toks[last] = key, Q
            want = lo.forward(cfg, W, toks)[last:]
            eng.reset()
            check(eng.eval(toks, [last]), want, dtype, f"prompt, key {far} of {n}")
            eng.reset()
            eng.eval(toks[:last])
            check(eng.forward(Q)[None], want, dtype, f"decoded, key {far} of {n}")
            ends.append(want)
        visible = last - far < window or far < keep
        moved = lc.row_error(ends[0], ends[1]).max()
        assert moved > 0.05 if visible else moved < (1e-9 if last - far > 2 else 1.0), f"key {far} of {n}: {moved}"
        seen_some, hidden_some = seen_some or visible, hidden_some or not visible
    assert seen_some and hidden_some
    eng.close()


def test_each_constant_of_the_attention_shows(pkg, gpu):
    """The engine follows the oracle when one thing changes, and each change moves the logits: sinks, temperatures, norm weights, kept
    tokens, the window by one, the cap, the scale, the convolution, a norm's factor, the shared expert, the router."""
    lay = lambda **kw: lc.tied(window=24, keep=2, cap=3.0, scale=0.4, **kw)
    cfg = lc.sandwich([lay(mlp=lc.moe()), lay()])
    toks = lc.tokens(60, cfg["vocab"], 8)
    W = lc.Weights(pkg.layered_model.parse_config(cfg), 4)
    W["l0.mix.sink"][:] = 4.0
    ref = lo.forward(cfg, W, toks)

    def run(c, w, what):
        eng, _ = make(pkg, c, "f32", weights=w)
        want = lo.forward(c, w, toks)
        assert what is None or lc.row_error(want, ref).max() > 1e-3, f"{what} changes nothing"
        check(eng.eval(toks, range(60)), want, "f32", f"prompt: {what}")
        eng.reset()
        check(stepwise(eng, toks), want, "f32", f"steps: {what}")
        eng.close()
    run(cfg, W, None)
    for name in ("l0.mix.sink", "l0.mix.temp", "l0.mix.q.norm", "l1.mix.k.norm", "l0.norm1.alpha", "l0.norm1b.alpha", "l1.norm1.b", "l0.canon1", "l0.canon2",
                 "l0.mlp.shared.down", "l0.mlp.router", "l0.norm2b.b", "final.norm.alpha", "final.norm.b"):
        w = lc.Weights(pkg.layered_model.parse_config(cfg), 4)
        w["l0.mix.sink"][:] = 4.0
        w[name] = lc.bf16(w[name] * -0.5 + 0.1)
        run(cfg, w, name)
    for key, value in (("softcap", 0.5), ("scale", 0.9), ("mask", {"size": 25, "keep_first": 2}), ("mask", {"size": 24, "keep_first": 3}), ("mask", None)):
        c = json.loads(json.dumps(cfg))
        c["layers"][0]["mixer"][key] = value
        run(c, W, f"{key} {value}")


def test_long_decode(pkg, gpu):
    """700 decoded tokens: the window passes over decoded tokens many times, kept tokens stay at their true distance."""
    cfg = lc.sandwich([lc.tied(heads=4, kv_heads=2, window=50, keep=4, mlp=lc.moe()), lc.tied(heads=2, kv_heads=1, window=0)], taps=5)
    eng, W = engine(pkg, cfg, "f32", max_seq=740, seed=7)
    toks = lc.tokens(740, cfg["vocab"], 11)
    want = lo.forward(cfg, W, toks)
    check(np.concatenate([eng.eval(toks[:40], range(40)), stepwise(eng, toks[40:])]), want, "f32", "long decode")
    eng.reset()
    check(eng.eval(toks, range(740)), want, "f32", "the same as one prompt")
    eng.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_prompts_longer_than_one_block(pkg, gpu, dtype):
    """The block path takes 2048 tokens at a time: the border inside one call, and a second long portion after it."""
    cfg = lc.sandwich([lc.tied(heads=2, kv_heads=1, dim=16, window=300, keep=4, mlp=lc.moe(experts=3, top=1, ff=16, shared=0)),
                       lc.tied(heads=2, kv_heads=1, dim=16, window=0)], width=40, vocab=64, taps=4)
    eng, W = engine(pkg, cfg, dtype, max_seq=2400, seed=13)
    toks = lc.tokens(2400, cfg["vocab"], 15)
    want = lo.forward(cfg, W, toks)
    places = list(range(2020, 2080)) + [2299]
    check(eng.eval(toks[:2300], places), want[places], dtype, "one call")
    check(eng.eval(toks[2300:2390], range(90)), want[2300:2390], dtype, "the next portion")
    check(stepwise(eng, toks[2390:]), want[2390:], dtype, "decoded")
    eng.close()


def test_first_tokens(pkg, gpu):
    """Nothing lies before a sequence's first token, however its first portions are cut, also right after another sequence."""
    cfg = lc.sandwich([lc.tied(mlp=lc.moe(top=1)), lc.tied()], taps=6)
    eng, W = engine(pkg, cfg, "f32", max_seq=64)
    toks = lc.tokens(9, cfg["vocab"], 17)
    want = lo.forward(cfg, W, toks)
    for cuts in ([9], [1] * 9, [2, 1, 3, 3], [1, 8], [1, 1, 7], [5, 4]):
        eng.reset()
        eng.eval(lc.tokens(23, cfg["vocab"], 18))
        eng.reset()
        at, rows = 0, []
        for n in cuts:
            rows.append(eng.eval(toks[at:at + n], range(n)))
            at += n
        check(np.concatenate(rows), want, "f32", f"cuts {cuts}")
    eng.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_reset_forgets_everything(pkg, gpu, dtype):
    """A sequence after others is bit for bit the sequence in a fresh context: cache rows, key factors and the convolutions' inputs are left
    over but not read."""
    cfg = case("mixed")
    eng, W = engine(pkg, cfg, dtype, max_seq=200)
    a, b = lc.tokens(150, cfg["vocab"], 21), lc.tokens(90, cfg["vocab"], 22)
    run = lambda e, t: np.concatenate([e.eval(t[:70], range(70)), stepwise(e, t[70:])])
    first = run(eng, b)
    eng.reset()
    run(eng, a)
    eng.decode_greedy(3, 20)
    eng.reset()
    assert np.array_equal(run(eng, b), first)
    eng.reset()
    one = eng.forward(b[0])                          # a sequence that starts with a single token
    fresh, _ = make(pkg, cfg, dtype, max_seq=200, weights=W)
    assert np.array_equal(run(fresh, b), first)
    fresh.reset()
    assert np.array_equal(fresh.forward(b[0]), one)
    eng.close()
    fresh.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_graph_replays_equal_eager_launches(pkg, gpu, dtype):
    cfg = case("mixed")
    eng, W = engine(pkg, cfg, dtype)
    eager, _ = make(pkg, cfg, dtype, flags=pkg.hip_backend.FLAG_NO_GRAPH, weights=W)
    toks = lc.tokens(60, cfg["vocab"], 31)
    for i, t in enumerate(toks):
        assert np.array_equal(eng.forward(t), eager.forward(t)), f"token {i}"
        if i % 20 == 19:                             # the engine's own eager work between replays
            eng.eval(toks[:3])
            eager.eval(toks[:3])
            eng.synchronize()
    eng.close()
    eager.close()


def test_greedy_generation_through_the_engine(pkg, gpu):
    """GpuModelWrapper + decode_greedy (token fed back on the device) against the oracle's arg-max, token by token; and stepwise."""
    cfg = lc.sandwich([lc.tied(window=12, mlp=lc.moe()), lc.tied(heads=4, kv_heads=1, window=0, mlp=lc.moe(top=1, shared=0))], vocab=97)
    eng, W = engine(pkg, cfg, "f32", max_seq=120)
    prompt = lc.tokens(17, cfg["vocab"], 41)
    wrap, ctx = pkg.GpuModelWrapper(eng), pkg.InferenceContext()
    logits = wrap.forward(prompt, ctx)
    first = int(np.flatnonzero(logits == logits.max())[-1])
    out = eng.decode_greedy(first, 50).tolist()
    seq = prompt + [first] + out
    want = lo.forward(cfg, W, seq[:-1])
    for i, tok in enumerate(seq[len(prompt):]):
        row = want[len(prompt) - 1 + i]
        top = np.sort(row)[::-1]
        assert tok == int(row.argmax()) or top[0] - row[tok] < 1e-4, f"generated token {i}"
    eng.reset()
    eng.forward_batch(prompt[:-1])                   # the block path, then one token at a time
    tok, again = prompt[-1], []
    for _ in range(51):
        tok = eng.forward_argmax(tok)
        again.append(tok)
    assert again == [first] + out
    assert eng.position() == len(prompt) + 50
    eng.close()


def test_exact_prefill_flag_and_split_counts(pkg, gpu):
    cfg = case("mixed")
    toks = lc.tokens(140, cfg["vocab"], 51)
    ref = None
    for kw in (dict(flags=pkg.hip_backend.FLAG_EXACT_PREFILL), dict(attn_splits=1), dict(attn_splits=3), dict(attn_splits=128)):
        eng, W = engine(pkg, cfg, "f32", **kw)
        ref = lo.forward(cfg, W, toks) if ref is None else ref
        assert eng.prefill_is_batched() == ("flags" not in kw)
        check(np.concatenate([eng.eval(toks[:90], range(90)), eng.eval(toks[90:101], range(11)), stepwise(eng, toks[101:])]), ref, "f32", str(kw))
        eng.close()


def test_parts_combine_with_the_other_design(pkg, gpu):
    """Mixers and feed-forwards are shared between designs: mixtures and tied attention under layer norm on the sublayers' outputs, latent
    attention, matrix memories and dense feed-forwards between squashing norms."""
    for cfg in (lc.config([lc.tied(mlp=lc.moe()), lc.mem(), lc.tied(mlp=lc.moe(top=3, shared=0)), dict(lc.attn(), mlp=lc.moe(top=1))]),
                lc.sandwich([lc.attn(), lc.mem(), lc.tied(mlp=lc.moe()), dict(lc.mem(), mlp=lc.moe(shared=0)), lc.mem(ff=50)])):
        eng, W = engine(pkg, cfg, "f32", max_seq=120, seed=3)
        toks = lc.tokens(110, cfg["vocab"], 55)
        want = lo.forward(cfg, W, toks)
        check(np.concatenate([eng.eval(toks[:80], range(80)), stepwise(eng, toks[80:105]), eng.eval(toks[105:], range(5))]), want, "f32", cfg["architecture"])
        eng.close()


def test_refusals_leave_the_sequence_intact(pkg, gpu):
    cfg = lc.sandwich([lc.tied(mlp=lc.moe())])
    eng, W = engine(pkg, cfg, "f32", max_seq=24)
    toks = lc.tokens(24, cfg["vocab"], 61)
    want = lo.forward(cfg, W, toks)
    eng.eval(toks[:20])

    def refused(f, variant):
        with pytest.raises(pkg.BackendError) as ei:
            f()
        assert ei.value.variant == variant and eng.position() == 20
    refused(lambda: eng.eval(toks[:5]), "InvalidArgument")                  # past max_seq_len
    refused(lambda: eng.eval([1, cfg["vocab"]]), "InvalidArgument")         # no such token
    refused(lambda: eng.kv_truncate(10), "Unsupported")                     # the convolutions' earlier inputs are gone
    refused(lambda: eng.kv_shift_left(4), "Unsupported")
    refused(lambda: eng.batch_create(2), "Unsupported")
    check(eng.eval(toks[20:], range(4)), want[20:], "f32", "after the refusals")
    eng.kv_truncate(0)
    check(eng.eval(toks, range(24)), want, "f32", "after a truncation to nothing")
    eng.close()

    class Short(pkg.LayeredModel):
        def tensors(self):
            return (t for t in super().tensors() if t[0] != "l0.mlp.e4.up")
    with pytest.raises(pkg.BackendError, match="l0.mlp.e4.up"):
        pkg.HipGpuInference.from_layered(Short(pkg.layered_model.parse_config(cfg), W), 16)


@pytest.mark.parametrize("dtype", DTYPES)
def test_bench_like_sizes(pkg, gpu, dtype):
    """Sizes a real layer has, against the oracle: 128-wide heads, groups of four, a window of several tiles, experts of several hundred."""
    cfg = lc.sandwich([lc.tied(heads=8, kv_heads=2, dim=128, window=150, keep=4, cap=50.0, mlp=lc.moe(experts=12, top=4, ff=320, shared=700))],
                      width=1024, vocab=300, taps=4)
    eng, W = engine(pkg, cfg, dtype, max_seq=320)
    toks = lc.tokens(280, cfg["vocab"], 71)
    want = lo.forward(cfg, W, toks)
    check(np.concatenate([eng.eval(toks[:200], range(200)), eng.eval(toks[200:220], range(20)), stepwise(eng, toks[220:])]), want, dtype)
    eng.close()


def test_trace_run_program(pkg, gpu, tmp_path):
    """bin/trace_run on a model folder: steps in, logits out, two requests one after the other, both number formats."""
    cfg = lc.sandwich([lc.tied(window=10, mlp=lc.moe()), lc.tied()])
    W = lc.clear_calls(lc.Weights(pkg.layered_model.parse_config(cfg), 5), cfg)
    (tmp_path / "m").mkdir()
    lc.write_dir(tmp_path / "m", cfg, W)
    a, b = lc.tokens(30, cfg["vocab"], 81), lc.tokens(12, cfg["vocab"], 82)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:20], "want": [0, 5, 19]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[20:22], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[22:23], "want": [0]}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "b", "tokens": b, "want": list(range(12))}], "end": ["b"]}]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    A, B = lo.forward(cfg, W, a), lo.forward(cfg, W, b)
    for dtype, name in (("f32", "float32"), ("bf16", "bfloat16")):
        out = tmp_path / name
        out.mkdir()
        p = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", str(tmp_path / "m"), "--dtype", name, "--out", str(out),
                            "--max-tokens", "30"], input="\n".join(map(json.dumps, steps)) + "\n", capture_output=True, text=True, timeout=100)
        assert p.returncode == 0, p.stderr[-2000:]
        assert [ln for ln in p.stdout.splitlines() if ln.startswith("done")] == ["done 0", "done 1", "done 2", "done 3"]
        rows = lambda n: np.fromfile(out / f"{n}.f32", "<f4").reshape(-1, cfg["vocab"])
        check(rows(0), A[[0, 5, 19]], dtype)
        check(rows(2), A[[22]], dtype)
        check(rows(3), B, dtype)
