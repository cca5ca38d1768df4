"""GPU: models described layer by layer against the plain restatement (oracle/layered.py), through the C ABI.

f32 contexts are the sharp test (differences of rounding only); bf16 contexts are held to bf16 rounding of operands.  Prompts, single
tokens, portions and resets must all agree with ONE whole-sequence run of the oracle."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import layered_cases as lc
from oracle import layered as lo

pytestmark = pytest.mark.gpu
TOL, DTYPES, make, check, stepwise = lc.TOL, lc.DTYPES, lc.make, lc.check, lc.stepwise


# every mechanism alone, and sizes at and around the kernels' granules: 1, not a multiple of 4 / 16 / 32 / 64, above a tile
SHAPES = {
    "attention": [lc.attn(ff=0)],
    "attention one head": [lc.attn(heads=1, dim=1, rot=2, vdim=1, rank=1, ff=0)],
    "attention 17 heads": [lc.attn(heads=17, dim=8, rot=4, vdim=6, rank=18, ff=0)],
    "attention rank 130": [lc.attn(heads=2, dim=100, rot=28, vdim=130, rank=130, ff=0)],
    "attention rank 530": [lc.attn(heads=2, dim=33, rot=6, vdim=65, rank=530, ff=0)],
    "attention wide head": [lc.attn(heads=2, dim=250, rot=22, vdim=260, rank=64, ff=0)],
    "attention long rotated part": [lc.attn(heads=2, dim=16, rot=96, vdim=32, rank=48, ff=0)],
    "attention yarn": [lc.attn(rot=32, scaling=lc.YARN, ff=0)],
    "attention partly rotated": [lc.attn(rot=12, dims=4, base=50.0, ff=0)],
    "attention not rotated": [lc.attn(rotate=False, ff=0)],
    "attention sharp": [lc.attn(heads=4, scale=3.0, ff=0)],
    "memory": [lc.mem()],
    "memory one": [lc.mem(heads=1, dim=1, vdim=1)],
    "memory 130": [lc.mem(heads=3, dim=130, vdim=70)],
    "memory 260": [lc.mem(heads=1, dim=260, vdim=17)],
    "memory 520": [lc.mem(heads=1, dim=520, vdim=530)],
    "memory odd": [lc.mem(heads=5, dim=13, vdim=9, cap=2.0)],
    "memory with feed-forward": [lc.mem(ff=50)],
    "feed-forward": [lc.attn(ff=129)],
    "two rotations": [lc.attn(scaling=lc.YARN), lc.attn(base=300.0, heads=2, rot=4)],
    "mixed": [lc.mem(), lc.attn(scaling=lc.YARN), lc.attn(heads=4, rank=33), lc.mem(heads=3), lc.mem(), lc.attn()],
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(SHAPES))
def test_prompt_and_decode_match_the_oracle(pkg, gpu, name, dtype):
    if name in ("attention one head",) and dtype == "bf16":
        dtype = "f32"                               # one value per head: the layer norm divides by what rounding leaves of it
    print(name, dtype, flush=True)
    cfg = lc.config(SHAPES[name], width=88 if "wide" not in name else 301, bigram=None if name == "attention" else (61, 13, 5))
    eng, W = make(pkg, cfg, dtype)
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
    check(stepwise(eng, toks[:40]), want[:40], dtype, "token by token")
    eng.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_portions_of_any_size_agree(pkg, gpu, dtype):
    """Cuts at and around multiples of the kernels' tiles (32 keys, 64-token chunks, 64-token path switch), down to two tokens."""
    cfg = lc.config(SHAPES["mixed"])
    eng, W = make(pkg, cfg, dtype, max_seq=400)
    toks = lc.tokens(330, cfg["vocab"], 5)
    want = lo.forward(cfg, W, toks)
    for cuts in ([2] * 20, [3, 1, 2, 1, 5], [63, 1, 64, 2], [64, 64, 64], [65, 63, 129], [31, 33, 2, 30], [200, 2, 100], [1, 2, 127, 3, 128, 2]):
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
def test_far_keys_and_tile_borders(pkg, gpu, dtype):
    """One key stands out for one query: the query at the end and a single token far back match in a direction nothing else has.  The
    result must move with that token's value wherever it lies, and must not see one position too many."""
    lay = lc.attn(heads=2, dim=32, rot=8, vdim=32, rank=64, ff=0)
    cfg = lc.config([lay, lc.mem()], width=96, vocab=120, bigram=None)
    parsed = pkg.layered_model.parse_config(cfg)
    W = lc.Weights(parsed, 3)
    Q, KA, KB = 117, 118, 119                       # the asking token, and two keys that answer differently
    for t in (Q, KA, KB):
        W["embed"][t] = lc.bf16(W["embed"][t] * 0.3)
    W["embed"][:, :3] = 0.0
    W["embed"][Q, 0] = 6.0                          # the question's direction, the keys' direction, and what they answer
    W["embed"][[KA, KB], 2] = 6.0
    W["embed"][KA, 1], W["embed"][KB, 1] = 5.0, -5.0
    W["l0.mix.dkv"][:, :3] = 0.0
    W["l0.mix.dkv"][0, 2] = 4.0                     # the latent's first value carries the keys' direction, its second the answer
    W["l0.mix.dkv"][1, 1] = 4.0
    W["l0.mix.dkv.norm"][:2] = 1.0
    W["l0.mix.uk"][0, :] = 0.0
    W["l0.mix.uk"][0, 0] = 4.0
    W["l0.mix.q"][0, :] = 0.0
    W["l0.mix.q"][0, 0] = 4.0
    eng, _ = make(pkg, cfg, dtype, max_seq=1200, weights=W)
    base = [t % 110 for t in lc.tokens(1100, 110, 9)]
    for n in (33, 65, 129, 1025, 1060):
        for far in (0, 1, 31, 32, 63, 64, n - 34, n - 33, n - 3):
            if not 0 <= far < n - 1:
                continue
            ends = {}
            for key in (KA, KB):
                toks = list(base[:n])
                toks[far], toks[n - 1] = key, Q
                if n < 200 or key == KA:
                    want = lo.forward(cfg, W, toks)[n - 1:]
                    eng.reset()
                    check(eng.eval(toks, [n - 1]), want, dtype, f"prompt, key {far} of {n}")
                    ends[key] = want
                eng.reset()
                eng.eval(toks[:n - 1])
                got = eng.forward(Q)[None]
                if key in ends:
                    check(got, ends[key], dtype, f"decoded, key {far} of {n}")
                ends.setdefault(key, got)
            assert lc.row_error(ends[KA], ends[KB]).max() > 0.05, f"the key at {far} of {n} makes no difference"
    eng.close()


def test_long_decode_and_memory_that_lasts(pkg, gpu):
    """600 decoded tokens; forget gates near 1, so that tokens hundreds of steps back still count."""
    cfg = lc.config([lc.mem(heads=2, dim=32, vdim=32), lc.attn(heads=2), lc.mem(heads=1, dim=16, vdim=48)], mult=0.8)
    W = lc.Weights(pkg.layered_model.parse_config(cfg), 7)
    for i in (0, 2):
        W[f"l{i}.mix.f.b"][:] = 9.5
        W[f"l{i}.mix.f"] *= 0.25
    toks = lc.tokens(640, cfg["vocab"], 11)
    want = lo.forward(cfg, W, toks)
    other = list(toks)
    other[2] = (other[2] + 1) % cfg["vocab"]
    assert lc.row_error(lo.forward(cfg, W, other)[-1:], want[-1:]).max() > 1e-3      # the third token is remembered
    eng, _ = make(pkg, cfg, "f32", max_seq=640, weights=W)
    check(np.concatenate([eng.eval(toks[:40], range(40)), stepwise(eng, toks[40:])]), want, "f32", "long decode")
    eng.reset()
    check(eng.eval(toks, range(640)), want, "f32", "the same as one prompt")
    eng.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_prompts_longer_than_one_block(pkg, gpu, dtype):
    """The block path takes 2048 tokens at a time: the border inside one call, and a second long portion after it."""
    cfg = lc.config([lc.mem(heads=1, dim=16, vdim=16), lc.attn(heads=2, dim=16, rot=8, vdim=16, rank=32, ff=0)], width=40, vocab=64)
    W = lc.Weights(pkg.layered_model.parse_config(cfg), 13)
    W["l0.mix.f.b"][:] = 8.0
    toks = lc.tokens(2400, cfg["vocab"], 15)
    want = lo.forward(cfg, W, toks)
    eng, _ = make(pkg, cfg, dtype, max_seq=2400, weights=W)
    places = list(range(2020, 2080)) + [2299]
    check(eng.eval(toks[:2300], places), want[places], dtype, "one call")
    check(eng.eval(toks[2300:2390], range(90)), want[2300:2390], dtype, "the next portion")
    check(stepwise(eng, toks[2390:]), want[2390:], dtype, "decoded")
    eng.close()


def test_first_tokens_and_the_pair_embedding(pkg, gpu):
    """The first token has a pair row of its own; the previous token crosses portion and decode boundaries; products above 2^31."""
    cfg = lc.config([lc.attn(heads=1)], vocab=4000, bigram=(1013, 3000017, 2000003))
    eng, W = make(pkg, cfg, "f32", max_seq=64)
    toks = [3999, 3999, 0, 0, 3998, 1, 3999, 7]
    want = lo.forward(cfg, W, toks)
    for cuts in ([8], [1] * 8, [2, 1, 3, 2], [1, 7]):
        eng.reset()
        at, rows = 0, []
        for n in cuts:
            rows.append(eng.eval(toks[at:at + n], range(n)))
            at += n
        check(np.concatenate(rows), want, "f32", f"cuts {cuts}")
    eng.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_reset_forgets_everything(pkg, gpu, dtype):
    """A sequence after others is bit for bit the sequence in a fresh context: cache rows, states and the previous token are left over
    but not read."""
    cfg = lc.config(SHAPES["mixed"])
    eng, W = make(pkg, cfg, dtype, max_seq=200)
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
    fresh, _ = make(pkg, cfg, dtype, max_seq=200)
    assert np.array_equal(run(fresh, b), first)
    fresh.reset()
    assert np.array_equal(fresh.forward(b[0]), one)
    eng.close()
    fresh.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_graph_replays_equal_eager_launches(pkg, gpu, dtype):
    cfg = lc.config(SHAPES["mixed"])
    eng, W = make(pkg, cfg, dtype)
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
    cfg = lc.config([lc.mem(), lc.attn(scaling=lc.YARN), lc.attn(heads=2)], vocab=97)
    eng, W = make(pkg, cfg, "f32", max_seq=120)
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
    cfg = lc.config(SHAPES["mixed"])
    toks = lc.tokens(140, cfg["vocab"], 51)
    ref = None
    for kw in (dict(flags=pkg.hip_backend.FLAG_EXACT_PREFILL), dict(attn_splits=1), dict(attn_splits=7), dict(attn_splits=128)):
        eng, W = make(pkg, cfg, "f32", **kw)
        ref = lo.forward(cfg, W, toks) if ref is None else ref
        assert eng.prefill_is_batched() == ("flags" not in kw)
        check(np.concatenate([eng.eval(toks[:90], range(90)), stepwise(eng, toks[90:])]), ref, "f32", str(kw))
        eng.close()


def test_refusals_leave_the_sequence_intact(pkg, gpu):
    cfg = lc.config([lc.attn(), lc.mem()])
    eng, W = make(pkg, cfg, "f32", max_seq=24)
    toks = lc.tokens(24, cfg["vocab"], 61)
    want = lo.forward(cfg, W, toks)
    eng.eval(toks[:20])

    def refused(f, variant):
        with pytest.raises(pkg.BackendError) as ei:
            f()
        assert ei.value.variant == variant and eng.position() == 20
    refused(lambda: eng.eval(toks[:5]), "InvalidArgument")                  # past max_seq_len
    refused(lambda: eng.eval([1, cfg["vocab"]]), "InvalidArgument")         # no such token
    refused(lambda: eng.eval(toks[20:22], [1, 0]), "InvalidArgument")       # places must ascend
    refused(lambda: eng.eval(toks[20:22], [2]), "InvalidArgument")
    refused(lambda: eng.kv_truncate(10), "Unsupported")                     # a recurrence cannot go back
    refused(lambda: eng.kv_shift_left(4), "Unsupported")
    refused(lambda: eng.batch_create(2), "Unsupported")
    refused(lambda: eng.stage_prefill_batch(toks[:2], 2), "Unsupported")
    check(eng.eval(toks[20:], range(4)), want[20:], "f32", "after the refusals")
    with pytest.raises(pkg.BackendError):
        eng.forward(1)
    eng.kv_truncate(0)
    check(eng.eval(toks, range(24)), want, "f32", "after a truncation to nothing")
    eng.close()
    eng, W = make(pkg, lc.config([lc.attn(), lc.attn()]), "f32", max_seq=64)   # attention alone can go back
    t = lc.tokens(40, 150, 62)
    want = lo.forward(lc.config([lc.attn(), lc.attn()]), W, t[:10] + t[20:])
    eng.eval(t[:20])
    eng.kv_truncate(10)
    check(eng.eval(t[20:], range(20)), want[10:], "f32", "after a truncation")
    eng.close()


def test_missing_and_misshapen_tensors_are_named(pkg, gpu):
    cfg = lc.config([lc.attn()])
    parsed = pkg.layered_model.parse_config(cfg)
    W = lc.Weights(parsed)

    class Short(pkg.LayeredModel):
        def tensors(self):
            return (t for t in super().tensors() if t[0] != "l0.mlp.up")
    with pytest.raises(pkg.BackendError, match="l0.mlp.up"):
        pkg.HipGpuInference.from_layered(Short(parsed, W), 16)

    class Wrong(pkg.LayeredModel):
        def tensors(self):
            return ((n, t, ne if n != "l0.mix.o" else ne[::-1], d) for n, t, ne, d in super().tensors())
    with pytest.raises(pkg.BackendError, match="l0.mix.o"):
        pkg.HipGpuInference.from_layered(Wrong(parsed, W), 16)


@pytest.mark.parametrize("dtype", DTYPES)
def test_bench_like_sizes(pkg, gpu, dtype):
    """Sizes a real layer has (latent 512 + 64, 128-wide heads, memories of 256 x 512 and 512 x 64), against the oracle."""
    cfg = lc.config([lc.attn(heads=5, dim=128, rot=64, vdim=128, rank=512, ff=700), lc.mem(heads=2, dim=256, vdim=512), lc.mem(heads=1, dim=512, vdim=64)],
                    width=640, vocab=300)
    eng, W = make(pkg, cfg, dtype, max_seq=320)
    toks = lc.tokens(280, cfg["vocab"], 71)
    want = lo.forward(cfg, W, toks)
    check(np.concatenate([eng.eval(toks[:200], range(200)), eng.eval(toks[200:220], range(20)), stepwise(eng, toks[220:])]), want, dtype)
    eng.close()


def test_trace_run_program(pkg, gpu, tmp_path):
    """bin/trace_run on a model folder: steps in, logits out, two requests one after the other, both number formats."""
    cfg = lc.config([lc.mem(), lc.attn(scaling=lc.YARN)])
    W = lc.Weights(pkg.layered_model.parse_config(cfg), 5)
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
        assert not (out / "1.f32").exists()
        check(rows(0), A[[0, 5, 19]], dtype)
        check(rows(2), A[[22]], dtype)
        check(rows(3), B, dtype)
