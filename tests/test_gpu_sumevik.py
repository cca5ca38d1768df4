"""GPU: the Sumevik design (gated linear recurrences, gated chunked attention beside gated linear attention, grouped mixtures with identity experts,
RMS norms in front of the sublayers, the embedding table as output projection) against the plain restatement (oracle/layered.py), through the C ABI.

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
        W = lc.Weights(lc.parse(pkg, cfg), kw.pop("seed", 0))
        if dtype == "bf16":
            lc.clear_calls_prenorm(W, cfg)
    return make(pkg, cfg, dtype, weights=W, **kw)


# every mechanism alone, sizes at and around the kernels' granules, and sizes that another model of the design might have
CASES = {
    "recurrence": dict(layers=[lc.rglru()]),
    "recurrence, one tap": dict(layers=[lc.rglru(taps=1)]),
    "recurrence, two taps": dict(layers=[lc.rglru(taps=2)]),
    "recurrence, three taps": dict(layers=[lc.rglru(taps=3)]),
    "recurrence, five taps": dict(layers=[lc.rglru(taps=5)]),
    "recurrence, nineteen taps": dict(layers=[lc.rglru(taps=19)]),
    "recurrence, one block": dict(layers=[lc.rglru(width=130, blocks=1)]),
    "recurrence, blocks of one": dict(layers=[lc.rglru(width=11, blocks=11)]),
    "recurrence, blocks of 64": dict(layers=[lc.rglru(width=320, blocks=5)]),
    "recurrence, blocks of 65": dict(layers=[lc.rglru(width=195, blocks=3)]),
    "recurrence, blocks of 320": dict(layers=[lc.rglru(width=640, blocks=2)]),
    "recurrence, blocks of 18": dict(layers=[lc.rglru(width=90, blocks=5)]),
    "attention": dict(layers=[lc.gated()]),
    "attention, no chunks": dict(layers=[lc.gated(chunk=0)]),
    "attention, no rotation": dict(layers=[lc.gated(rot=0)]),
    "attention, all rotated": dict(layers=[lc.gated(dim=24, rot=24)]),
    "chunks of one": dict(layers=[lc.gated(chunk=1)]),
    "chunks of two": dict(layers=[lc.gated(chunk=2)]),
    "chunks of 64": dict(layers=[lc.gated(chunk=64)]),
    "one head of one value": dict(layers=[lc.gated(heads=1, kv_heads=1, dim=1, vdim=1, rot=0)]),
    "odd heads": dict(layers=[lc.gated(heads=5, kv_heads=5, dim=33, vdim=41)]),
    "eleven heads on one": dict(layers=[lc.gated(heads=11, kv_heads=1, dim=72, vdim=40)]),
    "groups of seven": dict(layers=[lc.gated(heads=14, kv_heads=2, dim=34, vdim=70)]),
    "heads of 64": dict(layers=[lc.gated(heads=4, kv_heads=2, dim=64, vdim=64, rot=32)]),
    "keys of 64, values of 256": dict(layers=[lc.gated(heads=2, kv_heads=1, dim=64, vdim=256)]),
    "keys of 200, values of 8": dict(layers=[lc.gated(heads=3, kv_heads=3, dim=200, vdim=8)]),
    "keys of 256, values of 192": dict(layers=[lc.gated(heads=2, kv_heads=2, dim=256, vdim=192)]),
    "keys of 16, values of 330": dict(layers=[lc.gated(heads=2, kv_heads=1, dim=16, vdim=330)]),
    "keys of 16, values of 450": dict(layers=[lc.gated(heads=4, kv_heads=1, dim=16, vdim=450)]),
    "keys of 300, values of 31": dict(layers=[lc.gated(heads=3, kv_heads=1, dim=300, vdim=31)]),
    "linear attention": dict(layers=[lc.gla()]),
    "linear attention, one of one": dict(layers=[lc.gla(heads=1, dim=1, vdim=1, rank=1)]),
    "linear attention, rank 40": dict(layers=[lc.gla(heads=2, dim=64, vdim=64, rank=40)]),
    "linear attention, keys of 130": dict(layers=[lc.gla(heads=2, dim=130, vdim=33, rank=16)]),
    "linear attention, keys of 300": dict(layers=[lc.gla(heads=1, dim=300, vdim=20, rank=3)]),
    "linear attention, keys of 530": dict(layers=[lc.gla(heads=1, dim=530, vdim=20, rank=3)]),
    "linear attention, tau 1": dict(layers=[lc.gla(tau=1.0)]),
    "parallel": dict(layers=[lc.parallel()]),
    "parallel, one side weak": dict(layers=[lc.parallel(scales=(1.0, -0.1))]),
    "parallel, odd": dict(layers=[lc.parallel(lc.gated(heads=3, kv_heads=1, dim=22, vdim=13, chunk=9, rot=2), lc.gla(heads=5, dim=9, vdim=7, rank=5, tau=2.0))], width=77, vocab=61),
    "dense": dict(layers=[lc.rglru(mlp=lc.dense(100))]),
    "mixture": dict(layers=[lc.rglru(mlp=lc.grouped())]),
    "mixture, no identity": dict(layers=[lc.rglru(mlp=lc.grouped(8, 0, 2, 33, (4, 3)))]),
    "mixture, no groups": dict(layers=[lc.rglru(mlp=lc.grouped(7, 2, 3, 24, None))]),
    "mixture, groups of one": dict(layers=[lc.rglru(mlp=lc.grouped(5, 2, 2, 24, (7, 3)))]),
    "mixture, one group open": dict(layers=[lc.rglru(mlp=lc.grouped(10, 2, 3, 24, (3, 1)))]),
    "mixture, everything chosen": dict(layers=[lc.rglru(mlp=lc.grouped(3, 3, 6, 24, (2, 2)))]),
    "mixture, mostly identity": dict(layers=[lc.rglru(mlp=lc.grouped(2, 10, 4, 24, (4, 3)))]),
    "mixture, one expert": dict(layers=[lc.rglru(mlp=lc.grouped(1, 0, 1, 24, (1, 1)))]),
    "mixture, many experts": dict(layers=[lc.rglru(mlp=lc.grouped(60, 12, 6, 16, (8, 3), 0.4))]),
    "mixture, wide limit": dict(layers=[lc.rglru(mlp=lc.grouped(limit=50.0))]),
    "odd width": dict(layers=[lc.rglru(mlp=lc.grouped(ff=33)), lc.parallel(mlp=lc.dense(50))], width=301, vocab=77),
    "wide": dict(layers=[lc.parallel(lc.gated(heads=10, kv_heads=2, dim=64, vdim=64, rot=32), lc.gla(4, 64, 32, rank=16), mlp=lc.grouped(6, 2, 2, 200, (4, 2)))], width=640),
    "mixed": dict(layers=[lc.rglru(mlp=lc.dense()), lc.parallel(mlp=lc.grouped()), lc.rglru(width=60, blocks=2, taps=3),
                          lc.parallel(lc.gated(4, 4, 30, 18, 17, 10), lc.gla(2, 40, 36, 2.0, 20), (1.5, 0.4), lc.grouped(5, 1, 2, 20, (2, 2))), lc.rglru(mlp=lc.grouped(top=1))],
                  logit_scale=0.6),
}


def case(name):
    return lc.prenorm(**CASES[name])


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
    check(stepwise(eng, toks[:70]), want[:70], dtype, "token by token")
    eng.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_portions_of_any_size_agree(pkg, gpu, dtype):
    """Cuts at and around multiples of the kernels' tiles (16 tokens: the decode kernel's portions; 32 / 64 keys, the recurrences' chunks of 64
    tokens; 64 / 128 queries), inside attention's chunks and at their edges, down to two tokens, and single tokens between them."""
    cfg = case("mixed")
    eng, W = engine(pkg, cfg, dtype, max_seq=400)
    toks = lc.tokens(330, cfg["vocab"], 5)
    want = lo.forward(cfg, W, toks)
    for cuts in ([2] * 20, [3, 1, 2, 1, 5], [16, 17, 15, 2, 16], [39, 2, 39, 1, 40], [63, 1, 64, 2], [64, 64, 64], [65, 63, 129], [31, 33, 2, 30], [200, 2, 100],
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
@pytest.mark.parametrize("chunk,n", [(50, 140), (64, 200), (63, 130), (129, 300), (40, 79), (40, 80), (40, 81), (2, 20), (1, 9), (0, 260)])
def test_a_key_just_inside_and_just_outside(pkg, gpu, dtype, chunk, n):
    """One key stands out for the last token's query.  In the query's own chunk its value must decide the logits, one position before the chunk it
    must not matter at all, in a prompt, in decoding and at the start of a portion; the oracle says which is which."""
    cfg = lc.prenorm([lc.gated(heads=2, kv_heads=1, dim=16, vdim=12, chunk=chunk, rot=6, scale=1.0)], width=96, vocab=120)
    W = lc.Weights(lc.parse(pkg, cfg), 3)
    Q, KA, KB = 117, 118, 119                       # the asking token, and two keys that answer differently
    for t in (Q, KA, KB):
        W["embed"][t] = 0.0
    W["embed"][:, :3] = 0.0
    W["embed"][Q, 0] = 3.0                          # the question's direction, the keys' direction, and what they answer
    W["embed"][[KA, KB], 2] = 3.0
    W["embed"][KA, 1], W["embed"][KB, 1] = 3.0, -3.0
    W["l0.norm1"][:3] = 0.0
    for name in ("q", "k", "v"):
        W[f"l0.mix.{name}.b"][:] = 0.0
    W["l0.mix.q"][[8, 24], :] = 0.0
    W["l0.mix.q"][[8, 24], 0] = 8.0                 # both heads ask in a value that is not rotated
    W["l0.mix.q.norm"][8] = W["l0.mix.k.norm"][8] = 3.0
    W["l0.mix.k"][8, :] = 0.0
    W["l0.mix.k"][8, 2] = 8.0
    W["l0.mix.v"][0, :] = 0.0
    W["l0.mix.v"][0, 1] = 4.0
    eng, _ = make(pkg, cfg, dtype, max_seq=320, weights=W)
    base = [t % 110 for t in lc.tokens(n, 110, 9)]
    last = n - 1
    start = last // chunk * chunk if chunk else 0
    places = {0, 1, start - 2, start - 1, start, start + 1, last - 1, 31, 32, 63, 64}
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
            if last - far >= 3:
                eng.reset()
                eng.eval(toks[:last - 1])
                check(eng.eval(toks[last - 1:], [1]), want, dtype, f"a portion of two, key {far} of {n}")
            ends.append(want)
        moved = lc.row_error(ends[0], ends[1]).max()
        assert moved > 0.05 if far >= start else moved < 1e-9, f"key {far} of {n}: {moved}"
    eng.close()


def test_each_constant_and_weight_shows(pkg, gpu):
    """The engine follows the oracle when one thing changes, and each change moves the logits."""
    par = lambda **kw: lc.parallel(lc.gated(chunk=24, scale=0.4), lc.gla(), **kw)
    cfg = lc.prenorm([lc.rglru(mlp=lc.grouped()), par(mlp=lc.dense())])
    toks = lc.tokens(60, cfg["vocab"], 8)
    W = lc.Weights(lc.parse(pkg, cfg), 4)
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
    for name in ("l0.norm1", "l0.norm2", "final.norm", "l0.mix.y.b", "l0.mix.x.b", "l0.mix.conv", "l0.mix.conv.b", "l0.mix.ra", "l0.mix.ra.b", "l0.mix.ri", "l0.mix.ri.b", "l0.mix.lam",
                 "l0.mlp.correction", "l0.mlp.router", "l1.mix.left.q.b", "l1.mix.left.k.b", "l1.mix.left.v.b", "l1.mix.left.q.norm", "l1.mix.left.k.norm", "l1.mix.left.g",
                 "l1.mix.right.g", "l1.mix.right.norm", "l1.mix.right.a1", "l1.mix.right.a2", "l1.mix.right.a2.b", "l1.mix.right.o", "l1.mlp.up"):
        w = lc.Weights(lc.parse(pkg, cfg), 4)
        w[name] = lc.bf16(w[name][..., ::-1] * -0.5 + 0.1)
        run(cfg, w, name)
    mixer = lambda c, i: c["layers"][i]["mixer"]
    for what, change in (("left_scale", lambda c: mixer(c, 1).update(left_scale=0.2)), ("right_scale", lambda c: mixer(c, 1).update(right_scale=0.2)),
                         ("scale", lambda c: mixer(c, 1)["left"].update(scale=0.9)), ("chunk", lambda c: mixer(c, 1)["left"]["mask"].update(size=25)),
                         ("no chunks", lambda c: mixer(c, 1)["left"].pop("mask")), ("rotation base", lambda c: mixer(c, 1)["left"]["rot"].update(base=10.0)),
                         ("rotated values", lambda c: mixer(c, 1)["left"]["rot"].update(dims=4)), ("tau", lambda c: mixer(c, 1)["right"].update(tau=3.0)),
                         ("limit", lambda c: c["layers"][0]["mlp"]["expert"].update(limit=0.3)), ("open groups", lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(keep=1)),
                         ("groups", lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(count=2)), ("logit_scale", lambda c: c.update(logit_scale=-0.5)),
                         ("eps", lambda c: c["norm"].update(eps=0.3))):
        c = json.loads(json.dumps(cfg))
        change(c)
        run(c, W, what)


def test_states_last(pkg, gpu):
    """States that hardly decay: the sequence's first tokens still show hundreds of tokens later, through prompts, portions and decoding."""
    cfg = lc.prenorm([lc.rglru(mlp=lc.dense()), lc.gla(rank=4)], vocab=90)
    W = lc.Weights(lc.parse(pkg, cfg), 6)
    W["l0.mix.lam"][:] = -12.0
    W["l1.mix.a2.b"][:] = 9.0
    eng, _ = make(pkg, cfg, "f32", max_seq=420, weights=W)
    a = lc.tokens(400, 90, 31)
    b = lc.tokens(12, 90, 32) + a[12:]
    want = lo.forward(cfg, W, a)
    assert lc.row_error(lo.forward(cfg, W, b)[-1:], want[-1:]).max() > 5e-3
    check(eng.eval(a, range(400)), want, "f32", "prompt")
    eng.reset()
    check(np.concatenate([eng.eval(a[:130], range(130)), eng.eval(a[130:257], range(127)), stepwise(eng, a[257:])]), want, "f32", "portions and decoding")
    eng.close()


def test_strong_decays(pkg, gpu):
    """States that forget within a token or two: exponents far below what 32-bit holds, and gates at their ends."""
    cfg = lc.prenorm([lc.rglru(), lc.gla(heads=2, dim=40, vdim=16, tau=0.25, rank=6)])
    for bias, lam in ((-8.0, 3.0), (-40.0, 30.0), (30.0, -40.0)):
        W = lc.Weights(lc.parse(pkg, cfg), 9)
        W["l1.mix.a2.b"][:] = lc.bf16(W["l1.mix.a2.b"] + bias)
        W["l0.mix.lam"][:] = lc.bf16(W["l0.mix.lam"] + lam)
        eng, _ = make(pkg, cfg, "f32", weights=W)
        toks = lc.tokens(150, cfg["vocab"], 33)
        want = lo.forward(cfg, W, toks)
        got = np.concatenate([eng.eval(toks[:110], range(110)), stepwise(eng, toks[110:])])
        assert np.isfinite(got).all()
        assert lc.row_error(got, want).max() < 1e-4, (bias, lam)   # (a read-out that nearly vanishes is normed to 1 all the same)
        eng.close()


def test_long_decode(pkg, gpu):
    """700 decoded tokens: chunks begin among decoded tokens many times, states run on."""
    cfg = lc.prenorm([lc.rglru(mlp=lc.grouped()), lc.parallel(lc.gated(4, 2, chunk=50)), lc.parallel(lc.gated(2, 1, chunk=0), lc.gla(2, 16, 16))])
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
    cfg = lc.prenorm([lc.rglru(width=32, blocks=2, mlp=lc.grouped(3, 1, 2, 16, (2, 2))), lc.parallel(lc.gated(2, 1, 16, 16, 300), lc.gla(2, 16, 16, rank=4))], width=40, vocab=64)
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
    cfg = lc.prenorm([lc.rglru(taps=6, mlp=lc.grouped(top=1)), lc.parallel(lc.gated(chunk=4)), lc.rglru(taps=2)])
    eng, W = engine(pkg, cfg, "f32", max_seq=64)
    toks = lc.tokens(9, cfg["vocab"], 17)
    want = lo.forward(cfg, W, toks)
    for cuts in ([9], [1] * 9, [2, 1, 3, 3], [1, 8], [1, 1, 7], [5, 4], [2, 2, 5]):
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
    """A sequence after others is bit for bit the sequence in a fresh context: cache rows, states and the convolutions' inputs are left over but
    not read."""
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
    cfg = lc.prenorm([lc.rglru(mlp=lc.grouped()), lc.parallel(lc.gated(chunk=12), mlp=lc.dense())], vocab=97)
    W = lc.Weights(lc.parse(pkg, cfg), 0)
    W["final.norm"] = lc.bf16(2.0 * np.sign(np.random.default_rng(5).standard_normal(cfg["width"])) - 1.0)   # the next token is not the one just read
    eng, _ = make(pkg, cfg, "f32", max_seq=120, weights=W)
    prompt = lc.tokens(17, cfg["vocab"], 41)
    wrap, ctx = pkg.GpuModelWrapper(eng), pkg.InferenceContext()
    logits = wrap.forward(prompt, ctx)
    first = int(np.flatnonzero(logits == logits.max())[-1])
    out = eng.decode_greedy(first, 50).tolist()
    assert len(set(out)) > 5
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


def test_hidden_state_and_refusals(pkg, gpu):
    cfg = lc.prenorm([lc.rglru(mlp=lc.grouped()), lc.parallel()])
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
    refused(lambda: eng.kv_truncate(10), "Unsupported")                     # the states before are gone
    refused(lambda: eng.kv_shift_left(4), "Unsupported")
    refused(lambda: eng.batch_create(2), "Unsupported")
    check(eng.eval(toks[20:], range(4)), want[20:], "f32", "after the refusals")
    eng.kv_truncate(0)
    check(eng.eval(toks, range(24)), want, "f32", "after a truncation to nothing")
    eng.close()

    class Short(pkg.LayeredModel):
        def tensors(self):
            return (t for t in super().tensors() if t[0] != "l1.mix.left.k.b")
    with pytest.raises(pkg.BackendError, match="l1.mix.left.k.b"):
        pkg.HipGpuInference.from_layered(Short(lc.parse(pkg, cfg), W), 16)


@pytest.mark.parametrize("dtype", DTYPES)
def test_bench_like_sizes(pkg, gpu, dtype):
    """Sizes a real layer has, against the oracle: 128-wide heads, groups of four, diagonal blocks of 256, states of 128 x 256, experts of several hundred."""
    cfg = lc.prenorm([lc.rglru(width=1024, blocks=4, mlp=lc.grouped(14, 4, 3, 320, (6, 2), 5.0)),
                      lc.parallel(lc.gated(8, 2, 128, 128, 150, 64), lc.gla(3, 128, 256, rank=16), (1.0, 0.7), lc.dense(700))], width=1024, vocab=300)
    eng, W = engine(pkg, cfg, dtype, max_seq=320)
    toks = lc.tokens(280, cfg["vocab"], 71)
    want = lo.forward(cfg, W, toks)
    check(np.concatenate([eng.eval(toks[:200], range(200)), eng.eval(toks[200:220], range(20)), stepwise(eng, toks[220:])]), want, dtype)
    eng.close()


def test_trace_run_program(pkg, gpu, tmp_path):
    """bin/trace_run on a model folder: steps in, logits out, two requests one after the other, both number formats."""
    cfg = lc.prenorm([lc.rglru(mlp=lc.grouped()), lc.parallel(lc.gated(chunk=10))])
    W = lc.clear_calls_prenorm(lc.Weights(lc.parse(pkg, cfg), 5), cfg)
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
