"""GPU: the Tarudra design (windowed grouped attention with a sink, partly on another layer's keys; windowed latent attention with query latents;
gated delta rules; layer norms on both sides of every sublayer; squashed logits) against the plain restatement (oracle/layered.py), through the C ABI.

f32 contexts are the sharp test; bf16 contexts are held to bf16 rounding of operands.  Prompts, single tokens, portions and resets must all agree
with ONE whole-sequence run of the oracle."""
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
G, L, D = lc.grouped_attn, lc.latent2, lc.delta
TWO = lambda **kw: [G(window=30), G(source=0, **kw)]

# every mechanism alone, sizes at and around the kernels' granules, and sizes that another model of the design might have
CASES = {
    "attention": dict(layers=[G()]),
    "attention, no window": dict(layers=[G(window=0)]),
    "attention, no rotation": dict(layers=[G(rot=0)]),
    "attention, all rotated, scaled": dict(layers=[G(rot=24, scaling=lc.YARN)]),
    "attention, scaled past its ends": dict(layers=[G(rot=8, base=50.0, scaling={"factor": 8.0, "original": 20, "fast": 40.0, "slow": 0.01})]),
    "window of one": dict(layers=[G(window=1)]),
    "window of two": dict(layers=[G(window=2)]),
    "window of 64": dict(layers=[G(window=64)]),
    "window of 65": dict(layers=[G(window=65)]),
    "window beyond the sequence": dict(layers=[G(window=5000)]),
    "one head of one value": dict(layers=[G(heads=1, kv_heads=1, dim=1, vdim=1, rot=0)]),
    "odd heads": dict(layers=[G(heads=5, kv_heads=5, dim=33, vdim=41)]),
    "eleven heads on one": dict(layers=[G(heads=11, kv_heads=1, dim=72, vdim=40)]),
    "groups of seven": dict(layers=[G(heads=14, kv_heads=2, dim=34, vdim=70, rot=34)]),
    "heads of 64": dict(layers=[G(heads=4, kv_heads=2, dim=64, vdim=64, rot=32)]),
    "keys of 64, values of 256": dict(layers=[G(heads=2, kv_heads=1, dim=64, vdim=256)]),
    "keys of 200, values of 8": dict(layers=[G(heads=3, kv_heads=3, dim=200, vdim=8, rot=200)]),
    "keys of 300, values of 31": dict(layers=[G(heads=3, kv_heads=1, dim=300, vdim=31)]),
    "strong scores": dict(layers=[G(scale=2.0)]),
    "weak scores": dict(layers=[G(scale=0.01)]),
    "shared keys": dict(layers=TWO(window=30)),
    "shared keys, wider window": dict(layers=TWO(window=47)),
    "shared keys, narrower window": dict(layers=TWO(window=11)),
    "shared keys, no window": dict(layers=TWO(window=0)),
    "shared keys, other scale": dict(layers=TWO(scale=0.7)),
    "shared keys, two readers": dict(layers=[D(), G(heads=4, kv_heads=4, dim=64, vdim=40), G(4, 4, 64, 40, source=1), L(), G(4, 4, 64, 40, window=5, source=1)]),
    "latent": dict(layers=[L()]),
    "latent, no window": dict(layers=[L(window=0)]),
    "latent, no rotation": dict(layers=[L(rotate=False)]),
    "latent, part rotated": dict(layers=[L(rot=12, dims=6)]),
    "latent, scaled rotation": dict(layers=[L(rot=16, scaling=lc.YARN)]),
    "latent, two rotated values": dict(layers=[L(rot=2)]),
    "latent, window of one": dict(layers=[L(window=1)]),
    "latent, window of 33": dict(layers=[L(window=33)]),
    "latent, window of 64": dict(layers=[L(window=64)]),
    "latent, window beyond the sequence": dict(layers=[L(window=5000)]),
    "latent, one head": dict(layers=[L(heads=1, dim=1, rot=2, vdim=2, rank=3, q_rank=2)]),
    "latent, eleven heads": dict(layers=[L(heads=11, dim=33, rot=10, vdim=41, rank=70, q_rank=67)]),
    "latent, wide": dict(layers=[L(heads=4, dim=128, rot=64, vdim=128, rank=256, q_rank=192)]),
    "latent, heads too wide to expand": dict(layers=[L(heads=2, dim=250, rot=16, vdim=40, rank=30, q_rank=300)]),
    "latent, wide values": dict(layers=[L(heads=2, dim=16, rot=8, vdim=300, rank=64, q_rank=16)]),
    "latent, query latent wider than the stream": dict(layers=[L(q_rank=2300)]),
    "delta": dict(layers=[D()]),
    "delta, one head": dict(layers=[D(1, 1, 4, 3)]),
    "delta, keys of one": dict(layers=[D(3, 1, 1, 5)]),
    "delta, own keys": dict(layers=[D(3, 3, 17, 33)]),
    "delta, one key head": dict(layers=[D(7, 1, 30, 15)]),
    "delta, keys of 16, values of 16": dict(layers=[D(2, 1, 16, 16)]),
    "delta, keys of 64, values of 128": dict(layers=[D(4, 2, 64, 128)]),
    "delta, keys of 65": dict(layers=[D(2, 1, 65, 40)]),
    "delta, keys of 128, values of 64": dict(layers=[D(2, 2, 128, 64)]),
    "delta, keys of 150, values of 300": dict(layers=[D(2, 1, 150, 300)]),
    "delta, keys of 256": dict(layers=[D(2, 1, 256, 32)]),
    "delta, keys of 300": dict(layers=[D(1, 1, 300, 20)]),
    "delta, keys of 512": dict(layers=[D(1, 1, 512, 33)]),
    "delta, keys of 530": dict(layers=[D(1, 1, 530, 20)]),
    "delta, one tap": dict(layers=[D(taps=1)]),
    "delta, two taps": dict(layers=[D(taps=2)]),
    "delta, three taps": dict(layers=[D(taps=3)]),
    "delta, five taps": dict(layers=[D(taps=5)]),
    "delta, nineteen taps": dict(layers=[D(taps=19)]),
    "feed-forward": dict(layers=[D(mlp=lc.dense(100))]),
    "feed-forward, odd": dict(layers=[G(mlp=lc.dense(33)), G(mlp=lc.dense(1))]),
    "odd width": dict(layers=[G(mlp=lc.dense(50)), D(), L()], width=301, vocab=77),
    "wide stream": dict(layers=[D(mlp=lc.dense(70)), G()], width=1040, vocab=61),
    "wider stream": dict(layers=[L(mlp=lc.dense(70)), D()], width=4200, vocab=61),
    "loose cap": dict(layers=[G(mlp=lc.dense())], cap=50.0),
    "tight cap": dict(layers=[G(mlp=lc.dense())], cap=0.3),
    "mixed": dict(layers=[G(mlp=lc.dense()), D(mlp=lc.dense(90)), G(window=25, source=0, mlp=lc.dense()), L(mlp=lc.dense()), L(window=17), D(5, 5, 40, 28, 3), G(4, 4, 30, 18, 17, 10),
                          G(4, 4, 30, 18, 33, 10, source=6, mlp=lc.dense(40))]),
}


F32_ONLY = {"delta, keys of one"}   # (a unit vector of one value is a sign: rounding may turn it)


def case(name):
    return lc.sandwich_ln(**CASES[name])


@pytest.mark.parametrize("name,dtype", [(n, d) for n in CASES for d in DTYPES if d == "f32" or n not in F32_ONLY])
def test_prompt_and_decode_match_the_oracle(pkg, gpu, name, dtype):
    print(name, dtype, flush=True)
    cfg = case(name)
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
        assert (d[-1] <= 2e-5 if dtype == "f32" else d[-7] <= 3e-2), f"layer {i}: {d[-7:]}"
    check(got, want, dtype, "whole prompt")
    eng.reset()
    check(stepwise(eng, toks[:70]), want[:70], dtype, "token by token")
    eng.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_portions_of_any_size_agree(pkg, gpu, dtype):
    """Cuts at and around multiples of the kernels' tiles (16 tokens: the decode kernel's portions; 32 / 64 keys, the delta rule's chunks of 64
    tokens; 64 / 128 queries), inside windows and at their edges, down to two tokens, and single tokens between them."""
    cfg = case("mixed")
    eng, W = make(pkg, cfg, dtype, max_seq=400)
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


def asking(cfg, W, layers):
    """Token 117 asks, 118 and 119 are keys that answer differently; in `layers` one key stands out for the question, by a score that no rotation
    changes.  Channel 0 of the stream is the question, 1 the answer, 2 marks a key; no sublayer writes to them."""
    W["embed"][:, :3] = 0.0
    W["embed"][[117, 118, 119]] = 0.0
    W["embed"][117, 0] = 3.0
    W["embed"][[118, 119], 2] = 3.0
    W["embed"][118, 1], W["embed"][119, 1] = 3.0, -3.0

    def row(name, r, channel, v):
        W[name][r, :] = 0.0
        W[name][r, channel] = v
    for i in layers:
        p, mx = f"l{i}.mix.", cfg["layers"][i]["mixer"]
        W[f"l{i}.norm1"][:3] = 1.0
        W[f"l{i}.norm1b"][:3] = 0.0
        d = mx["dim"]
        if cfg["layers"][i]["type"] == "attention":
            for n in range(mx["heads"]):
                row(p + "q", n * d + 8, 0, 1.0)
            for name in ("q", "k", "v"):
                if p + name in W:
                    W[p + name + ".b"][:] = 0.0
            if p + "k" in W:
                for g in range(mx["kv_heads"]):
                    row(p + "k", g * d + 8, 2, 1.0)
                    row(p + "v", g * mx["vdim"], 1, 2.0)
        else:
            row(p + "dq", 0, 0, 8.0)
            row(p + "dkv", 0, 2, 8.0)
            row(p + "dkv", 1, 1, 8.0)
            for n in range(mx["heads"]):
                row(p + "uq", n * (d + mx["rot_dim"]), 0, 2.0)
                row(p + "uk", n * d, 0, 2.0)
    return 117, 118, 119


FAR = {
    "attention": lambda w: ([G(2, 1, 16, 12, w, 6, scale=0.7)], [0], w),
    "shared keys": lambda w: ([G(2, 1, 16, 12, max(w // 2, 1), 6, scale=0.7), G(2, 1, 16, 12, w, 6, scale=0.7, source=0)], [0, 1], w),
    "latent": lambda w: ([L(2, 12, 6, 10, 20, 16, w, 1.0)], [0], w),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", list(FAR))
@pytest.mark.parametrize("window,n", [(50, 140), (64, 200), (63, 130), (129, 300), (32, 97), (40, 41), (2, 20), (1, 9), (0, 260)])
def test_a_key_just_inside_and_just_outside(pkg, gpu, dtype, kind, window, n):
    """One key stands out for the last token's query.  Inside the window its value must decide the logits, one position before it must not matter at
    all, in a prompt, in decoding and at the start of a portion; the oracle says which is which."""
    layers, who, window = FAR[kind](window)
    cfg = lc.sandwich_ln(layers, width=96, vocab=120)
    W = lc.Weights(lc.parse(pkg, cfg), 3)
    Q, KA, KB = asking(cfg, W, who)
    eng, _ = make(pkg, cfg, dtype, max_seq=320, weights=W)
    def near(got, want, what):
        assert lc.row_error(got, want).max() <= (2e-5 if dtype == "f32" else 0.06), what
    base = [t % 110 for t in lc.tokens(n, 110, 9)]
    last = n - 1
    start = max(last - window + 1, 0) if window else 0
    places = {0, 1, start - 2, start - 1, start, start + 1, last - 1, 31, 32, 63, 64}
    for far in sorted(p for p in places if 0 <= p < last):
        ends = []
        for key in (KA, KB):
            toks = list(base)
            toks[far], toks[last] = key, Q
            want = lo.forward(cfg, W, toks)[last:]
            eng.reset()
            near(eng.eval(toks, [last]), want, f"prompt, key {far} of {n}")
            eng.reset()
            eng.eval(toks[:last])
            near(eng.forward(Q)[None], want, f"decoded, key {far} of {n}")
            if last - far >= 3:
                eng.reset()
                eng.eval(toks[:last - 1])
                near(eng.eval(toks[last - 1:], [1]), want, f"a portion of two, key {far} of {n}")
            ends.append(want)
        moved = lc.row_error(ends[0], ends[1]).max()
        assert moved > 0.2 if far >= start else moved < 1e-9, f"key {far} of {n}: {moved}"
    eng.close()


def test_the_sink_takes_its_share(pkg, gpu):
    """Scores far below the sink's leave almost nothing of the values; far above it almost everything; the first token has one key and the sink."""
    for shift in (-30.0, -4.0, 0.0, 4.0, 30.0):
        cfg = lc.sandwich_ln([G(4, 2, 16, 12, 50, 0, scale=1.0)], width=64)
        W = lc.Weights(lc.parse(pkg, cfg), 8)
        W["l0.mix.q"][:] = lc.bf16(0.1 * W["l0.mix.q"])
        W["l0.mix.q"][::16] = 0.0
        W["l0.mix.k"][::16] = 0.0
        W["l0.mix.q.b"][::16], W["l0.mix.k.b"][::16] = shift, 1.0    # every score is about `shift`
        W["l0.mix.o.b"][:] = lc.bf16(W["l0.mix.o.b"] * 0.05)         # (a norm follows: what the values leave shows beside the bias)
        eng, _ = make(pkg, cfg, "f32", weights=W)
        toks = lc.tokens(90, cfg["vocab"], 12)
        want = lo.forward(cfg, W, toks)
        check(eng.eval(toks, range(90)), want, "f32", f"prompt, scores about {shift}")
        eng.reset()
        check(np.concatenate([stepwise(eng, toks[:60]), eng.eval(toks[60:70], range(10)), eng.eval(toks[70:], range(20))]), want, "f32", f"steps, scores about {shift}")
        eng.close()


def test_each_constant_and_weight_shows(pkg, gpu):
    """The engine follows the oracle when one thing changes, and each change moves the logits."""
    cfg = lc.sandwich_ln([G(window=24, rot=12, scale=0.4, scaling=lc.YARN, mlp=lc.dense()), D(), G(window=18, rot=12, scale=0.4, scaling=lc.YARN, source=0),
                          L(window=20, scale=0.4, mlp=lc.dense(30))])
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
    for name in W:
        if name in ("embed", "head") or (name.startswith("l2.") and "mix" not in name):
            continue
        w = lc.Weights(lc.parse(pkg, cfg), 4)
        w[name] = lc.bf16(w[name][..., ::-1] * -0.5 + 0.1)
        run(cfg, w, name)
    mixer = lambda c, i: c["layers"][i]["mixer"]
    yarn = lambda c, **kw: [mixer(c, i)["rot"]["scaling"].update(**kw) for i in (0, 2)]
    rot = lambda c, **kw: [mixer(c, i)["rot"].update(**kw) for i in (0, 2)]
    for what, change in (("scale", lambda c: mixer(c, 0).update(scale=0.9)), ("window", lambda c: mixer(c, 0)["mask"].update(size=25)), ("no window", lambda c: mixer(c, 0).pop("mask")),
                         ("the reader's scale", lambda c: mixer(c, 2).update(scale=0.9)), ("the reader's window", lambda c: mixer(c, 2)["mask"].update(size=19)),
                         ("rotation base", lambda c: rot(c, base=10.0)), ("rotated values", lambda c: rot(c, dims=4)), ("scaling factor", lambda c: yarn(c, factor=2.0)),
                         ("scaling, original", lambda c: yarn(c, original=300)), ("scaling, fast", lambda c: yarn(c, fast=2.0)), ("scaling, slow", lambda c: yarn(c, slow=0.01)),
                         ("no scaling", lambda c: [mixer(c, i)["rot"].pop("scaling") for i in (0, 2)]), ("latent scale", lambda c: mixer(c, 3).update(scale=0.9)),
                         ("latent window", lambda c: mixer(c, 3)["mask"].update(size=19)), ("latent rotation base", lambda c: mixer(c, 3)["rot"].update(base=10.0)),
                         ("latent rotated values", lambda c: mixer(c, 3)["rot"].update(dims=4)), ("logit cap", lambda c: c.update(logit_softcap=0.9)), ("eps", lambda c: c["norm"].update(eps=0.3))):
        c = json.loads(json.dumps(cfg))
        change(c)
        run(c, W, what)


def test_states_last(pkg, gpu):
    """States that hardly decay and are hardly corrected: the sequence's first tokens still show hundreds of tokens later, through prompts, portions and
    decoding."""
    cfg = lc.sandwich_ln([D(4, 2, 40, 16)], vocab=90)
    W = lc.Weights(lc.parse(pkg, cfg), 6)
    W["l0.mix.dt_bias"][:], W["l0.mix.A_log"][:] = -12.0, -2.0
    W["l0.mix.b"][:] = lc.bf16(W["l0.mix.b"] * 0.1)
    eng, _ = make(pkg, cfg, "f32", max_seq=420, weights=W)
    a = lc.tokens(400, 90, 31)
    b = lc.tokens(12, 90, 32) + a[12:]
    want = lo.forward(cfg, W, a)
    assert lc.row_error(lo.forward(cfg, W, b)[-1:], want[-1:]).max() > 1e-4
    check(eng.eval(a, range(400)), want, "f32", "prompt")
    eng.reset()
    check(np.concatenate([eng.eval(a[:130], range(130)), eng.eval(a[130:257], range(127)), stepwise(eng, a[257:])]), want, "f32", "portions and decoding")
    eng.close()


@pytest.mark.parametrize("what", ["decays", "steps of one on the same key", "no steps", "opposite keys"])
def test_extreme_decays_and_steps(pkg, gpu, what):
    """Exponents far below what 32-bit holds beside tokens that keep everything; values written whole onto a key that hardly changes; nothing written."""
    cfg = lc.sandwich_ln([D(3, 1, 40, 16)])
    W = lc.Weights(lc.parse(pkg, cfg), 9)
    if what == "decays":
        W["l0.mix.A_log"][:] = 3.0
        W["l0.mix.a"][:] = lc.bf16(W["l0.mix.a"] * 12.0)      # log decays between -1e-5 and -1e3 within one chunk
    elif what == "no steps":
        W["embed"][:, 0], W["l0.norm1"][0] = 4.0, 1.0
        W["l0.mix.b"][:, 0] = -12.0
    else:
        W["embed"][:, 0], W["l0.norm1"][0] = 6.0, 1.0
        W["l0.mix.b"][:, 0] = 6.0
        W["l0.mix.dt_bias"][:] = -9.0
        W["l0.mix.k"][:] = lc.bf16(W["l0.mix.k"] * 0.02)
        W["l0.mix.k"][:20, 0] = 1.0
        W["l0.mix.k.conv"][:] = [[0.0, 0.0, 0.0, 1.0]]
        if what == "opposite keys":
            W["l0.mix.k"][:20, 1] = 1.5
            W["embed"][::2, 1], W["embed"][1::2, 1] = 9.0, -9.0
    eng, _ = make(pkg, cfg, "f32", weights=W)
    toks = lc.tokens(200, cfg["vocab"], 33)
    want = lo.forward(cfg, W, toks)
    got = np.concatenate([eng.eval(toks[:150], range(150)), stepwise(eng, toks[150:])])
    assert np.isfinite(got).all()
    err = lc.row_error(got, want)
    assert err.max() < 2e-4, (what, int(err.argmax()), err.max())   # (a read-out that nearly vanishes is normed to 1 all the same)
    eng.close()


def test_long_decode(pkg, gpu):
    """700 decoded tokens: every window passes over decoded tokens many times, states run on."""
    cfg = lc.sandwich_ln([G(4, 2, window=50, mlp=lc.dense()), D(), G(4, 2, window=70, source=0), L(2, window=60), G(2, 1, window=0), L(2, window=0)])
    eng, W = make(pkg, cfg, "f32", max_seq=740, seed=7)
    toks = lc.tokens(740, cfg["vocab"], 11)
    want = lo.forward(cfg, W, toks)
    check(np.concatenate([eng.eval(toks[:40], range(40)), stepwise(eng, toks[40:])]), want, "f32", "long decode")
    eng.reset()
    check(eng.eval(toks, range(740)), want, "f32", "the same as one prompt")
    eng.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_prompts_longer_than_one_block(pkg, gpu, dtype):
    """The block path takes 2048 tokens at a time: the border inside one call, and a second long portion after it."""
    cfg = lc.sandwich_ln([G(2, 1, 16, 16, 300), D(2, 1, 16, 16), G(2, 1, 16, 16, 500, source=0), L(2, 8, 4, 8, 12, 10, 200)], width=40, vocab=64)
    eng, W = make(pkg, cfg, dtype, max_seq=2400, seed=13)
    toks = lc.tokens(2400, cfg["vocab"], 15)
    want = lo.forward(cfg, W, toks)
    places = list(range(2020, 2080)) + [2299]
    check(eng.eval(toks[:2300], places), want[places], dtype, "one call")
    check(eng.eval(toks[2300:2390], range(90)), want[2300:2390], dtype, "the next portion")
    check(stepwise(eng, toks[2390:]), want[2390:], dtype, "decoded")
    eng.close()


def test_first_tokens(pkg, gpu):
    """Nothing lies before a sequence's first token, however its first portions are cut, also right after another sequence."""
    cfg = lc.sandwich_ln([D(taps=6), G(window=4), G(window=3, source=1), L(window=5), D(taps=2, mlp=lc.dense())])
    eng, W = make(pkg, cfg, "f32", max_seq=64)
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
    fresh, _ = make(pkg, cfg, dtype, max_seq=200, weights=W)
    assert np.array_equal(run(fresh, b), first)
    fresh.reset()
    assert np.array_equal(fresh.forward(b[0]), one)
    eng.close()
    fresh.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_graph_replays_equal_eager_launches(pkg, gpu, dtype):
    cfg = case("mixed")
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
    cfg = lc.sandwich_ln([G(window=12, mlp=lc.dense()), D(), G(window=9, source=0), L(window=10, mlp=lc.dense())], vocab=97)
    eng, W = make(pkg, cfg, "f32", max_seq=120)
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
        eng, W = make(pkg, cfg, "f32", **kw)
        ref = lo.forward(cfg, W, toks) if ref is None else ref
        assert eng.prefill_is_batched() == ("flags" not in kw)
        check(np.concatenate([eng.eval(toks[:90], range(90)), eng.eval(toks[90:101], range(11)), stepwise(eng, toks[101:])]), ref, "f32", str(kw))
        eng.close()


def test_hidden_state_and_refusals(pkg, gpu):
    cfg = lc.sandwich_ln([D(mlp=lc.dense()), G(), L(), G(source=1)])
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
    refused(lambda: eng.kv_truncate(10), "Unsupported")                     # the states before are gone
    refused(lambda: eng.kv_shift_left(4), "Unsupported")
    refused(lambda: eng.batch_create(2), "Unsupported")
    check(eng.eval(toks[20:], range(4)), want[20:], "f32", "after the refusals")
    eng.kv_truncate(0)
    check(eng.eval(toks, range(24)), want, "f32", "after a truncation to nothing")
    eng.close()

    class Short(pkg.LayeredModel):
        def tensors(self):
            return (t for t in super().tensors() if t[0] != "l0.mix.k.conv")
    with pytest.raises(pkg.BackendError, match="l0.mix.k.conv"):
        pkg.HipGpuInference.from_layered(Short(lc.parse(pkg, cfg), W), 16)


def test_cutting_back_a_model_without_states(pkg, gpu):
    """Attention layers alone keep rows by position: a sequence may be cut back and go on, also where another layer's rows are read."""
    cfg = lc.sandwich_ln([G(window=12), G(window=20, source=0), L(window=9)])
    eng, W = make(pkg, cfg, "f32", max_seq=100)
    toks, other = lc.tokens(80, cfg["vocab"], 63), lc.tokens(30, cfg["vocab"], 64)
    eng.eval(toks)
    eng.kv_truncate(41)
    seq = toks[:41] + other
    want = lo.forward(cfg, W, seq)[41:]
    check(np.concatenate([eng.eval(other[:10], range(10)), stepwise(eng, other[10:])]), want, "f32")
    eng.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_bench_like_sizes(pkg, gpu, dtype):
    """Sizes a real layer has, against the oracle: 128-wide heads, groups of four, latents of several hundred, states of 128 x 128."""
    cfg = lc.sandwich_ln([G(8, 2, 128, 128, 150, 128, scaling=dict(lc.YARN, original=200), mlp=lc.dense(700)), D(6, 3, 128, 128), G(8, 2, 128, 128, 100, 128, scaling=dict(lc.YARN, original=200), source=0),
                          L(8, 128, 64, 128, 512, 384, 120)], width=1024, vocab=300)
    eng, W = make(pkg, cfg, dtype, max_seq=320)
    toks = lc.tokens(280, cfg["vocab"], 71)
    want = lo.forward(cfg, W, toks)
    check(np.concatenate([eng.eval(toks[:200], range(200)), eng.eval(toks[200:220], range(20)), stepwise(eng, toks[220:])]), want, dtype)
    eng.close()


def test_trace_run_program(pkg, gpu, tmp_path):
    """bin/trace_run on a model folder: steps in, logits out, two requests one after the other, both number formats."""
    cfg = lc.sandwich_ln([D(mlp=lc.dense()), G(window=10), L(window=7), G(window=8, source=1)])
    W = lc.Weights(lc.parse(pkg, cfg), 5)
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
