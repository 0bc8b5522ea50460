"""MI355X: the layer-list engine serving Faguzen models against the plain float64 restatement
in tests/faguzen_ref.py, on small random models made here.

Errors are per position: || got - ref || / || ref || over the vocabulary. With f32 matrices
the engine differs from the restatement by f32 rounding only (F32_TOL); with bf16 matrices by
the rounding of the products' inputs and of the cached keys and values (BF16_TOL; a model with
routed experts may miss it at a few positions where that rounding flips a router near-tie). A
lost key, a score cap or a pass vector left out, a wrong normaliser, a state that is not carried
or a token one place off moves the logits by orders of magnitude more than F32_TOL.
"""
import copy
import dataclasses
import json
import os
import subprocess

import numpy as np
import pytest

import faguzen_cases as C
import faguzen_ref as R

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
F32_TOL, BF16_TOL = 2e-4, 6e-2


@pytest.fixture(scope="module")
def rt():
    from yalm_amd import runtime

    runtime.check(runtime.lib.yalm_set_device(0))
    return runtime


def make(cfg, seed=0):
    from yalm_amd import layered as Ly

    return Ly.faguzen_random_tensors(cfg, seed=seed)


def f64(t):
    return {k: v.astype(np.float64) for k, v in t.items()}


def build(rt, cfg, wdt, seed=0, max_tokens=512, tensors=None):
    from yalm_amd import layered as Ly

    t = tensors if tensors is not None else make(cfg, seed)
    c = Ly.faguzen_config(cfg, max_tokens=max_tokens, weight_dtype=wdt)
    model = rt.SeqModel.from_packed(c, Ly.faguzen_pack(c, t, cfg))
    return model, rt.SeqDecoder(model), f64(t)


def rel_err(got, ref):
    return np.linalg.norm(got - ref, axis=-1) / np.linalg.norm(ref, axis=-1)


def wdt_of(dtype):
    from yalm_amd import models as M

    return M.F32 if dtype == "f32" else M.BF16


def routed(cfg):
    return any(e.get("mlp") for e in cfg["layers"])


def agrees(got, ref, dtype, cfg):
    e = rel_err(got, ref)
    if dtype == "f32":
        return e.max() < F32_TOL
    if routed(cfg):  # a flipped near-tie of a router: a few positions, never the bulk
        return np.mean(e > BF16_TOL) <= 0.1 and np.median(e) < BF16_TOL / 3
    return e.max() < BF16_TOL


def run_portions(dec, tok, sizes):
    """Feed tok in portions of the given sizes (the last one takes the rest), asking for
    every position's logits."""
    out, at = [], 0
    for s in list(sizes) + [len(tok)]:
        s = min(s, len(tok) - at)
        if s <= 0:
            break
        out.append(dec.step(tok[at:at + s], list(range(s))))
        at += s
    return np.concatenate(out)


# ------------------------------------------------------------------ mechanisms alone
@pytest.mark.parametrize("name", ["only_pair", "only_moe"])
@pytest.mark.parametrize("dtype", ["f32", "bf16"])
def test_each_sublayer_kind_alone(rt, name, dtype):
    cfg = C.ALL[name]
    model, dec, w = build(rt, cfg, wdt_of(dtype), seed=1)
    try:
        tok = C.tokens(cfg, 70, 1)
        ref = R.forward(cfg, w, tok)
        assert agrees(dec.step(tok, list(range(len(tok)))), ref, dtype, cfg)
        dec.reset()
        assert agrees(run_portions(dec, tok, [30] + [1] * 40), ref, dtype, cfg)
    finally:
        dec.close()
        model.close()


def parts_of(cfg, t):
    """The packed one-layer pair model of cfg: (LayeredConfig, packed, the attention's and the
    memory's own (spec, tensors), each projecting for itself)."""
    from yalm_amd import layered as Ly
    from yalm_amd import models as M

    c = Ly.faguzen_config(cfg, max_tokens=256, weight_dtype=M.F32)
    p = Ly.faguzen_pack(c, t, cfg)
    d, l = p["layers"][0], c.layers[0]
    own = l.in_rows
    left = dataclasses.replace(l, side=None, side_shares_in=False)
    ld = {k: v for k, v in d.items() if k != "side"}
    ld.update(w_in=np.ascontiguousarray(d["w_in"][:own]), in_bias=np.ascontiguousarray(d["in_bias"][:own]))
    right = dataclasses.replace(l.side, in_biased=True)
    rd = dict(d["side"], w_in=np.ascontiguousarray(d["w_in"][own:]), in_bias=np.ascontiguousarray(d["in_bias"][own:]))
    return c, p, (left, ld), (right, rd)


def finish(cfg, w, x):
    return R.soft_cap(R.tanh_norm(x, w, "final.norm") @ w["head"].T, cfg["logit_softcap"])


@pytest.mark.parametrize("which", ["left", "right"])
def test_each_mixer_of_a_pair_alone(rt, which):
    """The two mixers of a pair are ordinary mixers of the engine: a one-layer stack put together
    by hand with the attention alone, or the matrix memory alone (no second mixer, no join)."""
    from yalm_amd import layered as Ly

    cfg = C.ONLY_PAIR
    t = make(cfg, 31)
    w = f64(t)
    c, p, (left, ld), (right, rd) = parts_of(cfg, t)
    if which == "left":
        spec, pd = left, ld
    else:
        spec, pd = dataclasses.replace(right, ff_normed=True, layer_scaled=False), dict(rd, norm1=ld["norm1"])
    c1 = c.with_(layers=[spec])
    assert set(pd) == set(Ly.packed_shapes(c1, spec))
    model = rt.SeqModel.from_packed(c1, dict(p, layers=[pd]))
    dec = rt.SeqDecoder(model)
    try:
        tok = C.tokens(cfg, 90, 31)
        m = cfg["layers"][0]["mixer"]
        x = w["embed"][tok]
        h = R.tanh_norm(x, w, "l0.norm1")
        x = x + cfg["residual_mult"] * (R.mixer_attention(cfg, w, "l0.mix.left.", h, m["left"]) if which == "left"
                                        else R.mixer_memory(cfg, w, "l0.mix.right.", h, m["right"]))
        ref = finish(cfg, w, x)
        for sizes in ([90], [40] + [1] * 50, [2, 9, 3, 8, 33]):
            dec.reset()
            assert rel_err(run_portions(dec, tok, sizes), ref).max() < F32_TOL
    finally:
        dec.close()
        model.close()


def test_pair_with_a_projection_each(rt):
    """A pair whose mixers project for themselves computes what the shared projection does."""
    cfg = C.ONLY_PAIR
    t = make(cfg, 32)
    c, p, (left, ld), (right, rd) = parts_of(cfg, t)
    c1 = c.with_(layers=[dataclasses.replace(left, side=right)])
    model = rt.SeqModel.from_packed(c1, dict(p, layers=[dict(ld, side=rd)]))
    dec = rt.SeqDecoder(model)
    try:
        tok = C.tokens(cfg, 60, 32)
        ref = R.forward(cfg, f64(t), tok)
        for sizes in ([60], [20] + [1] * 40):
            dec.reset()
            assert rel_err(run_portions(dec, tok, sizes), ref).max() < F32_TOL
    finally:
        dec.close()
        model.close()


@pytest.mark.parametrize("ff", [False, True])
@pytest.mark.parametrize("width", [96, 4104])
def test_mechanisms_in_serial_blocks(rt, ff, width):
    """Tanh norms, the residual scale, the plain join of a pair and identity outputs are mechanisms of
    the engine, not of one envelope: the same layer in serial blocks with opening and closing norms,
    in the seam kernels that hold the row in registers and in LDS."""
    from yalm_amd import layered as Ly

    cfg = C.config([(C.pair(C.attn(heads=2, kv_heads=1, dim=16, vdim=8), C.memory(heads=2, dim=8, vdim=8)),
                     C.moe(ff=8, shared=8) if ff else None)], width=width, vocab=53)
    t = make(cfg, 33)
    w = f64(t)
    c, p, _, _ = parts_of(cfg, t)
    rng = np.random.default_rng(5)
    closing = [np.concatenate([rng.uniform(0.5, 1.5, width), 0.2 * rng.standard_normal(width), [a]]).astype(np.float32)
               for a in (0.7, 1.3)]
    for k, v in enumerate(closing):
        w.update({f"c{k}": v[:width].astype(np.float64), f"c{k}.b": v[width:-1].astype(np.float64),
                  f"c{k}.alpha": np.float64(v[-1])})
    spec = dataclasses.replace(c.layers[0], ff_normed=False)
    c1 = c.with_(layers=[spec], block_kind=Ly.BLOCK_SERIAL)
    pd = dict(p["layers"][0], norm1b=closing[0], **({"norm2b": closing[1]} if ff else {}))
    assert set(pd) - {"side"} == set(Ly.packed_shapes(c1, spec))
    model = rt.SeqModel.from_packed(c1, dict(p, layers=[pd]))
    dec = rt.SeqDecoder(model)
    try:
        tok = C.tokens(cfg, 40, 33)
        e, m = cfg["layers"][0], cfg["residual_mult"]
        x = w["embed"][tok]
        x = x + m * R.tanh_norm(R.mixer_pair(cfg, w, "l0.mix.", R.tanh_norm(x, w, "l0.norm1"), e["mixer"]), w, "c0")
        if ff:
            picks = []
            y = R.feed_forward(w, "l0.mlp.", R.tanh_norm(x, w, "l0.norm2"), e["mlp"], picks)
            assert any((i >= e["mlp"]["router"]["experts"]).any() for i, _ in picks)
            x = x + m * R.tanh_norm(y, w, "c1")
        ref = finish(cfg, w, x)
        for sizes in ([40], [15] + [1] * 25, [2, 9, 3, 8]):
            dec.reset()
            assert rel_err(run_portions(dec, tok, sizes), ref).max() < F32_TOL
    finally:
        dec.close()
        model.close()


@pytest.mark.parametrize("r", [C.rot(dims=24, scaled=False), C.rot(dims=2), C.rot(dims=24, base=3.0, original=700),
                               C.rot(dims=10, base=90.0, low=0.5, high=0.5), C.rot(dims=12, base=2.0, original=3, factor=1.0)],
                         ids=["all_plain", "one_pair", "all_three_ranges", "step", "factor_one"])
def test_rotation(rt, r):
    """Half-split pairs and the three ranges of the frequency rescaling, on keys and queries that
    weigh the rotated entries heavily."""
    from yalm_amd import models as M

    cfg = C.config([(C.pair(C.attn(dim=24, softcap=30.0, r=r)), None)])
    t = make(cfg, 34)
    t["l0.mix.left.q"] = t["l0.mix.left.q"] * 3.0
    model, dec, w = build(rt, cfg, M.F32, tensors=t)
    try:
        tok = C.tokens(cfg, 120, 34)
        ref = R.forward(cfg, w, tok)
        if r.get("scaling") and r["scaling"]["factor"] != 1.0:
            plain = copy.deepcopy(cfg)
            del plain["layers"][0]["mixer"]["left"]["rot"]["scaling"]
            if not np.allclose(R.rotation_frequencies(r["dims"], r["base"], r["scaling"]),
                               R.rotation_frequencies(r["dims"], r["base"], None)):
                assert rel_err(R.forward(plain, w, tok), ref).max() > 20 * F32_TOL
        for sizes in ([120], [50] + [1] * 70):
            dec.reset()
            assert rel_err(run_portions(dec, tok, sizes), ref).max() < F32_TOL
    finally:
        dec.close()
        model.close()


@pytest.mark.parametrize("dtype", ["f32", "bf16"])
@pytest.mark.parametrize("cap", [0.4, 3.0, 1000.0])
def test_score_cap(rt, cap, dtype):
    """Caps far below the scores, among them and far above, in all attention kernels."""
    cfg = C.config([(C.pair(C.attn(heads=4, kv_heads=2, dim=32, vdim=48, scale=0.8, softcap=cap, r=C.rot(dims=16)),
                            C.memory(heads=1, dim=4, vdim=4), 4.0, 0.05), None)])
    model, dec, w = build(rt, cfg, wdt_of(dtype), seed=35)
    try:
        tok = C.tokens(cfg, 130, 35)
        ref = R.forward(cfg, w, tok)
        off = copy.deepcopy(cfg)
        off["layers"][0]["mixer"]["left"]["softcap"] = None
        if cap < 100:
            assert rel_err(R.forward(off, w, tok), ref).max() > 3 * BF16_TOL
        for sizes in ([130], [60] + [1] * 70, [5, 6, 40, 7]):
            dec.reset()
            assert agrees(run_portions(dec, tok, sizes), ref, dtype, cfg)
    finally:
        dec.close()
        model.close()


def memory_trace(cfg, w, tok):
    """Running maxima and read-out normalisers of layer 0's memory, as the design gives them."""
    m = cfg["layers"][0]["mixer"]["right"]
    h = R.tanh_norm(w["embed"][tok], w, "l0.norm1")
    i, f = R.memory_gates(h, w, "l0.mix.right.", m["gate_cap"])
    H, D = m["heads"], m["dim"]
    q = (h @ w["l0.mix.right.q"].T).reshape(len(tok), H, D) * D ** -0.5
    k = (h @ w["l0.mix.right.k"].T).reshape(len(tok), H, D)
    ms, floors = np.zeros((len(tok), H)), np.zeros((len(tok), H), bool)
    for hd in range(H):
        mx, n = 0.0, np.zeros(D)
        for t in range(len(tok)):
            new = max(f[t, hd] + mx, i[t, hd])
            n = np.exp(f[t, hd] + mx - new) * n + np.exp(i[t, hd] - new) * k[t, hd]
            mx = new
            ms[t, hd], floors[t, hd] = mx, abs(n @ q[t, hd]) < np.exp(-mx)
    return ms, floors


@pytest.mark.parametrize("bias", [-6.0, 0.0, 6.0])
def test_memory_maximum_and_normaliser(rt, bias):
    """Input gates far below, around and far above the starting maximum: the maximum decays from its
    start, moves up and down, or jumps; the normaliser takes both sides of its floor. A large constant
    under the root of the heads' norm keeps the read-outs' size, and with it the normaliser, visible."""
    from yalm_amd import models as M

    cfg = C.config([(C.pair(C.attn(heads=1, kv_heads=1, dim=4, vdim=4, r=C.rot(dims=2)),
                            C.memory(heads=4, dim=16, vdim=24, gate_cap=9.0), 0.1, 1.0), None)], eps=0.5)
    t = make(cfg, 36)
    t["l0.mix.right.i.b"] = np.full_like(t["l0.mix.right.i.b"], bias)
    t["l0.mix.right.i"] = t["l0.mix.right.i"] * 3.0
    model, dec, w = build(rt, cfg, M.F32, tensors=t)
    keep = R.normaliser
    try:
        tok = C.tokens(cfg, 100, 36)
        ms, floors = memory_trace(cfg, w, tok)
        assert (np.diff(ms, axis=0) > 0).any() and (np.diff(ms, axis=0) < 0).any()
        if bias <= 0:
            assert floors.any()
        if bias >= 0:
            assert (~floors).any()
        ref = R.forward(cfg, w, tok)
        for other in ([lambda nq, m: abs(nq) + 1e-6] if bias < 0 else []) + [lambda nq, m: 1.0]:
            R.normaliser = other
            assert rel_err(R.forward(cfg, w, tok), ref).max() > 100 * F32_TOL
            R.normaliser = keep
        for sizes in ([100], [17, 2, 16, 31] + [1] * 40, [8, 9, 1, 15]):
            dec.reset()
            assert rel_err(run_portions(dec, tok, sizes), ref).max() < F32_TOL
    finally:
        R.normaliser = keep
        dec.close()
        model.close()


MLPS = [C.moe(), C.moe(experts=5, identity=0, top=1, ff=24, shared=0), C.moe(experts=3, identity=2, top=5, ff=16, shared=8),
        C.moe(experts=70, identity=5, top=7, ff=8, shared=0), C.moe(experts=1, identity=6, top=3, ff=8, shared=16)]


@pytest.mark.parametrize("k", range(len(MLPS)))
def test_routed_experts_follow_the_restatement(rt, k):
    """Every token's chosen outputs and weights, through the logits: the correction moves choices,
    identity outputs are chosen (several per token), top = 1, top = all outputs, more outputs than
    a wave has lanes, no shared expert."""
    from yalm_amd import models as M

    mlp = MLPS[k]
    cfg = C.config([(C.TINY, mlp)], width=48, vocab=77)
    t = make(cfg, 41 + k)
    t["l0.mlp.router"] = t["l0.mlp.router"] * 3.0
    t["l0.mlp.correction"] = t["l0.mlp.correction"] * (0.2 if mlp["router"]["experts"] > 64 else 2.0)
    model, dec, w = build(rt, cfg, M.F32, tensors=t)
    try:
        tok = C.tokens(cfg, 50, 41)
        picks = []
        ref = R.forward(cfg, w, tok, choice_out=picks)
        r = mlp["router"]
        if r["identity"]:
            assert any((i >= r["experts"]).any() for i, _ in picks) and any((i < r["experts"]).any() for i, _ in picks)
        if r["top"] < r["experts"] + r["identity"]:
            assert len({tuple(sorted(i.tolist())) for i, _ in picks}) > 1
            flat = dict(w)
            flat["l0.mlp.correction"] = np.zeros_like(w["l0.mlp.correction"])
            assert rel_err(R.forward(cfg, flat, tok), ref).max() > 100 * F32_TOL
        for sizes in ([50], [20, 5, 1, 1, 9] + [1] * 14):
            dec.reset()
            assert rel_err(run_portions(dec, tok, sizes), ref).max() < F32_TOL
    finally:
        dec.close()
        model.close()


# ------------------------------------------------------------------ whole models
@pytest.mark.parametrize("name", ["mixed", "odd", "wide", "no_router"])
def test_residual_stream_after_every_layer_run(rt, name):
    from yalm_amd import models as M

    cfg = C.ALL[name]
    model, dec, w = build(rt, cfg, M.F32, seed=2)
    try:
        tok = C.tokens(cfg, 57, 2)
        layers = []
        R.forward(cfg, w, tok, layers_out=layers)
        assert len(layers) == len(model.cfg.layers) == len(R.run_order(cfg))
        dec.layer_dump(True)
        dec.step(tok)
        got = dec.get_layers(len(tok))
        for i, ref in enumerate(layers):
            e = np.abs(got[i] - ref).max() / np.abs(ref).max()
            assert e < 1e-4, f"layer run {i}: {e}"
    finally:
        dec.close()
        model.close()


@pytest.mark.parametrize("name", ["mixed", "odd", "wide", "no_router"])
@pytest.mark.parametrize("dtype", ["f32", "bf16"])
def test_prefill_then_token_by_token(rt, name, dtype):
    """A prompt in one step, then single tokens through the caches and states."""
    cfg = C.ALL[name]
    model, dec, w = build(rt, cfg, wdt_of(dtype), seed=3, max_tokens=700)
    try:
        n = 420 if name in ("wide", "no_router") else 150
        tok = C.tokens(cfg, n, 3)
        ref = R.forward(cfg, w, tok)
        assert agrees(run_portions(dec, tok, [n - 60] + [1] * 60), ref, dtype, cfg)
        dec.reset()
        assert agrees(dec.step(tok, list(range(n))), ref, dtype, cfg)
    finally:
        dec.close()
        model.close()


PORTIONS = [[2] * 30, [3, 2, 9, 8, 2, 64, 65], [1, 2, 3, 4, 5, 6, 7, 8, 9, 10], [128, 2, 2, 1, 40], [7, 200]]


@pytest.mark.parametrize("name", ["mixed", "odd", "wide"])
@pytest.mark.parametrize("sizes", PORTIONS, ids=[str(i) for i in range(len(PORTIONS))])
def test_portions_of_any_size(rt, name, sizes):
    """Portions cut anywhere (inside recurrence chunks and attention tiles, down to two tokens)
    against the whole sequence; the GEMV / tile switch (8 | 9 tokens, which is also where the log
    gates move out of the recurrence kernel) and tile edges (64 | 65) included."""
    from yalm_amd import models as M

    cfg = C.ALL[name]
    model, dec, w = build(rt, cfg, M.F32, seed=4)
    try:
        tok = C.tokens(cfg, 260, 4)
        ref = R.forward(cfg, w, tok)
        assert rel_err(run_portions(dec, tok, sizes), ref).max() < F32_TOL
    finally:
        dec.close()
        model.close()


def test_portions_bf16_differ_by_rounding_only(rt):
    from yalm_amd import models as M

    cfg = C.NO_ROUTER
    model, dec, w = build(rt, cfg, M.BF16, seed=5, max_tokens=700)
    try:
        tok = C.tokens(cfg, 600, 5)
        ref = R.forward(cfg, w, tok)
        for sizes in ([600], [300, 2, 170, 1, 1, 1], [64] * 9):
            dec.reset()
            assert rel_err(run_portions(dec, tok, sizes), ref).max() < BF16_TOL
    finally:
        dec.close()
        model.close()


@pytest.mark.parametrize("loop", [None, (0, 1, 2), (1, 2, 1), (1, 3, 2), (0, 3, 3)])
def test_loops(rt, loop):
    """No loop, one pass, several passes over any part: every pass keeps its own keys, values and
    states (the single tokens would show a pass that reads another's)."""
    from yalm_amd import models as M

    small = C.pair(C.attn(heads=2, kv_heads=1, dim=8, vdim=8, r=C.rot(dims=4)), C.memory(heads=2, dim=8, vdim=8))
    cfg = C.config([(small, None), (small, C.moe(ff=8, shared=0)), (small, None)], width=40, vocab=61, loop=loop)
    model, dec, w = build(rt, cfg, M.F32, seed=6)
    try:
        assert len(model.cfg.layers) == len(R.run_order(cfg))
        tok = C.tokens(cfg, 60, 6)
        ref = R.forward(cfg, w, tok)
        if loop:
            off = {**w, "loop.step": np.zeros_like(w["loop.step"])}
            assert rel_err(R.forward(cfg, off, tok), ref).max() > 100 * F32_TOL
        for sizes in ([60], [25, 2, 3] + [1] * 30):
            dec.reset()
            assert rel_err(run_portions(dec, tok, sizes), ref).max() < F32_TOL
    finally:
        dec.close()
        model.close()


# ------------------------------------------------------------------ caches and states
def test_decoder_reused_after_reset(rt):
    """States and cache rows of an ended sequence must not leak into the next one: the second
    sequence on a reused decoder equals the same sequence on a fresh decoder bit for bit."""
    from yalm_amd import models as M

    cfg = C.MIXED
    model, dec, w = build(rt, cfg, M.F32, seed=8)
    fresh = rt.SeqDecoder(model)
    try:
        a, b = C.tokens(cfg, 90, 6), C.tokens(cfg, 41, 7)
        run_portions(dec, a, [50, 1, 1, 38])
        dec.reset()
        assert dec.pos == 0
        got = run_portions(dec, b, [20, 1, 20])
        want = run_portions(fresh, b, [20, 1, 20])
        assert np.array_equal(got, want)
        assert rel_err(got, R.forward(cfg, w, b)).max() < F32_TOL
    finally:
        dec.close()
        fresh.close()
        model.close()


def test_live_sequences_do_not_mix(rt):
    """Three decoders on one model, unequal requests, their steps interleaved: each equals its
    sequence alone."""
    from yalm_amd import models as M

    cfg = C.MIXED
    model, d1, w = build(rt, cfg, M.F32, seed=20)
    decs = [d1, rt.SeqDecoder(model), rt.SeqDecoder(model)]
    try:
        seqs = [C.tokens(cfg, n, 20 + n) for n in (60, 45, 33)]
        cuts = [(20, 1, 9, 30), (3, 30, 1, 11), (1, 1, 2, 29)]
        got, at = [[], [], []], [0, 0, 0]
        for step in range(4):
            for i in range(3):
                s = cuts[i][step]
                got[i].append(decs[i].step(seqs[i][at[i]:at[i] + s], list(range(s))))
                at[i] += s
        for i in range(3):
            assert rel_err(np.concatenate(got[i]), R.forward(cfg, w, seqs[i])).max() < F32_TOL
    finally:
        for d in decs:
            d.close()
        model.close()


def _marked_key_model(seed=9):
    """A model in which one token's key stands out for every query: constant queries (their bias), keys
    along that constant in proportion to the input's likeness to the marked token's, in entries the
    rotation leaves alone."""
    from yalm_amd import layered as Ly

    cfg = C.config([(C.pair(C.attn(heads=2, kv_heads=1, dim=24, vdim=16, scale=0.5, softcap=40.0, r=C.rot(dims=8)),
                            C.memory(heads=1, dim=4, vdim=4), 8.0, 0.02), None)], width=64, vocab=101)
    t = make(cfg, seed)
    marked, q = 100, t["l0.mix.left.q.b"]
    h = R.tanh_norm(t["embed"].astype(np.float64), f64(t), "l0.norm1")
    c = np.zeros(24)
    c[8:] = np.sign(np.random.default_rng(seed).standard_normal(16))
    hs = h - h.mean(0)
    row = hs[marked] / (hs[marked] @ hs[marked])  # 1 at the marked token, about the others' likeness elsewhere
    t["l0.mix.left.q"] = np.zeros_like(t["l0.mix.left.q"])
    t["l0.mix.left.q.b"] = np.tile(c, 2).astype(q.dtype)
    t["l0.mix.left.k"] = np.outer(c, row * 3.0).astype(np.float32)
    t["l0.mix.left.k.b"] = (-c * float(h.mean(0) @ row) * 3.0).astype(np.float32)
    t = {k: Ly.bf16_to_f32(Ly.f32_to_bf16(v)).reshape(v.shape) for k, v in t.items()}
    return cfg, t, marked


@pytest.mark.parametrize("dtype", ["f32", "bf16"])
def test_far_and_tile_edge_keys_decide_the_output(rt, dtype):
    """One marked key wins almost every later query's softmax wherever it lies: the first positions,
    both sides of the attention kernels' 32- and 64-key tiles and of single-token key splits, hundreds
    back; prompts, portions and decoded queries. Without that token the restatement's logits move by
    far more than the tolerance."""
    cfg, t, marked = _marked_key_model()
    model, dec, w = build(rt, cfg, wdt_of(dtype), max_tokens=600, tensors=t)
    try:
        n = 440
        base = [x % 100 for x in C.tokens(cfg, n, 9)]
        for j in (0, 1, 31, 32, 63, 64, 65, 127, 128, 255, 256, 319, 389):
            a = list(base)
            a[j] = marked
            P = []
            ref = R.forward(cfg, w, a, weights_out=P)
            assert min(p[390:, j].min() for p in P) > 0.5
            assert rel_err(R.forward(cfg, w, base)[390:], ref[390:]).min() > 3 * BF16_TOL
            for sizes in ([n], [390, 2, 8] + [1] * 40, [j + 1, 1, 20, 200]):
                dec.reset()
                e = rel_err(run_portions(dec, a, sizes), ref)
                assert e.max() < (F32_TOL if dtype == "f32" else BF16_TOL), (j, sizes[:3], int(e.argmax()))
    finally:
        dec.close()
        model.close()


def test_recurrent_states_carry_far(rt):
    """A token hundreds of positions back still shows in the logits through the memory (forget gates
    close to one), across portion cuts and single-token steps."""
    from yalm_amd import models as M

    cfg = C.config([(C.pair(C.attn(heads=1, kv_heads=1, dim=8, vdim=8, r=C.rot(dims=4)),
                            C.memory(heads=2, dim=16, vdim=8, gate_cap=12.0), 0.9, 5.0), None)], width=32, vocab=53)
    t = make(cfg, 12)
    t["l0.mix.left.v"] = np.zeros_like(t["l0.mix.left.v"])      # the attention carries nothing
    t["l0.mix.right.f.b"] = np.full_like(t["l0.mix.right.f.b"], 9.0)
    model, dec, w = build(rt, cfg, M.F32, max_tokens=400, tensors=t)
    try:
        a = C.tokens(cfg, 330, 12)
        b = list(a)
        b[3] = (b[3] + 5) % cfg["vocab"]
        ra, rb = R.forward(cfg, w, a), R.forward(cfg, w, b)
        assert np.median(rel_err(ra[300:], rb[300:])) > 10 * F32_TOL
        for tok, ref in ((a, ra), (b, rb)):
            for sizes in ([330], [2, 100, 17, 150] + [1] * 61):
                dec.reset()
                assert rel_err(run_portions(dec, tok, sizes), ref).max() < F32_TOL
    finally:
        dec.close()
        model.close()


def test_every_mechanism_shows_in_the_logits(rt):
    """Taking one mechanism out of the restatement moves it far beyond the tolerance: the engine
    agreeing with the whole restatement means it computes each."""
    from yalm_amd import models as M

    cfg = C.MIXED
    model, dec, w = build(rt, cfg, M.F32, seed=11)
    try:
        tok = C.tokens(cfg, 40, 10)
        ref = R.forward(cfg, w, tok)

        def without(**changed):
            return rel_err(R.forward(cfg, {**w, **changed}, tok), ref).max()

        def other(path, value):
            c = copy.deepcopy(cfg)
            node = c
            for k in path[:-1]:
                node = node[k]
            node[path[-1]] = value
            return rel_err(R.forward(c, w, tok), ref).max()

        big = 50 * F32_TOL
        for name in ("l0.norm1", "l0.norm2", "final.norm", "l0.mix.right.norm", "l3.norm2.alpha", "final.norm.alpha"):
            assert without(**{name: np.ones_like(w[name])}) > big, name
        for name in ("l0.norm1.b", "l0.norm2.b", "final.norm.b", "l0.mix.left.q.b", "l0.mix.left.k.b", "l0.mix.left.v.b",
                     "l0.mix.left.o.b", "l0.mix.left.g", "l0.mix.right.g", "l0.mix.right.i.b", "l0.mix.right.f.b",
                     "l0.mlp.correction", "l0.mlp.shared.down", "loop.step"):
            assert without(**{name: np.zeros_like(w[name])}) > big, name
        left = ["layers", 0, "mixer", "left"]
        assert other(left + ["softcap"], None) > big
        assert other(left + ["rot", "dims"], 0) > big
        assert other(left + ["rot", "scaling"], None) > big
        assert other(["layers", 1, "mixer", "right", "gate_cap"], 5.0) > big
        assert other(["layers", 0, "mixer", "left_scale"], 1.0) > big
        assert other(["layers", 0, "mixer", "right_scale"], 1.0) > big
        assert other(["residual_mult"], 1.0) > big
        assert other(["logit_softcap"], None) > big
        assert rel_err(dec.step(tok, list(range(40))), ref).max() < F32_TOL
    finally:
        dec.close()
        model.close()


@pytest.mark.parametrize("n", [1, 2, 3, 5])
def test_first_tokens(rt, n):
    """The memory's first writes from its zero state, one visible key."""
    from yalm_amd import models as M

    cfg = C.MIXED
    model, dec, w = build(rt, cfg, M.F32, seed=12)
    try:
        tok = C.tokens(cfg, n, 9)
        ref = R.forward(cfg, w, tok)
        assert rel_err(dec.step(tok, list(range(n))), ref).max() < F32_TOL
        dec.reset()
        assert rel_err(run_portions(dec, tok, [1] * n), ref).max() < F32_TOL
    finally:
        dec.close()
        model.close()


@pytest.mark.parametrize("name", ["odd", "mixed"])
def test_long_decoding(rt, name):
    """200 single tokens: the states are carried through 200 steps."""
    from yalm_amd import models as M

    cfg = C.ALL[name]
    model, dec, w = build(rt, cfg, M.F32, seed=13)
    try:
        tok = C.tokens(cfg, 5 + 200, 10)
        got = run_portions(dec, tok, [5] + [1] * 200)
        assert rel_err(got, R.forward(cfg, w, tok)).max() < F32_TOL
    finally:
        dec.close()
        model.close()


def test_greedy_generation(rt):
    """The device greedy loop (no host round trip) picks the restatement's tokens, and the
    sequence can be continued by ordinary steps afterwards."""
    from yalm_amd import models as M

    cfg = C.MIXED
    model, dec, w = build(rt, cfg, M.F32, seed=14)
    try:
        prompt = C.tokens(cfg, 12, 11)
        dec.step(prompt[:-1])
        gen = dec.generate_greedy(prompt[-1], 40)
        seq = list(prompt)
        for g in gen:
            lg = R.forward(cfg, w, seq)[-1]
            top2 = np.sort(lg)[-2:]
            assert top2[1] - top2[0] > 1e-3, "the test's model has a near tie; pick another seed"
            assert int(np.argmax(lg)) == g
            seq.append(g)
        assert dec.pos == len(prompt) - 1 + len(gen)
        nxt = dec.step([gen[-1]], [0])
        assert rel_err(nxt, R.forward(cfg, w, seq)[-1:]).max() < F32_TOL
    finally:
        dec.close()
        model.close()


def test_greedy_graph_replays_match_eager_steps(rt):
    """The greedy loop replays one captured token graph. Several generate calls with ordinary
    (eager) steps and synchronisations between them: every replayed token equals the argmax of
    an eager step of a second decoder fed the same tokens."""
    from yalm_amd import models as M

    cfg = C.MIXED
    model, dec, w = build(rt, cfg, M.BF16, seed=15)
    eager = rt.SeqDecoder(model)
    try:
        prompt = C.tokens(cfg, 9, 16)
        dec.step(prompt[:-1])
        eager.step(prompt[:-1])
        tok = prompt[-1]
        for n in (3, 1, 6, 2):
            gen = dec.generate_greedy(tok, n)
            for g in gen:
                lg = eager.step([tok], [0])[0]
                assert int(np.argmax(lg)) == g
                tok = g
            extra = C.tokens(cfg, 2, 17 + n)
            a = dec.step(extra, [1])
            b = eager.step(extra, [1])
            assert np.array_equal(a, b)
            tok = int(np.argmax(a[0]))
        assert dec.pos == eager.pos
    finally:
        dec.close()
        eager.close()
        model.close()


_LONG_REF = {}


@pytest.mark.parametrize("dtype", ["f32", "bf16"])
def test_prompt_longer_than_one_internal_portion(rt, dtype):
    """A step of more tokens than the engine's work buffers hold (4096) is cut inside the engine;
    asked rows on both sides of the cut come back in order. The running maximum is carried over it."""
    cfg = C.config([(C.pair(C.attn(heads=2, kv_heads=1, dim=8, vdim=8, scale=0.35, r=C.rot(dims=8, original=900)),
                            C.memory(heads=2, dim=8, vdim=8)), None)], width=32, vocab=53)
    model, dec, w = build(rt, cfg, wdt_of(dtype), seed=16, max_tokens=4300)
    try:
        tok = C.tokens(cfg, 4200, 15)
        want = [0, 5, 3999, 4000, 4094, 4095, 4096, 4097, 4150, 4199]
        got = dec.step(tok, want)
        assert dec.pos == len(tok)
        if "ref" not in _LONG_REF:  # the same weights and tokens for both matrix types
            _LONG_REF["ref"] = R.forward(cfg, w, tok)[want]
        assert rel_err(got, _LONG_REF["ref"]).max() < (F32_TOL if dtype == "f32" else BF16_TOL)
    finally:
        dec.close()
        model.close()


@pytest.mark.parametrize("dtype", ["f32", "bf16"])
@pytest.mark.parametrize("dim,vdim", [(256, 128), (64, 200)])
def test_large_head_sizes(rt, dim, vdim, dtype):
    """The largest head sizes the kernels take, on both sides of a pair."""
    cfg = C.config([(C.pair(C.attn(heads=4, kv_heads=2, dim=dim, vdim=vdim, scale=0.06, r=C.rot(dims=dim // 2)),
                            C.memory(heads=2, dim=dim, vdim=vdim)), None)], width=128, vocab=101)
    model, dec, w = build(rt, cfg, wdt_of(dtype), seed=22, max_tokens=400)
    try:
        tok = C.tokens(cfg, 330, 22)
        ref = R.forward(cfg, w, tok)
        assert agrees(run_portions(dec, tok, [270, 5, 2, 20, 9] + [1] * 24), ref, dtype, cfg)
    finally:
        dec.close()
        model.close()


def test_portions_on_the_large_tiles(rt):
    """Sizes whose products of long portions take the large-tile GEMM (exact-gelu epilogue, a joint
    projection with a ragged last tile), bf16 against the restatement."""
    from yalm_amd import models as M

    cfg = C.config([(C.pair(C.attn(heads=4, kv_heads=2, dim=64, vdim=64, scale=0.125, r=C.rot(dims=32)),
                            C.memory(heads=3, dim=64, vdim=64)), C.moe(experts=4, identity=2, top=6, ff=128, shared=256))],
                   width=256, vocab=307)
    model, dec, w = build(rt, cfg, M.BF16, seed=24, max_tokens=400)
    try:
        tok = C.tokens(cfg, 330, 24)
        ref = R.forward(cfg, w, tok)
        got = dec.step(tok, list(range(330)))  # every output is chosen by every token: no near-tie can flip
        assert rel_err(got, ref).max() < BF16_TOL
    finally:
        dec.close()
        model.close()


def test_stream_wider_than_the_register_seam(rt):
    """A width above 4096 takes the seam kernel that keeps the row in LDS and the embedding / norm
    kernels' strided loops."""
    from yalm_amd import models as M

    small = C.pair(C.attn(heads=2, kv_heads=1, dim=16, vdim=8), C.memory(heads=2, dim=8, vdim=8))
    cfg = C.config([(small, C.moe(experts=3, identity=2, top=3, ff=8, shared=8)), (small, None)], width=4104, vocab=41,
                   loop=(0, 1, 2))
    model, dec, w = build(rt, cfg, M.F32, seed=23, max_tokens=64)
    try:
        tok = C.tokens(cfg, 40, 23)
        ref = R.forward(cfg, w, tok)
        assert rel_err(run_portions(dec, tok, [12, 3, 9] + [1] * 16), ref).max() < F32_TOL
    finally:
        dec.close()
        model.close()


def test_bad_configurations_are_refused(rt):
    """What the kernels do not do is an error at creation, not a wrong result."""
    from yalm_amd import layered as Ly
    from yalm_amd import models as M

    cfg = C.config([(C.pair(), C.moe())])
    t = make(cfg, 25)
    c = Ly.faguzen_config(cfg, max_tokens=64, weight_dtype=M.F32)
    p = Ly.faguzen_pack(c, t, cfg)

    def refused(**changed):
        spec = dataclasses.replace(c.layers[0], **changed)
        model = rt.SeqModel.from_packed(c.with_(layers=[spec]), p)
        try:
            with pytest.raises(rt.YalmError):
                rt.SeqDecoder(model)
        finally:
            model.close()

    refused(router_kind=Ly.ROUTER_TOP_SOFTMAX)          # identity outputs with another router
    refused(top=9)                                       # more than experts + identity outputs
    refused(ff_act=Ly.ACT_SILU)                          # a gated activation without gate matrices
    refused(rot_pairs=2)
    refused(softcap=-1.0)
    refused(out_gate=Ly.GATE_HEAD)                       # a per-head gate with a shared projection
    refused(side=dataclasses.replace(c.layers[0].side, gate_cap=0.0))
    refused(side=dataclasses.replace(c.layers[0].side, dim=300))


def test_sequence_cannot_pass_max_tokens(rt):
    from yalm_amd import models as M

    model, dec, _ = build(rt, C.ONLY_PAIR, M.F32, seed=13, max_tokens=16)
    try:
        dec.step(C.tokens(C.ONLY_PAIR, 16, 0))
        with pytest.raises(rt.YalmError):
            dec.step([1])
    finally:
        dec.close()
        model.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_runner(rt, tmp_path, dtype):
    """bin/trace_run on a checkpoint folder written here: two requests one after the other,
    in portions, the second on the decoder the first gave back."""
    from yalm_amd import layered as Ly
    from yalm_amd.yalmfile import write_yalm

    cfg = C.NO_ROUTER if dtype == "bfloat16" else C.MIXED
    t = make(cfg, 16)
    mdir = tmp_path / "model"
    mdir.mkdir()
    (mdir / "config.json").write_text(json.dumps(cfg))
    write_yalm(str(mdir / "model.safetensors"), {k: Ly.f32_to_bf16(v).reshape(v.shape) for k, v in t.items()}, {},
               {k: "BF16" for k in t})
    a, b = C.tokens(cfg, 30, 12), C.tokens(cfg, 19, 13)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:20], "want": [19, 0, 7]}], "end": []},
        {"step": 1, "entries": [{"id": "a", "tokens": a[20:22], "want": []}], "end": []},
        {"step": 2, "entries": [{"id": "a", "tokens": a[22:], "want": [7]}], "end": ["a"]},
        {"step": 3, "entries": [{"id": "b", "tokens": b[:18], "want": [17]}], "end": []},
        {"step": 4, "entries": [{"id": "b", "tokens": b[18:], "want": [0]}], "end": ["b"]},
    ]
    out = tmp_path / "out"
    p = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(mdir), "--dtype", dtype, "--out", str(out),
                        "--max-tokens", "64"], input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True,
                       text=True, timeout=300)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.splitlines() if l.startswith("done")] == ["done %d" % i for i in range(5)]
    assert not (out / "1.f32").exists()
    w = f64(t)
    ra, rb = R.forward(cfg, w, a), R.forward(cfg, w, b)
    lim = F32_TOL if dtype == "float32" else BF16_TOL
    V = cfg["vocab"]
    assert rel_err(np.fromfile(out / "0.f32", "<f4").reshape(-1, V), ra[[19, 0, 7]]).max() < lim
    assert rel_err(np.fromfile(out / "2.f32", "<f4").reshape(-1, V), ra[[29]]).max() < lim
    assert rel_err(np.fromfile(out / "3.f32", "<f4").reshape(-1, V), rb[[17]]).max() < lim
    assert rel_err(np.fromfile(out / "4.f32", "<f4").reshape(-1, V), rb[[18]]).max() < lim
