"""MI355X: the layer-list engine serving Gugozen models against the plain float64 restatement
in tests/gugozen_ref.py, on small random models made here.

Errors are per position: || got - ref || / || ref || over the vocabulary. With f32 matrices
the engine differs from the restatement by f32 rounding only (F32_TOL); with bf16 matrices by
the rounding of the products' inputs and of the cached rows (BF16_TOL; a model with routed
experts may miss it at a few positions where that rounding flips a router near-tie). A lost key,
a pair row of the wrong tokens, a norm's bias left out, a weight on the wrong side of an expert, a
state that is not carried or a token one place off moves the logits by orders of magnitude more
than F32_TOL.
"""
import copy
import dataclasses
import json
import os
import subprocess

import numpy as np
import pytest

import gugozen_cases as C
import gugozen_ref as R

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
F32_TOL, BF16_TOL = 2e-4, 6e-2


@pytest.fixture(scope="module")
def rt():
    from yalm_amd import runtime

    runtime.check(runtime.lib.yalm_set_device(0))
    return runtime


def make(cfg, seed=0, **kw):
    from yalm_amd import layered as Ly

    return Ly.gugozen_random_tensors(cfg, seed=seed, **kw)


def rounded(t):
    from yalm_amd import layered as Ly

    return {k: Ly.bf16_to_f32(Ly.f32_to_bf16(v)).reshape(v.shape) for k, v in t.items()}


def f64(t):
    return {k: v.astype(np.float64) for k, v in t.items()}


def build(rt, cfg, wdt, seed=0, max_tokens=512, tensors=None):
    from yalm_amd import layered as Ly

    t = tensors if tensors is not None else make(cfg, seed)
    c = Ly.gugozen_config(cfg, max_tokens=max_tokens, weight_dtype=wdt, shapes={k: v.shape for k, v in t.items()})
    model = rt.SeqModel.from_packed(c, Ly.gugozen_pack(c, t))
    return model, rt.SeqDecoder(model), f64(t)


def rel_err(got, ref):
    return np.linalg.norm(got - ref, axis=-1) / np.linalg.norm(ref, axis=-1)


def wdt_of(dtype):
    from yalm_amd import models as M

    return M.F32 if dtype == "f32" else M.BF16


def close_calls(cfg):
    """Has a router that chooses (top = all experts leaves nothing to flip)."""
    return any(e.get("mlp") and e["mlp"]["router"]["top"] < e["mlp"]["router"]["experts"] for e in cfg["layers"])


def agrees(got, ref, dtype, cfg):
    e = rel_err(got, ref)
    if dtype == "f32":
        return e.max() < F32_TOL
    if close_calls(cfg):  # a flipped near-tie of a router: a few positions, never the bulk
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


def check_sizes(dec, tok, ref, cuts, dtype="f32", cfg=None):
    for sizes in cuts:
        dec.reset()
        got = run_portions(dec, tok, sizes)
        assert agrees(got, ref, dtype, cfg or {"layers": []}), (sizes[:4], rel_err(got, ref).max())


# ------------------------------------------------------------------ mechanisms alone
@pytest.mark.parametrize("name", ["only_latent", "only_shared", "only_attn", "only_gla", "only_moe"])
@pytest.mark.parametrize("dtype", ["f32", "bf16"])
def test_each_sublayer_kind_alone(rt, name, dtype):
    cfg = C.ALL[name]
    model, dec, w = build(rt, cfg, wdt_of(dtype), seed=1)
    try:
        tok = C.tokens(cfg, 90, 1)
        check_sizes(dec, tok, R.forward(cfg, w, tok), ([90], [30] + [1] * 60, [40, 2, 9, 8, 31]), dtype, cfg)
    finally:
        dec.close()
        model.close()


@pytest.mark.parametrize("bigram", [(73, 29, 11), (1, 5, 3), (1000, 0, 1), (977, 3000000019, 4000000007)],
                         ids=["small", "one_bucket", "no_previous", "beyond_32_bits"])
def test_pair_embedding(rt, bigram):
    """The row of a token and the one before it: the first token's own row, a cut between the two, the
    single-token path, a row hash that needs 64 bits, and a sequence that starts over."""
    from yalm_amd import models as M

    cfg = C.config([(C.TINY, None)], width=40, vocab=61, bigram=bigram)
    model, dec, w = build(rt, cfg, M.F32, seed=2)
    try:
        tok = C.tokens(cfg, 40, 2)
        ref = R.forward(cfg, w, tok)
        off = {**w, "bigram": np.concatenate([w["bigram"][:-1], np.zeros_like(w["bigram"][-1:])])}
        assert rel_err(R.forward(cfg, off, tok), ref)[0] > 100 * F32_TOL
        if bigram[1] and bigram[0] > 1:
            twisted = copy.deepcopy(cfg)
            twisted["embedding"]["bigram"].update(mul_prev=bigram[2], mul_cur=bigram[1])
            assert np.median(rel_err(R.forward(twisted, w, tok), ref)) > 100 * F32_TOL
        check_sizes(dec, tok, ref, ([40], [1] * 40, [2] * 20, [13, 1, 9, 1, 8]))
    finally:
        dec.close()
        model.close()


def test_without_a_pair_embedding(rt):
    from yalm_amd import models as M

    cfg = C.config([(C.gla(), C.moe())], bigram=None)
    model, dec, w = build(rt, cfg, M.F32, seed=3)
    try:
        tok = C.tokens(cfg, 40, 3)
        check_sizes(dec, tok, R.forward(cfg, w, tok), ([40], [7] + [1] * 33))
    finally:
        dec.close()
        model.close()


def engine_norm(kind, x, v, n, eps):
    """The engine's norm kinds on vectors in its own layout."""
    from yalm_amd import layered as Ly

    if kind == Ly.NORM_TANH:
        return np.tanh(v[2 * n] * x) * v[:n] + v[n:2 * n]
    if kind == Ly.NORM_RMS:
        return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps) * v[:n]
    d = x - x.mean(-1, keepdims=True)
    return d / np.sqrt((d * d).mean(-1, keepdims=True) + eps) * v[:n] + (v[n:2 * n] if kind == Ly.NORM_LAYER_BIAS else 0.0)


NORM_KINDS = ["NORM_RMS", "NORM_LAYER", "NORM_TANH", "NORM_LAYER_BIAS"]
ENVELOPES = [("post", k) for k in NORM_KINDS] + [("serial", "NORM_LAYER_BIAS"), ("closing", "NORM_LAYER_BIAS"),
                                                 ("parallel", "NORM_LAYER_BIAS")]


@pytest.mark.parametrize("width", [96, 1100, 2056, 4104])
@pytest.mark.parametrize("envelope,kind", ENVELOPES)
def test_norms_and_envelopes(rt, envelope, kind, width):
    """The post-norm block takes every norm kind, and the layer norm with a bias every block: opening and
    closing norms, closing norms alone (a single token's are folded into the next product), parallel
    blocks with a norm per sublayer; seams with the row in registers and in LDS, weights on the
    experts' inputs in every seam, the model's residual scale."""
    from yalm_amd import layered as Ly
    from yalm_amd import models as M

    cfg = C.config([(C.attn(heads=2, kv_heads=1, dim=16, vdim=8), C.moe(experts=3, top=2, ff=8, shared=8)),
                    (C.attn(heads=1, kv_heads=1, dim=8, vdim=12), None),
                    (C.attn(heads=2, kv_heads=2, dim=8, vdim=8), None)], width=width, vocab=53)
    t = make(cfg, 4)
    w = f64(t)
    k = getattr(Ly, kind)
    n, eps, rs = width, cfg["norm"]["eps"], 0.7
    shapes = {a: b.shape for a, b in t.items()}
    base = Ly.gugozen_config(cfg, max_tokens=64, weight_dtype=M.F32, shapes=shapes)
    packed = Ly.gugozen_pack(base, t)
    block = {"post": Ly.BLOCK_POST, "parallel": Ly.BLOCK_PARALLEL}.get(envelope, Ly.BLOCK_SERIAL)
    pre = envelope in ("serial", "parallel")
    specs = [dataclasses.replace(l, ff_normed=True, layer_scaled=False) if envelope == "parallel" else l for l in base.layers]
    c = base.with_(norm_kind=k, block_kind=block, pre_norm=pre, residual_scale=rs, layers=specs)
    rng = np.random.default_rng(6)
    size = Ly.norm_shape(c)[0]

    def vector():
        v = np.concatenate([rng.uniform(0.5, 1.5, n), 0.3 * rng.standard_normal(n), [0.8]])[:size]
        return v.astype(np.float32)

    vs = [{name: vector() for name in Ly.packed_shapes(c, l) if name.startswith("norm")} for l in specs]
    final = vector()
    layers = [{**{a: b for a, b in d.items() if not a.startswith("norm")}, **v} for d, v in zip(packed["layers"], vs)]
    model = rt.SeqModel.from_packed(c, dict(packed, layers=layers, final_norm=final))
    dec = rt.SeqDecoder(model)
    try:
        tok = C.tokens(cfg, 30, 4)

        def norm(x, v):
            return engine_norm(k, x, v.astype(np.float64), n, eps)

        x = R.embedding(cfg, w, tok)
        for i, (e, v) in enumerate(zip(cfg["layers"], vs)):
            p = f"l{i}."

            def mix(h):
                return R.mixer_attention(cfg, w, p + "mix.", h, e["mixer"])

            def ff(h):
                return R.feed_forward(w, p + "mlp.", h, e["mlp"])

            if envelope == "parallel":
                y = mix(norm(x, v["norm1"]))
                x = x + rs * (y + ff(norm(x, v["norm2"])) if e["mlp"] else y)
                continue
            for f, a, b in ((mix, "norm1", "norm1b"),) + (((ff, "norm2", "norm2b"),) if e["mlp"] else ()):
                y = rs * f(norm(x, v[a]) if pre else x)
                x = norm(cfg["postln_alpha"] * x + y, v[b]) if envelope == "post" else x + rs * norm(y / rs, v[b])
        ref = norm(x, final) @ w["embed"].T
        check_sizes(dec, tok, ref, ([30], [12] + [1] * 18, [2, 9, 8]))
    finally:
        dec.close()
        model.close()


@pytest.mark.parametrize("tau,bias", [(0.5, 0.0), (1.0, -4.0), (1.0, 4.0), (16.0, -2.0), (40.0, 1.0)])
def test_gla_decays(rt, tau, bias):
    """Decays from nearly nothing kept to nearly everything kept, on both sides of tau = 1."""
    from yalm_amd import models as M

    cfg = C.config([(C.gla(heads=4, dim=24, vdim=20, tau=tau), None)])
    t = make(cfg, 5, decay_rank=5)
    t["l0.mix.a2.b"] = (t["l0.mix.a2.b"] * 0.3 + bias).astype(np.float32)
    t = rounded(t)
    model, dec, w = build(rt, cfg, M.F32, tensors=t)
    try:
        tok = C.tokens(cfg, 110, 5)
        ref = R.forward(cfg, w, tok)
        other = copy.deepcopy(cfg)
        other["layers"][0]["mixer"]["tau"] = tau * 1.5
        assert rel_err(R.forward(other, w, tok), ref).max() > 5 * F32_TOL
        check_sizes(dec, tok, ref, ([110], [33, 2, 16, 15] + [1] * 44, [8, 9, 1, 17]))
    finally:
        dec.close()
        model.close()


@pytest.mark.parametrize("dtype", ["f32", "bf16"])
@pytest.mark.parametrize("dim,vdim,heads", [(8, 4, 1), (32, 70, 3), (33, 16, 2), (64, 33, 2), (65, 8, 2), (200, 24, 2), (256, 40, 1)])
def test_gla_sizes(rt, dim, vdim, heads, dtype):
    """Every instantiation of the recurrence kernel and both sides of its switches."""
    cfg = C.config([(C.gla(heads=heads, dim=dim, vdim=vdim, tau=4.0), None)], width=64, vocab=101)
    model, dec, w = build(rt, cfg, wdt_of(dtype), seed=6)
    try:
        tok = C.tokens(cfg, 70, 6)
        check_sizes(dec, tok, R.forward(cfg, w, tok), ([70], [20, 3] + [1] * 47), dtype, cfg)
    finally:
        dec.close()
        model.close()


def test_gla_with_a_sigmoid_gate(rt):
    """The gate's activation is a parameter of the mixer."""
    from yalm_amd import layered as Ly
    from yalm_amd import models as M

    cfg = C.ONLY_GLA
    t = make(cfg, 7)
    c = Ly.gugozen_config(cfg, max_tokens=64, weight_dtype=M.F32, shapes={k: v.shape for k, v in t.items()})
    model = rt.SeqModel.from_packed(c.with_(layers=[dataclasses.replace(c.layers[0], gate_act=Ly.DELTA_GATE_SIGMOID)]),
                                    Ly.gugozen_pack(c, t))
    dec = rt.SeqDecoder(model)
    keep = R.silu
    try:
        tok = C.tokens(cfg, 30, 7)
        R.silu = R.sigmoid
        check_sizes(dec, tok, R.forward(cfg, f64(t), tok), ([30], [11] + [1] * 19))
    finally:
        R.silu = keep
        dec.close()
        model.close()


@pytest.mark.parametrize("dtype", ["f32", "bf16"])
@pytest.mark.parametrize("far", [False, True])
def test_latent_rows_of_another_layer(rt, far, dtype):
    """A layer that reads the rows of the layer before it, or of one several layers back, with its own
    heads and up-projections; another source's rows would show."""
    mid = [(C.gla(heads=2, dim=8, vdim=8), None), (C.latent(heads=2, dim=8, vdim=8), None)] if far else []
    cfg = C.config([(C.latent(), None)] + mid + [(C.latent(heads=4, dim=16, vdim=24, scale=0.3, kv_from=0), None),
                                                 (C.latent(heads=1, dim=40, vdim=8, kv_from=0), None)])
    model, dec, w = build(rt, cfg, wdt_of(dtype), seed=8)
    try:
        assert model.cfg.layers[-1].kv_from == 0
        tok = C.tokens(cfg, 110, 8)
        ref = R.forward(cfg, w, tok)
        if far:
            other = copy.deepcopy(cfg)
            other["layers"][-1]["mixer"]["kv_from"] = 2
            assert rel_err(R.forward(other, w, tok), ref).max() > BF16_TOL
        check_sizes(dec, tok, ref, ([110], [50, 2, 8, 9] + [1] * 41), dtype, cfg)
    finally:
        dec.close()
        model.close()


@pytest.mark.parametrize("pairs", ["ROT_INTERLEAVED", "ROT_HALVES"])
@pytest.mark.parametrize("dims", [0, 4, 12])
def test_latent_rotation_layouts(rt, pairs, dims):
    """Both pair layouts over none, some and all of the rotated part, put together by hand; the sink and
    the window of the latent mixer beside its output gate."""
    from yalm_amd import layered as Ly
    from yalm_amd import models as M

    cfg = C.config([(C.latent(heads=3, dim=8, rot_dim=12, vdim=16, scale=0.5, base=20.0), None)])
    t = make(cfg, 9)
    w = f64(t)
    c = Ly.gugozen_config(cfg, max_tokens=128, weight_dtype=M.F32, shapes={k: v.shape for k, v in t.items()})
    spec = dataclasses.replace(c.layers[0], rot_pairs=getattr(Ly, pairs), rot_dims=dims)
    model = rt.SeqModel.from_packed(c.with_(layers=[spec]), Ly.gugozen_pack(c, t))
    dec = rt.SeqDecoder(model)
    keep = R.rotate_halves

    def rotate(x, r):
        if dims == 0:
            return x
        part = {"dims": dims, "base": r["base"]}
        if pairs == "ROT_HALVES":
            return keep(x, part)
        order = [2 * i for i in range(dims // 2)] + [2 * i + 1 for i in range(dims // 2)] + list(range(dims, x.shape[-1]))
        out = np.empty_like(x)
        out[..., order] = keep(x[..., order], part)
        return out

    try:
        tok = C.tokens(cfg, 90, 9)
        R.rotate_halves = rotate
        ref = R.forward(cfg, w, tok)
        R.rotate_halves = keep
        if dims < 12 or pairs != "ROT_HALVES":
            assert rel_err(R.forward(cfg, w, tok), ref).max() > 50 * F32_TOL
        check_sizes(dec, tok, ref, ([90], [40, 2, 7] + [1] * 41))
    finally:
        R.rotate_halves = keep
        dec.close()
        model.close()


MLPS = [C.moe(), C.moe(experts=5, top=1, ff=24, shared=0), C.moe(experts=3, top=3, ff=16, limit=0.05, shared=8, shared_limit=2.0),
        C.moe(experts=70, top=7, ff=8, limit=50.0, shared=0), C.moe(experts=1, top=1, ff=8, shared=16, shared_limit=0.1)]


@pytest.mark.parametrize("k", range(len(MLPS)))
def test_routed_experts_follow_the_restatement(rt, k):
    """Every token's chosen experts and weights, through the logits: top = 1, top = all experts, more
    experts than a wave has lanes, clamps that bite and that do not, with and without a shared expert;
    the weight sits on the expert's input, not on its output."""
    from yalm_amd import models as M

    mlp = MLPS[k]
    cfg = C.config([(C.TINY, mlp)], width=48, vocab=77)
    t = make(cfg, 41 + k)
    t["l0.mlp.router"] = t["l0.mlp.router"] * 2.0
    model, dec, w = build(rt, cfg, M.F32, tensors=t)
    keep = R.feed_forward
    try:
        tok = C.tokens(cfg, 50, 41)
        picks = []
        ref = R.forward(cfg, w, tok, choice_out=picks)
        if mlp["router"]["top"] < mlp["router"]["experts"]:
            assert len({tuple(sorted(i.tolist())) for i, _ in picks}) > 1

        def on_output(w, pre, h, mlp, choice_out=None):
            out = np.zeros_like(h)
            for s in range(len(h)):
                for e, a in zip(*R.route(h[s] @ w[pre + "router"].T, mlp["router"]["top"])):
                    out[s] += a * R.expert(w, f"{pre}e{e}.", h[s:s + 1], mlp["expert"]["limit"])[0]
            return out + R.expert(w, pre + "shared.", h, mlp["shared"]["limit"]) if mlp.get("shared") else out

        R.feed_forward = on_output
        assert rel_err(R.forward(cfg, w, tok), ref).max() > 50 * F32_TOL
        R.feed_forward = keep
        check_sizes(dec, tok, ref, ([50], [20, 5, 1, 1, 9] + [1] * 14))
    finally:
        R.feed_forward = keep
        dec.close()
        model.close()


def test_router_orders_saturated_scores(rt):
    """Logits so large that every sigmoid rounds to one in f32 still rank by the logit."""
    from yalm_amd import models as M

    cfg = C.config([(C.TINY, C.moe(experts=9, top=2, ff=16))], width=48, vocab=77)
    t = make(cfg, 10)
    rng = np.random.default_rng(3)
    t["l0.norm1.b"] = np.full_like(t["l0.norm1.b"], 1.0)
    t["l0.mlp.router"] = (np.full_like(t["l0.mlp.router"], 1.0) + 0.2 * rng.standard_normal(t["l0.mlp.router"].shape)).astype(np.float32)
    t = rounded(t)
    model, dec, w = build(rt, cfg, M.F32, tensors=t)
    try:
        tok = C.tokens(cfg, 40, 10)
        picks = []
        ref = R.forward(cfg, w, tok, choice_out=picks)
        assert all((wt.astype(np.float32) == 1.0).all() for _, wt in picks) and len({tuple(i) for i, _ in picks}) > 3
        check_sizes(dec, tok, ref, ([40], [15] + [1] * 25))
    finally:
        dec.close()
        model.close()


@pytest.mark.parametrize("dtype", ["f32", "bf16"])
@pytest.mark.parametrize("sink", [-20.0, 0.0, 6.0])
def test_sink(rt, sink, dtype):
    """A sink that takes nothing, some and most of every softmax."""
    cfg = C.config([(C.attn(heads=4, kv_heads=2, dim=32, vdim=48, scale=0.3, r=C.rot(16)), None)])
    t = make(cfg, 11)
    t["l0.mix.sink"] = np.full_like(t["l0.mix.sink"], sink)
    model, dec, w = build(rt, cfg, wdt_of(dtype), tensors=t)
    try:
        tok = C.tokens(cfg, 130, 11)
        ref = R.forward(cfg, w, tok)
        if sink > -10:
            off = {**w, "l0.mix.sink": np.full_like(w["l0.mix.sink"], -1e9)}
            assert rel_err(R.forward(cfg, off, tok), ref).max() > 2 * BF16_TOL
        check_sizes(dec, tok, ref, ([130], [60] + [1] * 70, [5, 6, 40, 7]), dtype, cfg)
    finally:
        dec.close()
        model.close()


@pytest.mark.parametrize("r", [C.rot(24), C.rot(2), C.rot(10, 3.0), {"dims": 0, "base": 1.0}], ids=["all", "pair", "some", "none"])
def test_attention_rotation(rt, r):
    """Half-split pairs after the whole-projection norms."""
    from yalm_amd import models as M

    cfg = C.config([(C.attn(heads=6, kv_heads=3, dim=24, scale=0.4, r=r), None)])
    model, dec, w = build(rt, cfg, M.F32, seed=12)
    try:
        tok = C.tokens(cfg, 100, 12)
        check_sizes(dec, tok, R.forward(cfg, w, tok), ([100], [50, 3] + [1] * 47))
    finally:
        dec.close()
        model.close()


# ------------------------------------------------------------------ whole models
@pytest.mark.parametrize("name", ["mixed", "odd", "wide", "no_router"])
def test_residual_stream_after_every_layer(rt, name):
    from yalm_amd import models as M

    cfg = C.ALL[name]
    model, dec, w = build(rt, cfg, M.F32, seed=2)
    try:
        tok = C.tokens(cfg, 57, 2)
        layers = []
        R.forward(cfg, w, tok, layers_out=layers)
        dec.layer_dump(True)
        dec.step(tok)
        got = dec.get_layers(len(tok))
        assert len(layers) == len(got)
        for i, ref in enumerate(layers):
            e = np.abs(got[i] - ref).max() / np.abs(ref).max()
            assert e < 1e-4, f"layer {i}: {e}"
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
        check_sizes(dec, tok, R.forward(cfg, w, tok), ([n - 60] + [1] * 60, [n]), dtype, cfg)
    finally:
        dec.close()
        model.close()


PORTIONS = [[2] * 30, [3, 2, 9, 8, 2, 64, 65], [1, 2, 3, 4, 5, 6, 7, 8, 9, 10], [128, 2, 2, 1, 40], [7, 200], [31, 32, 33]]
_PORTION_REF = {}


@pytest.mark.parametrize("name", ["mixed", "odd", "wide"])
@pytest.mark.parametrize("sizes", PORTIONS, ids=[str(i) for i in range(len(PORTIONS))])
def test_portions_of_any_size(rt, name, sizes):
    """Portions cut anywhere (inside recurrence chunks and attention tiles, down to two tokens) against
    the whole sequence; the GEMV / tile switch (8 | 9 tokens), the switch between attending over latents
    and over expanded keys (31 | 32) and tile edges (64 | 65) included."""
    from yalm_amd import models as M

    cfg = C.ALL[name]
    model, dec, w = build(rt, cfg, M.F32, seed=4)
    try:
        tok = C.tokens(cfg, 260, 4)
        if name not in _PORTION_REF:  # the same weights and tokens for every cut
            _PORTION_REF[name] = R.forward(cfg, w, tok)
        check_sizes(dec, tok, _PORTION_REF[name], (sizes,))
    finally:
        dec.close()
        model.close()


def test_portions_bf16_differ_by_rounding_only(rt):
    from yalm_amd import models as M

    cfg = C.NO_ROUTER
    model, dec, w = build(rt, cfg, M.BF16, seed=5, max_tokens=700)
    try:
        tok = C.tokens(cfg, 600, 5)
        check_sizes(dec, tok, R.forward(cfg, w, tok), ([600], [300, 2, 170, 1, 1, 1], [64] * 9), "bf16", cfg)
    finally:
        dec.close()
        model.close()


# ------------------------------------------------------------------ caches and states
def test_decoder_reused_after_reset(rt):
    """States, cache rows and the previous token of an ended sequence must not leak into the next one:
    the second sequence on a reused decoder equals the same sequence on a fresh decoder bit for bit."""
    from yalm_amd import models as M

    cfg = C.MIXED
    model, dec, w = build(rt, cfg, M.F32, seed=8)
    fresh = rt.SeqDecoder(model)
    try:
        a, b = C.tokens(cfg, 90, 6), C.tokens(cfg, 41, 7)
        run_portions(dec, a, [50, 1, 1, 38])
        dec.generate_greedy(3, 5)
        dec.reset()
        assert dec.pos == 0
        got = run_portions(dec, b, [1, 20, 1, 19])
        want = run_portions(fresh, b, [1, 20, 1, 19])
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


def _marked_key_model(kind, seed=9):
    """A model in which one token's key stands out for every query of its (last) layer. Entry 0 of the
    stream is a constant every query reads, entry 1 marks the token: its key lies along the queries'
    common direction (in entries the rotation leaves alone), the others' keys are random."""
    mixer = {"attention": C.attn(heads=4, kv_heads=2, dim=24, vdim=16, scale=0.9, r=C.rot(8)),
             "latent": C.latent(heads=3, dim=16, rot_dim=8, vdim=16, kv_rank=24, scale=0.5),
             "shared": C.latent(heads=3, dim=16, rot_dim=8, vdim=16, kv_rank=24, scale=0.5)}[kind]
    layers = [(mixer, None)]
    if kind == "shared":
        layers.append((C.latent(heads=2, dim=12, rot_dim=8, vdim=20, kv_rank=24, scale=0.5, kv_from=0), None))
    cfg = C.config(layers, width=64, vocab=101, alpha=0.3)
    t = make(cfg, seed)
    rng, marked = np.random.default_rng(seed), 100
    t["embed"][:, 0], t["embed"][:, 1], t["embed"][marked, 1] = 3.0, 0.0, 4.0
    t["bigram"][:, :2] = 0.0
    for i, e in enumerate(cfg["layers"]):
        m, x = e["mixer"], f"l{i}.mix."
        H, D = m["heads"], m["dim"]
        t[f"l{i}.norm1.b"][0] = 4.0  # the constant survives the layer's norm
        t[f"l{i}.norm1"][0] = 0.1
        if e["type"] == "attention":
            c = np.zeros(D)
            c[8:] = np.sign(rng.standard_normal(D - 8))
            t[x + "q"] *= 0.1
            t[x + "q"][:, 0] = np.tile(c, H)
            t[x + "k"][:, 1] = 4.0 * np.tile(c, m["kv_heads"])
            t[x + "k"][:, 0] = 0.0
            t[x + "q.norm"][:] = t[x + "k.norm"][:] = 1.0
            t[x + "sink"][:] = -3.0
        else:
            R_ = m["rot_dim"]
            c = np.sign(rng.standard_normal(D))
            t[x + "q"] *= 0.1
            t[x + "q"][:, 0] = np.tile(np.concatenate([c, np.zeros(R_)]), H) * 0.5
            t[x + "uk"] *= 0.2
            t[x + "uk"][:, 0] = np.tile(c, H) * 0.4
            if f"{x}dkv" in t:
                t[x + "dkv"][0, :] = 0.0
                t[x + "dkv"][0, 1] = 6.0
                t[x + "dkv"][:, 0] = 0.0
                t[x + "dkv"][-R_:] *= 0.1
                t[x + "dkv.norm"][0] = 1.0
        t[x + "o"] *= 2.0
    return cfg, rounded(t), marked


@pytest.mark.parametrize("dtype", ["f32", "bf16"])
@pytest.mark.parametrize("kind", ["attention", "latent", "shared"])
def test_far_and_tile_edge_keys_decide_the_output(rt, kind, dtype):
    """One marked key wins every later query's softmax wherever it lies: the first positions, both sides
    of the attention kernels' 32- and 64-key tiles and of single-token key splits, hundreds back;
    prompts, portions and decoded queries. Without that token the restatement's logits move by far more
    than the tolerance."""
    cfg, t, marked = _marked_key_model(kind)
    model, dec, w = build(rt, cfg, wdt_of(dtype), max_tokens=600, tensors=t)
    try:
        n = 440
        base = [x % 100 for x in C.tokens(cfg, n, 9)]
        plain = R.forward(cfg, w, base)
        for j in (0, 1, 31, 32, 63, 64, 65, 127, 128, 255, 256, 319, 389):
            a = list(base)
            a[j] = marked
            P = []
            ref = R.forward(cfg, w, a, weights_out=P)
            assert min(p[391:, j].min() for p in P) > 0.5, min(p[391:, j].min() for p in P)
            assert rel_err(plain[391:], ref[391:]).min() > 2 * BF16_TOL
            check_sizes(dec, a, ref, ([n], [390, 2, 8] + [1] * 40, [j + 1, 1, 20, 200]), dtype, cfg)
    finally:
        dec.close()
        model.close()


def test_recurrent_states_carry_far(rt):
    """A token hundreds of positions back still shows in the logits through the linear attention's state
    (decays close to one), across portion cuts and single-token steps."""
    from yalm_amd import models as M

    cfg = C.config([(C.gla(heads=2, dim=16, vdim=8, tau=16.0), None)], width=32, vocab=53, alpha=0.5, bigram=None)
    t = make(cfg, 12)
    t["l0.mix.a2.b"] = np.full_like(t["l0.mix.a2.b"], 9.0)
    t["embed"][51:] *= 6.0
    t = rounded(t)
    model, dec, w = build(rt, cfg, M.F32, max_tokens=400, tensors=t)
    try:
        a = [x % 51 for x in C.tokens(cfg, 330, 12)]
        b = list(a)
        a[3], b[3] = 51, 52
        ra, rb = R.forward(cfg, w, a), R.forward(cfg, w, b)
        assert np.median(rel_err(ra[300:], rb[300:])) > 50 * F32_TOL
        for tok, ref in ((a, ra), (b, rb)):
            check_sizes(dec, tok, ref, ([330], [2, 100, 17, 150] + [1] * 61))
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

        big = 20 * F32_TOL
        for name in ("l0.norm1", "l0.norm2", "final.norm", "l0.mix.dkv.norm", "l1.mix.norm", "l2.mix.q.norm", "l2.mix.k.norm"):
            assert without(**{name: np.ones_like(w[name])}) > big, name
        for name in ("l0.norm1.b", "l0.norm2.b", "final.norm.b", "bigram", "l0.mix.g", "l3.mix.g", "l1.mix.g", "l1.mix.a2",
                     "l1.mix.a2.b", "l2.mix.sink", "l0.mlp.shared.down", "l3.mlp.router", "l7.mix.uk", "l7.mix.uv"):
            assert without(**{name: np.zeros_like(w[name])}) > big, name
        mixer = ["layers", 0, "mixer"]
        assert other(mixer + ["rot", "base"], 2.0) > big
        assert other(mixer + ["scale"], 0.4) > big
        assert other(["layers", 2, "mixer", "rot", "dims"], 8) > big
        assert other(["layers", 1, "mixer", "tau"], 1.0) > big
        assert other(["layers", 3, "mlp", "expert", "limit"], 7.0) > big
        assert other(["layers", 0, "mlp", "shared", "limit"], 7.0) > big
        assert other(["postln_alpha"], 1.0) > big
        assert rel_err(dec.step(tok, list(range(40))), ref).max() < F32_TOL
    finally:
        dec.close()
        model.close()


@pytest.mark.parametrize("n", [1, 2, 3, 5])
def test_first_tokens(rt, n):
    """The first writes into a zero state, one visible key, the first token's own pair row."""
    from yalm_amd import models as M

    cfg = C.MIXED
    model, dec, w = build(rt, cfg, M.F32, seed=12)
    try:
        tok = C.tokens(cfg, n, 9)
        check_sizes(dec, tok, R.forward(cfg, w, tok), ([n], [1] * n))
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
        check_sizes(dec, tok, R.forward(cfg, w, tok), ([5] + [1] * 200,))
    finally:
        dec.close()
        model.close()


def test_greedy_generation(rt):
    """The device greedy loop (no host round trip) picks the restatement's tokens, and the sequence can
    be continued by ordinary steps or another loop afterwards (the previous token crosses between host
    and device both ways)."""
    from yalm_amd import models as M

    cfg = C.MIXED
    model, dec, w = build(rt, cfg, M.F32, seed=14)
    try:
        seq = C.tokens(cfg, 12, 11)
        dec.step(seq[:-1])
        for n in (25, 1, 2, 12):
            gen = dec.generate_greedy(seq[-1], n)
            for g in gen:
                lg = R.forward(cfg, w, seq)[-1]
                top2 = np.sort(lg)[-2:]
                assert top2[1] - top2[0] > 1e-3, "the test's model has a near tie; pick another seed"
                assert int(np.argmax(lg)) == g
                seq.append(g)
            assert dec.pos == len(seq) - 1
            seq += [7, 4]
            nxt = dec.step(seq[-3:-1], [0, 1])
            assert rel_err(nxt, R.forward(cfg, w, seq[:-1])[-2:]).max() < F32_TOL
    finally:
        dec.close()
        model.close()


def test_greedy_loop_from_an_empty_sequence(rt):
    from yalm_amd import models as M

    cfg = C.MIXED
    model, dec, w = build(rt, cfg, M.F32, seed=14)
    try:
        for start in (5, 6):  # the second time after a reset
            seq = [start]
            for g in dec.generate_greedy(start, 6):
                assert int(np.argmax(R.forward(cfg, w, seq)[-1])) == g
                seq.append(g)
            dec.reset()
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
    asked rows on both sides of the cut come back in order, the pair of tokens across it included."""
    cfg = C.config([(C.attn(heads=2, kv_heads=1, dim=8, vdim=8, scale=0.35), None), (C.gla(heads=2, dim=8, vdim=8), None)],
                   width=32, vocab=53)
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
@pytest.mark.parametrize("dim,vdim,rank,rd", [(256, 128, 300, 64), (64, 200, 512, 32), (128, 128, 512, 64)])
def test_large_head_sizes(rt, dim, vdim, rank, rd, dtype):
    """Head sizes and latent ranks up to what real models use, on every kernel route."""
    cfg = C.config([(C.latent(heads=4, dim=min(dim, 160), rot_dim=rd, vdim=vdim, kv_rank=rank, scale=0.06), None),
                    (C.attn(heads=4, kv_heads=2, dim=dim, vdim=vdim, scale=0.06, r=C.rot(dim // 2)), None),
                    (C.latent(heads=3, dim=32, rot_dim=rd, vdim=64, kv_rank=rank, scale=0.06, kv_from=0), None)],
                   width=128, vocab=101)
    model, dec, w = build(rt, cfg, wdt_of(dtype), seed=22, max_tokens=400)
    try:
        tok = C.tokens(cfg, 330, 22)
        check_sizes(dec, tok, R.forward(cfg, w, tok), ([270, 5, 2, 20, 9] + [1] * 24,), dtype, cfg)
    finally:
        dec.close()
        model.close()


def test_portions_on_the_large_tiles(rt):
    """Sizes whose products of long portions take the large-tile GEMM and the 128-wide expert tiles, bf16
    against the restatement."""
    from yalm_amd import models as M

    full = C.moe(experts=4, top=4, ff=128, shared=256, limit=1.0, shared_limit=0.7)
    cfg = C.config([(C.latent(heads=4, dim=64, rot_dim=32, vdim=64, kv_rank=128, scale=0.1), full),
                    (C.gla(heads=3, dim=64, vdim=64), full), (C.attn(heads=4, kv_heads=2, dim=64, vdim=64, scale=0.125), full)],
                   width=320, vocab=307)
    model, dec, w = build(rt, cfg, M.BF16, seed=24, max_tokens=400)
    try:
        tok = C.tokens(cfg, 330, 24)
        got = dec.step(tok, list(range(330)))  # every expert is chosen by every token: no near-tie can flip
        assert rel_err(got, R.forward(cfg, w, tok)).max() < BF16_TOL
    finally:
        dec.close()
        model.close()


def test_stream_wider_than_the_register_seam(rt):
    """A width above 4096: the post-norm seam that keeps the row in LDS, the strided embedding and norms."""
    from yalm_amd import models as M

    cfg = C.config([(C.gla(heads=2, dim=8, vdim=8), C.moe(experts=3, top=3, ff=8, shared=8)),
                    (C.latent(heads=2, dim=8, rot_dim=4, vdim=8, kv_rank=12), None)], width=4104, vocab=41)
    model, dec, w = build(rt, cfg, M.F32, seed=23, max_tokens=64)
    try:
        tok = C.tokens(cfg, 40, 23)
        check_sizes(dec, tok, R.forward(cfg, w, tok), ([12, 3, 9] + [1] * 16,))
    finally:
        dec.close()
        model.close()


def test_bad_configurations_are_refused(rt):
    """What the kernels do not do is an error at creation, not a wrong result."""
    from yalm_amd import layered as Ly
    from yalm_amd import models as M

    cfg = C.MIXED
    t = make(cfg, 25)
    c = Ly.gugozen_config(cfg, max_tokens=64, weight_dtype=M.F32, shapes={k: v.shape for k, v in t.items()})
    p = Ly.gugozen_pack(c, t)

    def refused(i=None, whole=None, packed=p, **changed):
        layers = list(c.layers)
        if i is not None:
            layers[i] = dataclasses.replace(layers[i], **changed)
        model = rt.SeqModel.from_packed(c.with_(layers=layers, **(whole or {})), packed)
        try:
            with pytest.raises(rt.YalmError):
                rt.SeqDecoder(model)
        finally:
            model.close()

    refused(3, kv_from=5)                                # a later layer
    refused(3, kv_from=1)                                # not a latent layer
    refused(7, kv_from=3)                                # a layer without rows of its own
    refused(7, kv_from=0)                                # rows of another size
    refused(0, out_gate=Ly.GATE_HEAD)
    refused(0, rot_pairs=2)
    refused(1, decay_tau=0.0)
    refused(1, dim=300)
    refused(0, identity=1, router_kind=Ly.ROUTER_SOFTMAX_NORMED)  # weights on the inputs leave identity outputs no place
    refused(0, groups=2)
    refused(whole=dict(pre_norm=True))                   # post-norm blocks have no opening norms
    refused(whole=dict(norm_kind=4))
    refused(whole=dict(bigram_mul_prev=-1))
    refused(packed={k: v for k, v in p.items() if k != "bigram"})


def test_sequence_cannot_pass_max_tokens(rt):
    from yalm_amd import models as M

    model, dec, _ = build(rt, C.ONLY_GLA, M.F32, seed=13, max_tokens=16)
    try:
        dec.step(C.tokens(C.ONLY_GLA, 16, 0))
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
        {"step": 3, "entries": [{"id": "b", "tokens": b[:18], "want": [0, 17]}], "end": []},
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
    assert rel_err(np.fromfile(out / "3.f32", "<f4").reshape(-1, V), rb[[0, 17]]).max() < lim
    assert rel_err(np.fromfile(out / "4.f32", "<f4").reshape(-1, V), rb[[18]]).max() < lim
