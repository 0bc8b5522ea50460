"""Small Faguzen configurations for the tests (config.json dicts). Sizes are deliberately unequal to
one another (dim != vdim on both sides of a pair, kv_heads 1 / < heads / == heads, left and right
heads unequal), include values that are not multiples of the kernels' vector and tile widths, rotated
parts of no, two and all entries with and without rescaled frequencies, score caps the scores reach
and caps they do not, gate caps that bite, routers without identity outputs, with as many as experts,
top 1 and top = all outputs, loops of one and three passes at the start, the middle and the end."""


def rot(dims=8, base=500.0, factor=4.0, low=1.0, high=3.0, original=40, scaled=True):
    r = {"dims": dims, "base": base}
    if scaled:
        r["scaling"] = {"factor": factor, "low": low, "high": high, "original": original}
    return r


def attn(heads=4, kv_heads=2, dim=24, vdim=40, scale=0.21, softcap=6.0, r=None):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "softcap": softcap,
            "rot": r or rot()}


def memory(heads=3, dim=16, vdim=24, gate_cap=5.0):
    return {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": gate_cap}


def pair(left=None, right=None, left_scale=0.9, right_scale=0.7):
    return {"left": left or attn(), "right": right or memory(), "left_scale": left_scale, "right_scale": right_scale}


def moe(experts=6, identity=2, top=2, ff=40, shared=24):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "identity": identity, "top": top}}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def config(layers, width=96, vocab=211, eps=1e-5, mult=0.8, cap=9.0, loop=None):
    """layers: [(mixer, feed-forward or None)]; loop: (start, stop, times) or None."""
    c = {"architecture": "Faguzen", "norm": {"eps": eps}, "vocab": vocab, "width": width, "residual_mult": mult,
         "logit_softcap": cap, "layers": [{"type": "parallel", "mixer": m, "mlp": f} for m, f in layers]}
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


TINY = pair(attn(heads=1, kv_heads=1, dim=4, vdim=8, r=rot(dims=2)), memory(heads=1, dim=4, vdim=8))

# one mechanism at a time
ONLY_PAIR = config([(pair(), None)])
ONLY_MOE = config([(TINY, moe())])
# everything, different sizes per layer, a middle run walked three times
MIXED = config([
    (pair(attn(scale=0.7, softcap=2.0)), moe()),
    (pair(attn(heads=6, kv_heads=6, dim=16, vdim=8, scale=0.3, softcap=1.5, r=rot(dims=16, scaled=False)),
          memory(heads=5, dim=8, vdim=40, gate_cap=1.5), 1.3, 0.4), moe(experts=4, identity=0, top=1, ff=24, shared=0)),
    (pair(attn(heads=3, kv_heads=1, dim=32, vdim=24, scale=0.17, softcap=60.0, r=rot(dims=0, scaled=False)),
          memory(heads=2, dim=40, vdim=16, gate_cap=30.0), 0.5, 1.2), None),
    (pair(attn(heads=2, kv_heads=2, dim=20, vdim=16, scale=0.25, r=rot(dims=2, base=7.0)),
          memory(heads=1, dim=24, vdim=24)), moe(experts=3, identity=3, top=6, ff=16, shared=40)),
], loop=(1, 3, 3))
# sizes that defeat every vector path: odd width, odd head sizes and feed-forward sizes; one pass of a loop from the start
ODD = config([
    (pair(attn(heads=5, kv_heads=5, dim=10, vdim=3, scale=0.35, softcap=4.0, r=rot(dims=6, original=9)),
          memory(heads=3, dim=5, vdim=11, gate_cap=2.5)), moe(experts=3, identity=1, top=2, ff=7, shared=5)),
    (pair(attn(heads=2, kv_heads=1, dim=9, vdim=7, scale=0.5, softcap=3.0, r=rot(dims=4)),
          memory(heads=2, dim=7, vdim=5)), None),
    (pair(attn(heads=3, kv_heads=3, dim=7, vdim=5, scale=0.4, r=rot(dims=2)), memory(heads=1, dim=3, vdim=1)),
     moe(experts=5, identity=2, top=3, ff=9, shared=0)),
], width=51, vocab=37, eps=1e-4, mult=1.1, cap=5.0, loop=(0, 1, 1))
# wider sizes: several tiles per product, long key rows and states, many heads; a loop at the end
WIDE = config([
    (pair(attn(heads=8, kv_heads=2, dim=96, vdim=80, scale=0.1, softcap=20.0, r=rot(dims=64, base=10000.0, original=200)),
          memory(heads=4, dim=128, vdim=64, gate_cap=10.0)), moe(experts=8, identity=4, top=3, ff=64, shared=96)),
    (pair(attn(heads=12, kv_heads=4, dim=32, vdim=48, scale=0.15, r=rot(dims=32)),
          memory(heads=8, dim=64, vdim=32, gate_cap=4.0)), moe(experts=16, identity=2, top=4, ff=48, shared=0)),
], width=256, vocab=1000, cap=15.0, loop=(1, 2, 2))
# no router whose near-ties a rounding could flip (bf16 comparisons)
NO_ROUTER = config([
    (pair(attn(heads=4, kv_heads=2, dim=32, vdim=48, scale=0.15, softcap=8.0, r=rot(dims=16)),
          memory(heads=4, dim=32, vdim=16)), None),
    (pair(attn(heads=2, kv_heads=1, dim=48, vdim=64, scale=0.12, softcap=15.0, r=rot(dims=48, original=100)),
          memory(heads=2, dim=64, vdim=48, gate_cap=8.0), 0.6, 1.1), None),
], width=128, vocab=300, loop=(0, 2, 2))

ALL = {"only_pair": ONLY_PAIR, "only_moe": ONLY_MOE, "mixed": MIXED, "odd": ODD, "wide": WIDE, "no_router": NO_ROUTER}


def tokens(cfg, n, seed=0):
    import numpy as np

    return np.random.default_rng(4000 + seed).integers(0, cfg["vocab"], n).tolist()
