"""Small Gugozen configurations for the tests (config.json dicts). Sizes are deliberately unequal to
one another (dim != vdim, plain and rotated parts unequal, latent ranks of no special size, kv_heads 1
/ < heads / == heads), include values that are not multiples of the kernels' vector and tile widths,
latent layers that read another layer's rows with other heads and sizes of their own, next to it and
several layers on, decay roots below, at and above one, routers of top 1 and top = all, clamps that
bite and clamps that do not, with and without shared experts, feed-forwards and pair embeddings."""


def rot(dims=8, base=500.0):
    return {"dims": dims, "base": base}


def latent(heads=3, dim=24, rot_dim=8, vdim=20, kv_rank=36, scale=0.19, base=300.0, kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale,
         "rot": rot(rot_dim, base)}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return "latent_attention", m


def attn(heads=4, kv_heads=2, dim=24, vdim=40, scale=0.21, r=None):
    return "attention", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "rot": r or rot()}


def gla(heads=3, dim=20, vdim=28, tau=6.0):
    return "gla", {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}


def moe(experts=6, top=2, ff=40, limit=1.5, shared=24, shared_limit=0.8):
    m = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}
    if shared:
        m["shared"] = {"ff": shared, "limit": shared_limit}
    return m


def config(layers, width=96, vocab=211, eps=1e-5, alpha=1.7, bigram=(73, 29, 11)):
    """layers: [((type, mixer), feed-forward or None)]; bigram: (buckets, mul_prev, mul_cur) or None."""
    c = {"architecture": "Gugozen", "norm": {"eps": eps}, "vocab": vocab, "width": width, "postln_alpha": alpha,
         "layers": [{"type": t, "mixer": m, "mlp": f} for (t, m), f in layers]}
    if bigram:
        c["embedding"] = {"bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))}
    return c


TINY = attn(heads=1, kv_heads=1, dim=4, vdim=8, r=rot(2))

# one mechanism at a time
ONLY_LATENT = config([(latent(), None)])
ONLY_SHARED = config([(latent(), None), (latent(heads=5, dim=12, vdim=12, scale=0.3, kv_from=0), None)])
ONLY_ATTN = config([(attn(), None)])
ONLY_GLA = config([(gla(), None)])
ONLY_MOE = config([(TINY, moe())])
# everything, different sizes per layer
MIXED = config([
    (latent(), moe()),
    (gla(), moe(experts=4, top=1, ff=24, shared=0)),
    (attn(heads=6, kv_heads=6, dim=16, vdim=8, scale=0.3, r=rot(16, 40.0)), None),
    (latent(heads=5, dim=16, vdim=12, scale=0.25, kv_from=0), moe(experts=3, top=3, ff=16, limit=0.3, shared=40)),
    (gla(heads=2, dim=40, vdim=16, tau=0.5), None),
    (latent(heads=2, dim=8, rot_dim=12, vdim=36, kv_rank=20, base=7.0), moe(experts=5, top=2, shared_limit=30.0)),
    (attn(heads=3, kv_heads=1, dim=32, vdim=24, scale=0.17), moe(experts=7, top=4, ff=8, limit=9.0)),
    (latent(heads=1, dim=20, rot_dim=12, vdim=8, kv_rank=20, base=7.0, kv_from=5), None),
])
# sizes that defeat every vector path
ODD = config([
    (attn(heads=5, kv_heads=5, dim=10, vdim=3, scale=0.35, r=rot(6, 9.0)), moe(experts=3, top=2, ff=7, shared=5)),
    (latent(heads=3, dim=5, rot_dim=6, vdim=11, kv_rank=13, scale=0.4), None),
    (gla(heads=3, dim=7, vdim=5, tau=1.0), moe(experts=5, top=3, ff=9, shared=0)),
    (latent(heads=2, dim=9, rot_dim=6, vdim=7, kv_rank=13, scale=0.3, kv_from=1), None),
    (gla(heads=1, dim=3, vdim=1, tau=2.5), None),
], width=51, vocab=37, eps=1e-4, alpha=0.6, bigram=(13, 7, 5))
# wider sizes: several tiles per product, long key rows and states, many heads
WIDE = config([
    (latent(heads=8, dim=64, rot_dim=32, vdim=80, kv_rank=112, scale=0.1, base=10000.0), moe(experts=8, top=3, ff=64, shared=96)),
    (gla(heads=4, dim=128, vdim=64, tau=12.0), moe(experts=16, top=4, ff=48, shared=0)),
    (attn(heads=8, kv_heads=2, dim=96, vdim=80, scale=0.1, r=rot(64, 10000.0)), moe(experts=4, top=1, ff=72, shared=64)),
    (latent(heads=6, dim=32, rot_dim=32, vdim=48, kv_rank=112, scale=0.13, base=10000.0, kv_from=0), None),
], width=224, vocab=1000, alpha=3.1, bigram=(509, 1234577, 31))
# no router whose near-ties a rounding could flip (bf16 comparisons)
NO_ROUTER = config([
    (latent(heads=4, dim=32, rot_dim=16, vdim=24, kv_rank=64, scale=0.15), None),
    (gla(heads=4, dim=32, vdim=48), None),
    (attn(heads=4, kv_heads=2, dim=32, vdim=48, scale=0.15, r=rot(16)), moe(experts=3, top=3, ff=32, shared=24)),
    (latent(heads=2, dim=48, rot_dim=16, vdim=64, kv_rank=64, scale=0.12, kv_from=0), None),
], width=128, vocab=300)

ALL = {"only_latent": ONLY_LATENT, "only_shared": ONLY_SHARED, "only_attn": ONLY_ATTN, "only_gla": ONLY_GLA,
       "only_moe": ONLY_MOE, "mixed": MIXED, "odd": ODD, "wide": WIDE, "no_router": NO_ROUTER}


def tokens(cfg, n, seed=0):
    import numpy as np

    return np.random.default_rng(5000 + seed).integers(0, cfg["vocab"], n).tolist()
