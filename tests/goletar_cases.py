"""Small Goletar configurations for the tests: sizes, constants and orders of layers that differ in every way the design allows."""


def moe(experts=6, top=2, ff=40, limit=1.0):
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}


def latent(heads=4, dim=16, rot_dim=8, vdim=24, kv_rank=40, scale=0.3, base=10000.0, mlp="moe"):
    return {"type": "latent_attention", "mlp": moe() if mlp == "moe" else mlp,
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale, "rot": {"base": base, "dims": rot_dim}}}


def mingru(width=48, mlp="moe"):
    return {"type": "mingru", "mixer": {"width": width}, "mlp": moe() if mlp == "moe" else mlp}


def model(layers, width=64, vocab=97, eps=1e-5, buckets=211, mul_prev=31, mul_cur=7):
    return {"architecture": "Goletar", "embedding": {"bigram": {"buckets": buckets, "mul_cur": mul_cur, "mul_prev": mul_prev}}, "layers": layers,
            "norm": {"eps": eps}, "vocab": vocab, "width": width}


CASES = {
    # both mixers in either order, layers without a feed-forward behind either, one, two and all experts picked; a width of whole 64s
    # (in bfloat16 the experts run grouped), experts' units filled up to 64 and over
    "mixed": model([
        latent(),
        mingru(width=80, mlp=moe(experts=5, top=1, ff=64, limit=0.7)),
        mingru(width=24, mlp=None),
        latent(heads=3, dim=24, rot_dim=16, vdim=16, kv_rank=64, scale=0.2, base=500.0, mlp=moe(experts=3, top=3, ff=72, limit=2.5)),
        latent(heads=1, dim=8, rot_dim=4, vdim=32, kv_rank=24, mlp=None),
        mingru(width=64),
    ]),
    # sizes that are no multiples of anything a kernel would like (all experts as one product in either precision); one expert in all;
    # factors larger than the buckets, a bucket count of a few
    "odd": model([
        mingru(width=37, mlp=moe(experts=4, top=3, ff=10, limit=0.5)),
        latent(heads=5, dim=20, rot_dim=6, vdim=12, kv_rank=30, scale=0.25, base=777.0, mlp=moe(experts=1, top=1, ff=30, limit=3.0)),
        latent(heads=7, dim=12, rot_dim=10, vdim=20, kv_rank=21, scale=0.15, base=50.0, mlp=moe(experts=9, top=2, ff=18)),
        mingru(width=130, mlp=moe(experts=2, top=1, ff=50)),
    ], width=100, vocab=77, eps=1e-6, buckets=13, mul_prev=1009, mul_cur=100003),
    # wider: states of several blocks, more experts than the small router takes, rows of 192 and 288 cached elements, more layers of one
    # kind behind each other, many tiles an expert
    "wide": model([
        mingru(width=320, mlp=moe(experts=70, top=4, ff=64)),
        mingru(width=256, mlp=moe(experts=8, top=2, ff=128, limit=1.5)),
        latent(heads=6, dim=48, rot_dim=32, vdim=64, kv_rank=160, scale=0.11, base=20000.0, mlp=moe(experts=12, top=3, ff=96)),
        latent(heads=8, dim=64, rot_dim=32, vdim=40, kv_rank=256, scale=0.1, base=300.0, mlp=moe(experts=4, top=1, ff=192)),
    ], width=192, vocab=211, buckets=1021, mul_prev=257, mul_cur=65),
    # latents wider than the matrix-core kernel takes, one of them in whole sixteens and one not
    "large": model([
        latent(heads=3, dim=32, rot_dim=32, vdim=48, kv_rank=320, scale=0.12, base=5000.0, mlp=moe(experts=4, top=2, ff=128)),
        mingru(width=520, mlp=None),
        latent(heads=2, dim=40, rot_dim=38, vdim=72, kv_rank=300, scale=0.1, mlp=None),
    ], width=128, vocab=90),
    # one kind of mixer alone: no pages at all; and no state but the previous token
    "recurrent": model([mingru(width=96), mingru(width=40, mlp=None)], width=64, vocab=61, mul_prev=0, mul_cur=1),
    "attending": model([latent(), latent(heads=2, dim=32, rot_dim=2, vdim=48, kv_rank=96, scale=0.2)], width=80, vocab=130, mul_prev=1, mul_cur=0),
}
