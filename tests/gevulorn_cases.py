"""Small Gevulorn configurations for the tests: sizes, constants and orders of layers that differ in every way the design allows."""


def dense(ff=80):
    return {"kind": "dense", "ff": ff}


def moe(experts=6, top=2, ff=40, shared=56):
    out = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared:
        out["shared"] = {"ff": shared}
    return out


def gla(heads=2, dim=16, vdim=24, tau=8.0, mlp=None):
    return {"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}, "mlp": mlp}


def window(heads=4, kv_heads=2, dim=16, vdim=16, scale=0.6, base=1000.0, dims=None, size=24, keep_first=5, mlp=None):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "rot": {"base": base, "dims": dim if dims is None else dims}}
    if size:
        mixer["mask"] = {"size": size, "keep_first": keep_first}
    return {"type": "attention", "mixer": mixer, "mlp": mlp}


def chunked(heads=4, kv_heads=2, dim=16, vdim=16, scale=0.6, base=700.0, dims=None, scaling=(4.0, 1.0, 4.0, 64), softcap=9.0, size=40, mlp=None):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "rot": {"base": base, "dims": dim if dims is None else dims}}
    if scaling:
        mixer["rot"]["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    if softcap:
        mixer["softcap"] = softcap
    if size:
        mixer["mask"] = {"size": size}
    return {"type": "attention_2", "mixer": mixer, "mlp": mlp}


def model(layers, width=64, vocab=97, eps=1e-5, scale=3.0, softcap=12.0, loop=None):
    out = {"architecture": "Gevulorn", "embedding": {"scale": scale}, "layers": layers, "norm": {"eps": eps}, "vocab": vocab, "width": width}
    if softcap:
        out["logit_softcap"] = softcap
    if loop:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    return out


CASES = {
    # all three mixers, each kind of feed-forward and none, a loop in the middle over two kinds of layer; a width of whole 64s (in bfloat16 the
    # experts run in the streaming product); a shared expert larger and smaller than the others, and none
    "mixed": model([
        window(mlp=dense()),
        gla(mlp=moe(shared=150)),
        chunked(heads=6, kv_heads=2, dim=32, vdim=24, softcap=4.0, size=33, mlp=moe(experts=5, top=1, ff=64, shared=20)),
        gla(heads=3, dim=24, vdim=40, tau=1.0, mlp=None),
        window(heads=3, kv_heads=3, dim=24, vdim=32, size=7, keep_first=70, dims=8, mlp=moe(experts=4, top=4, ff=30, shared=None)),
    ], loop=(1, 3, 2)),
    # sizes that are no multiples of anything a kernel would like; a window of one, no kept keys, values wider and narrower than keys, no cap on
    # scores or logits, no stretched frequencies, a loop over the last layers
    "odd": model([
        gla(heads=3, dim=7, vdim=13, tau=3.0, mlp=moe(experts=7, top=3, ff=10, shared=33)),
        window(heads=5, kv_heads=1, dim=10, vdim=22, dims=6, size=1, keep_first=3, mlp=dense(50)),
        chunked(heads=2, kv_heads=1, dim=18, vdim=6, dims=10, scaling=None, softcap=None, size=5, mlp=moe(experts=1, top=1, ff=18, shared=70)),
        window(heads=2, kv_heads=2, dim=12, vdim=12, dims=4, size=65, keep_first=0, mlp=None),
    ], width=100, vocab=77, eps=1e-6, scale=1.0, softcap=None, loop=(2, 4, 3)),
    # wider: heads of 64 and 128 (the streaming prompt kernel, the split-key decode kernel), windows of pages, more experts than the small
    # router takes, a decay memory of several tiles; a loop over all layers
    "wide": model([
        window(heads=4, kv_heads=1, dim=64, vdim=64, scale=0.5, size=100, keep_first=64, mlp=moe(experts=70, top=4, ff=64, shared=128)),
        gla(heads=2, dim=96, vdim=128, tau=16.0, mlp=dense(256)),
        chunked(heads=2, kv_heads=2, dim=128, vdim=96, scale=0.3, size=150, softcap=30.0, mlp=dense(192)),
        gla(heads=4, dim=48, vdim=64, tau=2.0, mlp=moe(experts=8, top=2, ff=100, shared=100)),
    ], width=192, vocab=211, loop=(0, 4, 2)),
    # heads wider than the matrix-core prompt kernel takes, decay memories of 200 x 40 and 40 x 200, no masks at all, no loop
    "large": model([
        gla(heads=1, dim=200, vdim=40, tau=0.5, mlp=dense(64)),
        window(heads=2, kv_heads=1, dim=160, vdim=64, scale=0.2, size=None, mlp=None),
        gla(heads=2, dim=40, vdim=200, tau=30.0, mlp=moe(experts=3, top=2, ff=128, shared=64)),
        chunked(heads=2, kv_heads=1, dim=48, vdim=80, size=None, mlp=dense(100)),
    ], width=128, vocab=90, scale=7.5, softcap=3.0),
    # one kind of mixer alone: no pages at all, decays from all but none to all at once; and no state at all
    "recurrent": model([gla(heads=4, dim=8, vdim=8, tau=1.0, mlp=dense(64)), gla(heads=1, dim=33, vdim=17, tau=0.2)], width=64, vocab=61, loop=(1, 2, 4)),
    "attending": model([window(size=16, keep_first=16), chunked(size=16, mlp=moe()), window(size=200, keep_first=1, dim=32, vdim=32, mlp=dense())],
                       width=80, vocab=130, loop=(0, 1, 2)),
}
