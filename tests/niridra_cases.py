"""Small Niridra configurations shared by the CPU and GPU tests."""
from __future__ import annotations


def moe(experts=10, top=3, ff=40, groups=(2, 1), shared=56):
    return {"kind": "moe", "expert": {"ff": ff}, "shared": None if shared is None else {"ff": shared},
            "router": {"experts": experts, "top": top, "groups": None if groups is None else {"count": groups[0], "keep": groups[1]}}}


def lightning_layer(heads=3, dim=24, vdim=40, decay=None, mlp=None):
    decay = [0.3 + 0.69 * i / max(heads - 1, 1) for i in range(heads)] if decay is None else decay
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}, "mlp": mlp}


def latent_layer(heads=5, dim=40, vdim=24, rank=72, scale=0.5, kv_from=None, mlp=None):
    mixer = {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": rank, "scale": scale}
    if kv_from is not None:
        mixer["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": mixer, "mlp": mlp}


def config(layers, width=80, vocab=150, streams=3, eps=1e-3, scale=7.0, bigram=(37, 5, 3), **extra):
    names = ("buckets", "mul_prev", "mul_cur")
    return {"architecture": "Niridra", "layers": layers, "width": width, "vocab": vocab, "streams": streams, "norm": {"eps": eps},
            "embedding": {"scale": scale, "bigram": dict(zip(names, bigram)) if bigram else None}, **extra}


def mixed_config(**kw):
    """Unequal sizes everywhere, latents shared with a later layer of other heads, a layer without a feed-forward."""
    return config([lightning_layer(mlp=moe()), latent_layer(mlp=moe(experts=12, top=5, groups=(3, 2), ff=72)),
                   latent_layer(heads=3, dim=24, vdim=56, scale=-0.7, kv_from=1, mlp=moe(shared=None)), lightning_layer(heads=2, dim=20, vdim=12),
                   latent_layer(heads=2, dim=16, vdim=8, rank=40, scale=0.9), latent_layer(heads=4, dim=48, vdim=48, scale=0.4, kv_from=1)], **kw)


def other_config(**kw):
    """Latents first, more heads than one tile of the matrix unit, wide memory heads, one stream, all experts in one group."""
    return config([latent_layer(heads=18, dim=16, vdim=48, rank=150, scale=0.6, mlp=moe(experts=5, top=1, groups=None, ff=100, shared=30)),
                   lightning_layer(heads=2, dim=72, vdim=136, decay=[0.999, 0.05], mlp=moe(experts=6, top=6, groups=(1, 1)))],
                  width=100, vocab=96, streams=1, eps=1e-5, scale=1.0, **{"bigram": (1009, 70001, 90007), **kw})


def plain_config(**kw):
    """Equal sizes everywhere, heads of 64, groups of one expert's width, four streams, no second embedding."""
    return config([lightning_layer(heads=2, dim=64, vdim=64, mlp=moe(experts=8, top=2, groups=(4, 2), ff=64, shared=64)),
                   latent_layer(heads=2, dim=64, vdim=64, rank=64, mlp=moe(experts=8, top=2, groups=(4, 1), ff=64, shared=64))],
                  width=64, vocab=64, streams=4, eps=1e-6, **{"bigram": None, **kw})


CONFIGS = {"mixed": mixed_config, "other": other_config, "plain": plain_config}
