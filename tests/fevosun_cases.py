"""Small Fevosun configurations shared by the CPU and GPU tests."""
from __future__ import annotations

YARN = {"factor": 5.0, "fast": 6.0, "slow": 0.5, "original": 40}


def moe(experts=9, top=4, ff=40, identity=3, shared=56, limit=0.7, shared_limit=1.9):
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "identity": identity, "top": top},
            "shared": None if shared is None else {"ff": shared, "limit": shared_limit}}


def dense(ff=72):
    return {"kind": "dense", "ff": ff}


def attention_layer(heads=6, kv_heads=2, dim=40, window=20, scale=0.6, q_temp=(0.4, 7), mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale, "mask": {"size": window}}
    if q_temp is not None:
        m["q_temp"] = {"coef": q_temp[0], "every": q_temp[1]}
    return {"type": "attention", "mixer": m, "mlp": mlp}


def latent_layer(heads=5, dim=24, rot_dim=20, vdim=40, rank=72, q_rank=None, window=33, scale=0.5, base=700.0, scaling=YARN, mlp=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": rank, "scale": scale, "mask": {"size": window},
         "rot": {"base": base, "dims": rot_dim}}
    if scaling:
        m["rot"]["scaling"] = scaling
    if q_rank is not None:
        m["q_rank"] = q_rank
    return {"type": "latent_attention" if q_rank is None else "latent_attention_2", "mixer": m, "mlp": mlp}


def config(layers, width=80, vocab=150, eps=1e-3, scale=0.8, **extra):
    return {"architecture": "Fevosun", "layers": layers, "width": width, "vocab": vocab, "norm": {"eps": eps},
            "embedding": {"scale": scale}, **extra}


def mixed_config(**kw):
    """Every mixer and feed-forward, unequal sizes and windows everywhere, one window shared by two kinds of layer."""
    return config([latent_layer(q_rank=50, scaling=None, mlp=dense()), attention_layer(mlp=moe()),
                   latent_layer(heads=3, dim=40, rot_dim=12, vdim=16, rank=40, window=20, mlp=moe(experts=12, top=5, identity=1, shared=None)),
                   attention_layer(heads=4, kv_heads=4, dim=16, window=47, scale=-0.5, q_temp=None),
                   latent_layer(heads=2, dim=8, rot_dim=6, vdim=8, rank=24, q_rank=100, window=5, scaling=None, mlp=moe(identity=0, top=2))], **kw)


def other_config(**kw):
    """One kv head, more heads than one tile of the matrix unit, a window of one token, one that is a multiple of the page."""
    return config([attention_layer(heads=18, kv_heads=1, dim=72, window=64, scale=0.2, q_temp=(0.9, 1), mlp=dense(40)),
                   latent_layer(heads=17, dim=16, rot_dim=32, vdim=48, rank=150, window=48, mlp=moe(experts=5, top=1, identity=2, ff=100)),
                   attention_layer(heads=3, kv_heads=3, dim=24, window=1, mlp=None)], width=100, vocab=96, eps=1e-5, scale=1.0, **kw)


def plain_config(**kw):
    """Equal sizes everywhere, heads of 64, one window, every expert chosen."""
    return config([attention_layer(heads=2, kv_heads=2, dim=64, window=32, scale=0.125, mlp=moe(experts=3, top=4, identity=1, ff=64, shared=64, limit=1.0, shared_limit=1.0)),
                   latent_layer(heads=2, dim=64, rot_dim=64, vdim=64, rank=64, q_rank=64, window=32, scale=0.1, mlp=dense(64)),
                   latent_layer(heads=2, dim=64, rot_dim=64, vdim=64, rank=64, window=32, scale=0.1, mlp=dense(64))],
                  width=64, vocab=64, eps=1e-6, **kw)


CONFIGS = {"mixed": mixed_config, "other": other_config, "plain": plain_config}
