"""Small Lenuzen configurations shared by the CPU and GPU tests."""
from __future__ import annotations

YARN = {"factor": 5.0, "fast": 6.0, "slow": 0.5, "original": 40}
STEEP = {"factor": 3.0, "fast": 9.0, "slow": 2.0, "original": 300}


def dense(ff=72):
    return {"kind": "dense", "ff": ff}


def _layer(kind, heads, kv_heads, dim, vdim, size, rot, base, scaling, scale, mlp):
    r = {"base": base, "dims": dim if rot is None else rot}
    if scaling:
        r["scaling"] = scaling
    return {"type": kind, "mlp": mlp, "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale,
                                                "mask": {"size": size}, "rot": r}}


def unit_layer(heads=6, kv_heads=2, dim=40, vdim=24, window=20, rot=28, base=700.0, scaling=YARN, scale=0.6, mlp=None):
    """Sliding window, unit heads."""
    return _layer("attention", heads, kv_heads, dim, vdim, window, rot, base, scaling, scale, mlp)


def talk_layer(heads=6, kv_heads=2, dim=24, vdim=40, chunk=33, rot=10, base=90.0, scaling=STEEP, scale=0.3, mlp=None):
    """Chunks, mixed heads."""
    return _layer("attention_2", heads, kv_heads, dim, vdim, chunk, rot, base, scaling, scale, mlp)


def config(layers, width=80, vocab=150, eps=1e-3, scale=0.8, logit_scale=0.7, **extra):
    return {"architecture": "Lenuzen", "layers": layers, "width": width, "vocab": vocab, "norm": {"eps": eps},
            "embedding": {"scale": scale}, "logit_scale": logit_scale, **extra}


def mixed_config(**kw):
    """Unequal sizes, windows and chunks everywhere, three heads per key head, a layer without a feed-forward, no scaling once."""
    return config([talk_layer(mlp=dense()), unit_layer(mlp=dense(100)), unit_layer(heads=4, kv_heads=4, dim=16, vdim=36, window=47, rot=12, scaling=None, scale=-0.5),
                   talk_layer(heads=5, kv_heads=5, dim=32, vdim=32, chunk=20, rot=32, scaling=None, mlp=dense(30)),
                   unit_layer(heads=3, kv_heads=1, dim=64, vdim=50, window=33, rot=2, mlp=dense())], **kw)


def other_config(**kw):
    """One key head, more heads than one tile of the matrix unit, a window of one token, chunks of one and of whole pages."""
    return config([unit_layer(heads=18, kv_heads=1, dim=72, vdim=72, window=64, scale=0.2, mlp=dense(40)),
                   talk_layer(heads=20, kv_heads=1, dim=50, vdim=30, chunk=48, scale=0.1, mlp=dense(24)),
                   talk_layer(heads=3, kv_heads=3, dim=20, vdim=20, chunk=1), unit_layer(heads=2, kv_heads=2, dim=24, vdim=24, window=1, rot=6)],
                  width=100, vocab=96, eps=1e-5, scale=3.0, logit_scale=2.5, **kw)


def plain_config(**kw):
    """Equal sizes everywhere, heads of 64, windows and chunks of 32, everything that can be one is one."""
    return config([unit_layer(heads=1, kv_heads=1, dim=64, vdim=64, window=32, rot=64, scaling=None, scale=1.0, mlp=dense(64)),
                   talk_layer(heads=1, kv_heads=1, dim=64, vdim=64, chunk=32, rot=64, scaling=None, scale=1.0, mlp=dense(64)),
                   talk_layer(heads=2, kv_heads=2, dim=64, vdim=64, chunk=32, rot=64, scaling=None, scale=0.125, mlp=dense(64))],
                  width=64, vocab=64, eps=1e-6, scale=1.0, logit_scale=1.0, **kw)


def large_config(**kw):
    """Heads wider than the tiled kernels of mixed heads, many key heads, everything visible."""
    return config([talk_layer(heads=4, kv_heads=2, dim=160, vdim=130, chunk=0, scale=0.05), unit_layer(heads=2, kv_heads=1, dim=150, vdim=200, window=0, scale=0.3),
                   talk_layer(heads=36, kv_heads=12, dim=16, vdim=8, chunk=80, rot=0, mlp=dense(16))], width=130, vocab=70, **kw)


CONFIGS = {"mixed": mixed_config, "other": other_config, "plain": plain_config, "large": large_config}
