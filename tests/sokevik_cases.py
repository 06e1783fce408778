"""Small Sokevik configurations, steps and drivers shared by the CPU and GPU tests."""
from __future__ import annotations

import torch

from minivllm_amd.engine.hybrid_cache import HybridCacheManager
from minivllm_amd.engine.sequence import Sequence


def attention_layer(heads=6, kv_heads=2, dim=40, vdim=24, chunk=20, rot=16, base=1000.0, scale=0.3, scaling=True, ff=72):
    return {"type": "attention",
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "mask": {"size": chunk},
                      "rot": {"base": base, "dims": rot,
                              "scaling": {"factor": 3.0, "low": 1.0, "high": 3.5, "original": 48} if scaling else None}},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def mlstm_layer(heads=3, dim=24, vdim=40, cap=6.0, ff=None):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def shared(layer, j):
    return {**layer, "weights_of": j}


def config(layers, width=80, vocab=150, taps=3, eps=1e-3, **extra):
    return {"architecture": "Sokevik", "layers": layers, "width": width, "vocab": vocab, "canon": {"taps": taps},
            "norm": {"eps": eps}, **extra}


def mixed_config(**kw):
    """Two chunk sizes, unequal key and value sizes, shared weights of both kinds, a feed-forward behind either mixer."""
    a, b = attention_layer(), mlstm_layer(ff=56)
    c = attention_layer(heads=4, kv_heads=4, dim=16, vdim=36, chunk=33, rot=12, base=5e4, scale=-0.4, scaling=False, ff=None)
    return config([a, b, c, shared(a, 0), mlstm_layer(heads=2, dim=20, vdim=12), shared(b, 1), c], **kw)


def other_config(**kw):
    """Key size above the value size, one kv head, wide memory heads, a chunk above a page, short convolution."""
    return config([mlstm_layer(heads=2, dim=72, vdim=136, cap=11.0),
                   attention_layer(heads=5, kv_heads=1, dim=96, vdim=64, chunk=48, rot=96, scale=0.1, ff=40)],
                  width=100, vocab=96, taps=2, eps=1e-5, **kw)


def plain_config(**kw):
    """Equal sizes everywhere, one key / value head per query head, a chunk that is a multiple of the page, many taps."""
    return config([attention_layer(heads=2, kv_heads=2, dim=64, vdim=64, chunk=64, rot=64, scale=0.125, ff=64),
                   mlstm_layer(heads=2, dim=64, vdim=64, cap=15.0, ff=64)], width=64, vocab=64, taps=6, eps=1e-6, **kw)


CONFIGS = {"mixed": mixed_config, "other": other_config, "plain": plain_config}


def tokens(seed, n, vocab):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


class Driver:
    """Runs portions of requests through a runner as the engine's scheduler would, and collects logits."""

    def __init__(self, runner):
        self.runner, self.cache, self.live = runner, runner.cache_manager, {}
        self.logits = {}

    def step(self, portions: dict, end=()):
        """portions: request name -> its next tokens."""
        seqs = []
        for name, new in portions.items():
            seq = self.live.get(name)
            if seq is None:
                seq = self.live[name] = Sequence(list(new), block_size=self.runner.block_size)
                assert self.cache.can_allocate(seq)
                self.cache.allocate(seq)
            else:
                for t in new:
                    seq.append_token(t)
                assert self.cache.can_append(seq)
                self.cache.append(seq)
            seq.num_scheduled_tokens = len(new)
            seqs.append(seq)
        out = self.runner.step_logits(seqs, [range(len(n)) for n in portions.values()])
        at = 0
        for (name, new), seq in zip(portions.items(), seqs):
            self.logits.setdefault(name, []).append(out[at:at + len(new)].cpu())
            at += len(new)
            seq.num_computed_tokens += len(new)
        for name in end:
            self.cache.deallocate(self.live.pop(name))
        return out

    def run_alone(self, name, toks, sizes):
        """One request in portions of the given sizes (the last one repeats), then given back."""
        at, i = 0, 0
        while at < len(toks):
            n = min(sizes[min(i, len(sizes) - 1)], len(toks) - at)
            self.step({name: toks[at:at + n]}, end=[name] if at + n == len(toks) else [])
            at, i = at + n, i + 1
        return torch.cat(self.logits.pop(name))


def manager(windows=(20, 0), num_blocks=64, block_size=16, slots=4):
    return HybridCacheManager(list(windows), num_blocks, block_size, slots)
