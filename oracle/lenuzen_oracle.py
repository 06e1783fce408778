"""Plain restatement of the Lenuzen decoder, one function per mechanism, on CPU tensors of any float dtype.

Whole sequences only, one at a time: no cache, no batch, no folded factors.  Attention builds the full score matrix of every
head.  Weights are a dict of tensors under the checkpoint's names."""
from __future__ import annotations

import math

import torch


def unit(x, eps):
    """x over its root mean square along the last dim, eps under the root."""
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def centred_norm(x, w, eps):
    """Mean taken off, divided by the standard deviation (eps under the root), times a weight."""
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt(d.pow(2).mean(-1, keepdim=True) + eps) * w


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z.pow(3))))


def sliding_mask(n, size):
    """(n, n) bool: row i sees columns i - size + 1 .. i; size 0: 0 .. i."""
    away = torch.arange(n)[:, None] - torch.arange(n)[None, :]
    return (away >= 0) & (away < (size or n))


def chunk_mask(n, size):
    """(n, n) bool: row i sees the columns up to i that lie in its own chunk, chunks counted from 0; size 0: one chunk."""
    at = torch.arange(n)
    return (at[None, :] <= at[:, None]) & (at[:, None] // (size or n) == at[None, :] // (size or n))


def pair_frequencies(rot):
    """Angles per position of the rotated pairs and the amplitude, as Python floats; ``scaling`` is the YaRN blend."""
    dims, base = rot["dims"], float(rot["base"])
    freq = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    s = rot.get("scaling")
    if not s:
        return freq, 1.0

    def pair_that_turns(times):
        return dims * math.log(s["original"] / (2 * math.pi * times)) / (2 * math.log(base))

    lo, hi = max(math.floor(pair_that_turns(s["fast"])), 0), min(math.ceil(pair_that_turns(s["slow"])), dims - 1)
    slow = [min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0) for i in range(dims // 2)]
    return [f * (a / s["factor"] + 1 - a) for f, a in zip(freq, slow)], 0.1 * math.log(s["factor"]) + 1.0


def rotate(x, rot):
    """x (n, heads, d), row p at position p: pairs (2i, 2i + 1) of the first dims turned, the rest as they are."""
    freq, amplitude = pair_frequencies(rot)
    angle = torch.arange(x.shape[0], dtype=torch.float64)[:, None] * torch.tensor(freq, dtype=torch.float64)
    turn = torch.polar(torch.full_like(angle, amplitude), angle)[:, None, :]
    head = x[..., :2 * len(freq)].double().unflatten(-1, (len(freq), 2)).contiguous()
    turned = torch.view_as_real(torch.view_as_complex(head) * turn).flatten(-2)
    return torch.cat([turned.to(x.dtype), x[..., 2 * len(freq):]], -1)


def head_scores(q, k, scale):
    """(heads, n, n) of q (n, heads, d) and k (n, groups, d): neighbouring heads share a key head."""
    per = q.shape[1] // k.shape[1]
    return torch.stack([q[:, h] @ k[:, h // per].T * scale for h in range(q.shape[1])])


def mix_heads(scores, talk):
    """Row h of ``talk`` holds how much of every head's scores goes into head h's."""
    return torch.einsum("hg,gij->hij", talk, scores)


def weights_of(scores, see, sink=None):
    """Softmax over what is seen; ``sink``: one further term exp(sink) in the denominator."""
    s = scores.masked_fill(~see, float("-inf"))
    if sink is None:
        return torch.softmax(s, -1)
    extra = torch.full_like(s[..., :1], sink)
    return torch.softmax(torch.cat([s, extra], -1), -1)[..., :-1]


def values_out(weights, v):
    """(n, heads, vdim) of weights (heads, n, n) and v (n, groups, vdim)."""
    per = weights.shape[0] // v.shape[1]
    return torch.stack([weights[h] @ v[:, h // per] for h in range(weights.shape[0])], 1)


def split_heads(x, heads):
    return x.view(x.shape[0], heads, -1)


def attention(h, w, p, cfg, eps):
    """Biases in the projections, unit queries and keys behind the rotation, unit values, a factor per head on the scores, a
    sliding window, a gate per head."""
    q, k, v = (split_heads(h @ w[p + n].T + w[p + n + ".b"], heads)
               for n, heads in (("q", cfg["heads"]), ("k", cfg["kv_heads"]), ("v", cfg["kv_heads"])))
    q, k, v = unit(rotate(q, cfg["rot"]), eps), unit(rotate(k, cfg["rot"]), eps), unit(v, eps)
    scores = head_scores(q, k, cfg["scale"]) * w[p + "temp"][:, None, None]
    o = values_out(weights_of(scores, sliding_mask(h.shape[0], (cfg.get("mask") or {}).get("size", 0))), v)
    return (o * torch.sigmoid(h @ w[p + "g"].T)[..., None]).flatten(1) @ w[p + "o"].T


def talking_attention(h, w, p, cfg, eps):
    """Queries and keys normed over all heads at once, rotated; the heads' scores mixed; chunks; a sink at 0."""
    q, k = (unit(h @ w[p + n].T, eps) * w[p + n + ".norm"] for n in ("q", "k"))
    q, k, v = split_heads(q, cfg["heads"]), split_heads(k, cfg["kv_heads"]), split_heads(h @ w[p + "v"].T, cfg["kv_heads"])
    scores = mix_heads(head_scores(rotate(q, cfg["rot"]), rotate(k, cfg["rot"]), cfg["scale"]), w[p + "talk"])
    see = chunk_mask(h.shape[0], (cfg.get("mask") or {}).get("size", 0))
    return values_out(weights_of(scores, see, 0.0), v).flatten(1) @ w[p + "o"].T


def feed_forward(h, w, p):
    return gelu_tanh(h @ w[p + "up"].T) @ w[p + "down"].T


def layer(x, w, p, entry, eps):
    """Sublayers read the residual itself; what they return is normed on its way into it."""
    mixer = {"attention": attention, "attention_2": talking_attention}[entry["type"]]
    x = x + centred_norm(mixer(x, w, p + "mix.", entry["mixer"], eps), w[p + "norm1"], eps)
    if entry.get("mlp") is not None:
        x = x + centred_norm(feed_forward(x, w, p + "mlp."), w[p + "norm2"], eps)
    return x


def forward(tokens, weights, config, dtype=torch.float64, layer_outputs=None):
    """Logits (T, vocab) of one sequence; ``layer_outputs`` (a list) collects the residual after every layer."""
    w = {k: (t.to(dtype) if t.is_floating_point() else t) for k, t in weights.items()}
    eps = config["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens)] * config["embedding"]["scale"]
    for i, entry in enumerate(config["layers"]):
        x = layer(x, w, f"l{i}.", entry, eps)
        if layer_outputs is not None:
            layer_outputs.append(x)
    return centred_norm(x, w["final.norm"], eps) @ w["embed"].T * config["logit_scale"]


def random_weights(config, seed=0, dtype=torch.bfloat16):
    """Checkpoint tensors of a configuration, drawn so that every weight, bias and factor takes part."""
    g = torch.Generator().manual_seed(seed)
    width = config["width"]

    def normal(*shape, std=1.0, mean=0.0):
        return (torch.randn(shape, generator=g) * std + mean).to(dtype)

    def linear(rows, columns):
        return normal(rows, columns, std=columns ** -0.5)

    w = {"embed": normal(config["vocab"], width), "final.norm": normal(width, std=0.2, mean=1.0)}
    for i, entry in enumerate(config["layers"]):
        p, m, c = f"l{i}.", f"l{i}.mix.", entry["mixer"]
        heads, groups = c["heads"], c["kv_heads"]
        rows = {"q": heads * c["dim"], "k": groups * c["dim"], "v": groups * c["vdim"]}
        w[p + "norm1"] = normal(width, std=0.2, mean=1.0)
        w.update({m + n: linear(r, width) for n, r in rows.items()})
        w[m + "o"] = linear(width, heads * c["vdim"])
        if entry["type"] == "attention":
            w.update({f"{m}{n}.b": normal(r, std=0.5) for n, r in rows.items()})
            w[m + "temp"], w[m + "g"] = normal(heads, std=0.3, mean=1.0), normal(heads, width, std=2 * width ** -0.5)
        else:
            w.update({f"{m}{n}.norm": normal(rows[n], std=0.2, mean=1.0) for n in ("q", "k")})
            w[m + "talk"] = (torch.eye(heads) * 0.7 + torch.randn(heads, heads, generator=g) * heads ** -0.5).to(dtype)
        if entry.get("mlp") is not None:
            ff = entry["mlp"]["ff"]
            w.update({p + "norm2": normal(width, std=0.2, mean=1.0), p + "mlp.up": linear(ff, width), p + "mlp.down": linear(width, ff)})
    return w
