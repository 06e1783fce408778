"""Plain restatement of the Sokevik decoder, one function per mechanism, on CPU tensors of any float dtype.

Whole sequences only, one at a time: no cache, no batch, no chunked forms.  The mLSTM is the token-by-token recurrence and
attention builds the full score matrix.  Weights are a dict of tensors under the checkpoint's names."""
from __future__ import annotations

import math

import torch


def rms(x, eps):
    """x over its root mean square along the last dim, eps under the root."""
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def causal_conv(h, w):
    """Per-channel causal convolution over time: h (T, C), w (C, taps); tap ``taps - 1`` is the current step."""
    taps = w.shape[1]
    out = torch.zeros_like(h)
    for j in range(taps):
        back = taps - 1 - j
        if back < h.shape[0]:
            out[back:] += w[:, j] * h[:h.shape[0] - back]
    return out


def pair_frequencies(dims, base, scaling=None, dtype=torch.float64):
    """base^(-2i/dims); with ``scaling`` long wavelengths are stretched by ``factor``, short ones kept, a linear blend
    (in original/wavelength) in between."""
    f = base ** (-2.0 * torch.arange(dims // 2, dtype=torch.float64) / dims)
    if scaling is not None:
        out = []
        for x in f.tolist():
            wavelength = 2 * math.pi / x
            low, high, orig = scaling["low"], scaling["high"], scaling["original"]
            if wavelength < orig / high:
                out.append(x)
            elif wavelength > orig / low:
                out.append(x / scaling["factor"])
            else:
                s = (orig / wavelength - low) / (high - low)
                out.append((1 - s) * x / scaling["factor"] + s * x)
        f = torch.tensor(out, dtype=torch.float64)
    return f.to(dtype)


def rotate_pairs(x, positions, freqs, sign=1.0):
    """Turn dims (2i, 2i+1) of x (T, heads, D) by sign * position * freqs[i]; dims past 2 * len(freqs) pass."""
    n = freqs.numel()
    ang = sign * positions.double()[:, None] * freqs.double()[None, :]
    c, s = ang.cos().to(x.dtype)[:, None, :], ang.sin().to(x.dtype)[:, None, :]
    u, v = x[..., 0:2 * n:2], x[..., 1:2 * n:2]
    out = x.clone()
    out[..., 0:2 * n:2] = u * c - v * s
    out[..., 1:2 * n:2] = v * c + u * s
    return out


def chunk_mask(n, size):
    """(n, n) bool: row i sees column j."""
    i = torch.arange(n)
    see = i[None, :] <= i[:, None]
    if size:
        see &= (i[:, None] // size) == (i[None, :] // size)
    return see


def sink_softmax(scores, see, sink):
    """Softmax over the visible keys with one further term exp(sink) in the denominator; scores (H, T, S), sink (H,)."""
    s = scores.masked_fill(~see, float("-inf"))
    m = torch.maximum(s.max(-1, keepdim=True).values, sink[:, None, None])
    e = torch.exp(s - m)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink[:, None, None] - m))


def attention(h, w, p, cfg, eps):
    heads, groups, dim, vdim = cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"]
    n = h.shape[0]
    pos = torch.arange(n)
    q = (h @ w[p + "q"].T).view(n, heads, dim)
    k = (h @ w[p + "k"].T).view(n, groups, dim)
    v = (h @ w[p + "v"].T).view(n, groups, vdim)
    q = rms(q, eps) * w[p + "q.norm"]
    k = rms(k, eps) * w[p + "k.norm"]
    f = pair_frequencies(cfg["rot"]["dims"], cfg["rot"]["base"], cfg["rot"].get("scaling"))
    fv = pair_frequencies(vdim, cfg["rot"]["base"])
    q, k, v = rotate_pairs(q, pos, f), rotate_pairs(k, pos, f), rotate_pairs(v, pos, fv)
    rep = heads // groups
    k, v = k.repeat_interleave(rep, 1), v.repeat_interleave(rep, 1)
    scores = torch.einsum("ihd,jhd->hij", q, k) * cfg["scale"]
    wts = sink_softmax(scores, chunk_mask(n, cfg["mask"]["size"]), w[p + "sink"])
    o = torch.einsum("hij,jhd->ihd", wts, v)
    o = rotate_pairs(o, pos, fv, -1.0)
    o = o * torch.sigmoid(h @ w[p + "g"].T)[:, :, None]
    return o.reshape(n, -1) @ w[p + "o"].T


def mlstm_recurrence(q, k, v, log_i, log_f):
    """q, k (T, H, D), v (T, H, V), gates (T, H): the stabilised matrix-memory recurrence, token by token."""
    n, heads, dim = q.shape
    s = torch.zeros(heads, dim, v.shape[-1], dtype=q.dtype)
    z = torch.zeros(heads, dim, dtype=q.dtype)
    m = torch.zeros(heads, dtype=q.dtype)
    outs = []
    for t in range(n):
        m_new = torch.maximum(log_f[t] + m, log_i[t])
        keep, add = torch.exp(log_f[t] + m - m_new), torch.exp(log_i[t] - m_new)
        s = keep[:, None, None] * s + add[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        z = keep[:, None] * z + add[:, None] * k[t]
        m = m_new
        num = torch.einsum("hdv,hd->hv", s, q[t])
        den = torch.maximum((z * q[t]).sum(-1).abs(), torch.exp(-m)) + 1e-6
        outs.append(num / den[:, None])
    return torch.stack(outs)


def mlstm_gates(h, w, p, cap):
    """Capped log input gate and log forget gate."""
    i = cap * torch.tanh((h @ w[p + "i"].T + w[p + "i.b"]) / cap)
    f = torch.nn.functional.logsigmoid(cap * torch.tanh((h @ w[p + "f"].T + w[p + "f.b"]) / cap))
    return i, f


def mlstm(h, w, p, cfg, eps):
    heads, dim, vdim = cfg["heads"], cfg["dim"], cfg["vdim"]
    n = h.shape[0]
    q = (h @ w[p + "q"].T).view(n, heads, dim) * dim ** -0.5
    k = (h @ w[p + "k"].T).view(n, heads, dim)
    v = (h @ w[p + "v"].T).view(n, heads, vdim)
    o = rms(mlstm_recurrence(q, k, v, *mlstm_gates(h, w, p, cfg["gate_cap"])), eps).reshape(n, -1)
    return (o * w[p + "norm"] * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def feed_forward(h, w, p):
    gate = h @ w[p + "gate"].T
    return (gate * torch.sigmoid(gate) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def sublayer(x, w, p, number, fn, eps):
    """x + norm_b(fn(conv-mixed norm(x))), norms with one gain for all coordinates."""
    h = rms(x, eps) * w[f"{p}norm{number}"]
    h = h + causal_conv(h, w[f"{p}canon{number}"])
    return x + rms(fn(h), eps) * w[f"{p}norm{number}b"]


MIXERS = {"attention": attention, "mlstm": mlstm}


def forward(tokens, weights, config, dtype=torch.float64, layer_outputs=None):
    """Logits (T, vocab) of one sequence; ``layer_outputs`` (a list) collects the residual stream after every layer."""
    w = {k: (t.to(dtype) if t.is_floating_point() else t) for k, t in weights.items()}
    eps = config["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens)]
    for i, entry in enumerate(config["layers"]):
        p = f"l{entry.get('weights_of', i)}."
        mixer = MIXERS[entry["type"]]
        x = sublayer(x, w, p, 1, lambda h: mixer(h, w, p + "mix.", entry["mixer"], eps), eps)
        if entry.get("mlp") is not None:
            x = sublayer(x, w, p, 2, lambda h: feed_forward(h, w, p + "mlp."), eps)
        if layer_outputs is not None:
            layer_outputs.append(x.clone())
    return (rms(x, eps) * w["final.norm"]) @ w["head"].T


def random_weights(config, seed=0, dtype=torch.bfloat16):
    """Checkpoint tensors of a configuration, drawn so that gates, sinks and norms all take part."""
    g = torch.Generator().manual_seed(seed)
    width, taps = config["width"], config["canon"]["taps"]

    def normal(*shape, std=1.0, mean=0.0):
        return (torch.randn(shape, generator=g) * std + mean).to(dtype)

    w = {"embed": normal(config["vocab"], width), "head": normal(config["vocab"], width, std=width ** -0.5),
         "final.norm": normal(std=0.1, mean=1.0)}
    for i, entry in enumerate(config["layers"]):
        if "weights_of" in entry:
            continue
        p, c = f"l{i}.", entry["mixer"]
        names = ["1"] + (["2"] if entry.get("mlp") is not None else [])
        for s in names:
            w[p + f"norm{s}"] = normal(std=0.1, mean=1.0)
            w[p + f"norm{s}b"] = normal(std=0.1, mean=0.5)
            w[p + f"canon{s}"] = normal(width, taps, std=0.3)
        m = p + "mix."
        heads = c["heads"]
        kv = c.get("kv_heads", heads)
        w[m + "q"] = normal(heads * c["dim"], width, std=width ** -0.5)
        w[m + "k"] = normal(kv * c["dim"], width, std=width ** -0.5)
        w[m + "v"] = normal(kv * c["vdim"], width, std=width ** -0.5)
        w[m + "o"] = normal(width, heads * c["vdim"], std=(heads * c["vdim"]) ** -0.5)
        if entry["type"] == "attention":
            w[m + "q.norm"] = normal(c["dim"], std=0.2, mean=1.2)
            w[m + "k.norm"] = normal(c["dim"], std=0.2, mean=1.2)
            w[m + "sink"] = normal(heads, std=1.0, mean=1.0)
            w[m + "g"] = normal(heads, width, std=width ** -0.5)
        else:
            w[m + "g"] = normal(heads * c["vdim"], width, std=width ** -0.5)
            w[m + "norm"] = normal(heads * c["vdim"], std=0.2, mean=1.0)
            w[m + "i"] = normal(heads, width, std=2 * width ** -0.5)
            w[m + "i.b"] = normal(heads, std=1.0)
            w[m + "f"] = normal(heads, width, std=width ** -0.5)
            w[m + "f.b"] = normal(heads, std=1.0, mean=3.0)
        if entry.get("mlp") is not None:
            ff = entry["mlp"]["ff"]
            w[p + "mlp.gate"] = normal(ff, width, std=width ** -0.5)
            w[p + "mlp.up"] = normal(ff, width, std=width ** -0.5)
            w[p + "mlp.down"] = normal(width, ff, std=ff ** -0.5)
    return w
