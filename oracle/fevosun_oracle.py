"""Plain restatement of the Fevosun decoder, one function per mechanism, on CPU tensors of any float dtype.

Whole sequences only, one at a time: no cache, no batch, no absorbed latents.  Attention builds the full score matrix, and the
experts run token by token.  Weights are a dict of tensors under the checkpoint's names."""
from __future__ import annotations

import math

import torch


def rms(x, eps):
    """x over its root mean square along the last dim, eps under the root."""
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def shifted_norm(x, w, eps):
    """The norm's gain is one more than its stored weight."""
    return rms(x, eps) * (1 + w)


def silu(z):
    return z / (1 + torch.exp(-z))


def window_mask(n, size):
    """(n, n) bool: row i sees the columns i - size + 1 .. i; size 0: all of 0 .. i."""
    d = torch.arange(n)[:, None] - torch.arange(n)[None, :]
    return (d >= 0) & ((d < size) if size else torch.ones_like(d, dtype=torch.bool))


def query_temperature(positions, coef, every):
    """1 + coef ln(floor((p + 1) / every) + 1), float64."""
    return torch.tensor([1 + coef * math.log(math.floor((p + 1) / every) + 1) for p in positions], dtype=torch.float64)


def distance_slopes(heads):
    return torch.tensor([2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)], dtype=torch.float64)


def rotation(rot, n):
    """cos and sin (n, dims / 2) of positions 0 .. n - 1, float64; with ``scaling`` the YaRN frequencies and amplitude."""
    dims, base = rot["dims"], float(rot["base"])
    freq, amplitude = [base ** (-2.0 * i / dims) for i in range(dims // 2)], 1.0
    if rot.get("scaling"):
        s = rot["scaling"]

        def turn(t):
            return dims * math.log(s["original"] / (2 * math.pi * t)) / (2 * math.log(base))

        lo, hi = max(math.floor(turn(s["fast"])), 0), min(math.ceil(turn(s["slow"])), dims - 1)
        ramp = [min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0) for i in range(dims // 2)]
        freq = [f / s["factor"] * r + f * (1 - r) for f, r in zip(freq, ramp)]
        amplitude = 0.1 * math.log(s["factor"]) + 1.0
    angle = torch.arange(n, dtype=torch.float64)[:, None] * torch.tensor(freq, dtype=torch.float64)[None, :]
    return angle.cos() * amplitude, angle.sin() * amplitude


def rotate(x, cos, sin, interleaved):
    """x (n, ..., d) turned by its row's angles: pairs (2i, 2i + 1), or (i, i + dims / 2); dims past the pairs stay."""
    half = cos.shape[1]
    shape = (cos.shape[0],) + (1,) * (x.dim() - 2) + (half,)
    c, s = cos.to(x.dtype).view(shape), sin.to(x.dtype).view(shape)
    y = x.clone()
    a, b = (slice(0, 2 * half, 2), slice(1, 2 * half, 2)) if interleaved else (slice(0, half), slice(half, 2 * half))
    u, v = x[..., a], x[..., b]
    y[..., a], y[..., b] = u * c - v * s, v * c + u * s
    return y


def attend(scores, see, values):
    """softmax of scores (n, n) over what is seen, times values (n, d)."""
    return torch.softmax(scores.masked_fill(~see, float("-inf")), -1) @ values


def attention(h, w, p, cfg):
    """Grouped heads whose keys are their values, a distance bias, a query temperature, a window and an output gate."""
    n, heads, groups, d = h.shape[0], cfg["heads"], cfg["kv_heads"], cfg["dim"]
    q = (h @ w[p + "q"].T).view(n, heads, d)
    if cfg.get("q_temp"):
        q = q * query_temperature(range(n), cfg["q_temp"]["coef"], cfg["q_temp"]["every"]).to(h.dtype)[:, None, None]
    k = (h @ w[p + "k"].T).view(n, groups, d)
    slope = distance_slopes(heads).to(h.dtype)
    away = (torch.arange(n)[:, None] - torch.arange(n)[None, :]).to(h.dtype)
    see = window_mask(n, (cfg.get("mask") or {}).get("size", 0))
    out = torch.empty(n, heads, d, dtype=h.dtype)
    for i in range(heads):
        kv = k[:, i // (heads // groups)]
        out[:, i] = attend(q[:, i] @ kv.T * cfg["scale"] - slope[i] * away, see, kv)
    return (out.reshape(n, -1) * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def latent_attention(h, w, p, cfg, eps, interleaved):
    """Heads over keys and values made of one normed latent per token, beside a rotated part of the keys that the heads
    have in common; queries come from h, or (``dq`` present) from a normed latent of their own."""
    n, heads, d, r, rank = h.shape[0], cfg["heads"], cfg["dim"], cfg["rot_dim"], cfg["kv_rank"]
    if p + "dq" in w:
        q = (rms(h @ w[p + "dq"].T, eps) * w[p + "dq.norm"]) @ w[p + "uq"].T
    else:
        q = h @ w[p + "q"].T
    q = q.view(n, heads, d + r)
    down = h @ w[p + "dkv"].T
    c = rms(down[:, :rank], eps) * w[p + "dkv.norm"]
    cos, sin = rotation(cfg["rot"], n)
    k_rot, q_rot = rotate(down[:, rank:], cos, sin, interleaved), rotate(q[..., d:], cos, sin, interleaved)
    k = (c @ w[p + "uk"].T).view(n, heads, d)
    v = (c @ w[p + "uv"].T).view(n, heads, cfg["vdim"])
    see = window_mask(n, (cfg.get("mask") or {}).get("size", 0))
    out = torch.empty(n, heads, cfg["vdim"], dtype=h.dtype)
    for i in range(heads):
        out[:, i] = attend((q[:, i, :d] @ k[:, i].T + q_rot[:, i] @ k_rot.T) * cfg["scale"], see, v[:, i])
    return out.reshape(n, -1) @ w[p + "o"].T


def dense(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def clamped_expert(h, w, p, limit):
    g = (h @ w[p + "gate"].T).clamp(max=limit)
    u = (h @ w[p + "up"].T).clamp(-limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1)) @ w[p + "down"].T


def route(z, correction, top):
    """Choices and their weights of one token: z (experts + identity experts,) router logits."""
    s = torch.softmax(z, -1)
    choice = (s + correction).tolist()
    ids = sorted(range(len(choice)), key=lambda e: -choice[e])[:top]
    return ids, s[ids]


def experts(h, w, p, cfg):
    """Mixture of experts of which the last ones hand their input on, and a shared one; token by token."""
    z = h @ w[p + "router"].T
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, g in zip(*route(z[t], w[p + "correction"], cfg["router"]["top"])):
            out[t] += g * (h[t] if e >= cfg["router"]["experts"] else clamped_expert(h[t], w, f"{p}e{e}.", cfg["expert"]["limit"]))
    if cfg.get("shared"):
        out = out + clamped_expert(h, w, p + "shared.", cfg["shared"]["limit"])
    return out


def layer(x, w, p, entry, eps):
    """One norm, both sublayers on its output, their sum into the residual."""
    h = shifted_norm(x, w[p + "norm1"], eps)
    m, f, kind = entry["mixer"], entry.get("mlp"), entry["type"]
    y = attention(h, w, p + "mix.", m) if kind == "attention" else latent_attention(h, w, p + "mix.", m, eps, kind == "latent_attention_2")
    if f is not None:
        y = y + (dense(h, w, p + "mlp.") if f["kind"] == "dense" else experts(h, w, p + "mlp.", f))
    return x + y


def forward(tokens, weights, config, dtype=torch.float64, layer_outputs=None):
    """Logits (T, vocab) of one sequence; ``layer_outputs`` (a list) collects the residual after every layer."""
    w = {k: (t.to(dtype) if t.is_floating_point() else t) for k, t in weights.items()}
    eps = config["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens)] * config["embedding"]["scale"]
    for i, entry in enumerate(config["layers"]):
        x = layer(x, w, f"l{i}.", entry, eps)
        if layer_outputs is not None:
            layer_outputs.append(x)
    return shifted_norm(x, w["final.norm"], eps) @ w["head"].T


def random_weights(config, seed=0, dtype=torch.bfloat16):
    """Checkpoint tensors of a configuration, drawn so that every gain and correction takes part."""
    g = torch.Generator().manual_seed(seed)
    width = config["width"]

    def normal(*shape, std=1.0, mean=0.0):
        return (torch.randn(shape, generator=g) * std + mean).to(dtype)

    def linear(rows, columns):
        return normal(rows, columns, std=columns ** -0.5)

    w = {"embed": normal(config["vocab"], width), "head": linear(config["vocab"], width), "final.norm": normal(width, std=0.2)}
    for i, entry in enumerate(config["layers"]):
        p, c, e = f"l{i}.", entry["mixer"], entry.get("mlp")
        w[p + "norm1"] = normal(width, std=0.2)
        m, heads = p + "mix.", c["heads"]
        if entry["type"] == "attention":
            w[m + "q"], w[m + "k"] = linear(heads * c["dim"], width), linear(c["kv_heads"] * c["dim"], width)
            w[m + "g"], w[m + "o"] = linear(heads * c["dim"], width), linear(width, heads * c["dim"])
        else:
            r, rows = c["kv_rank"], heads * (c["dim"] + c["rot_dim"])
            if entry["type"] == "latent_attention_2":
                w[m + "dq"], w[m + "dq.norm"] = linear(c["q_rank"], width), normal(c["q_rank"], std=0.2, mean=1.0)
                w[m + "uq"] = linear(rows, c["q_rank"])
            else:
                w[m + "q"] = linear(rows, width)
            w[m + "dkv"], w[m + "dkv.norm"] = linear(r + c["rot_dim"], width), normal(r, std=0.2, mean=1.0)
            w[m + "uk"], w[m + "uv"] = linear(heads * c["dim"], r), linear(heads * c["vdim"], r)
            w[m + "o"] = linear(width, heads * c["vdim"])
        if e is None:
            continue
        forms = [(f"{p}mlp.", e["ff"])] if e["kind"] == "dense" else [(f"{p}mlp.e{j}.", e["expert"]["ff"]) for j in range(e["router"]["experts"])]
        if e["kind"] == "moe":
            if e.get("shared"):
                forms.append((p + "mlp.shared.", e["shared"]["ff"]))
            n = e["router"]["experts"] + e["router"].get("identity", 0)
            w[p + "mlp.router"] = normal(n, width, std=2 * width ** -0.5)
            w[p + "mlp.correction"] = normal(n, std=0.1)
        for name, ff in forms:
            w[name + "gate"], w[name + "up"], w[name + "down"] = linear(ff, width), linear(ff, width), linear(width, ff)
    return w
