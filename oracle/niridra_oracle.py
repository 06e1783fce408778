"""Plain restatement of the Niridra decoder, one function per mechanism, on CPU tensors of any float dtype.

Whole sequences only, one at a time: no cache, no batch, no absorbed or chunked forms.  The decaying memory is the
token-by-token recurrence, attention builds the full score matrix from keys and values made of the latents, and the experts
run token by token.  Weights are a dict of tensors under the checkpoint's names."""
from __future__ import annotations

import torch


def rms(x, eps):
    """x over its root mean square along the last dim, eps under the root."""
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def silu(z):
    return z / (1 + torch.exp(-z))


def bigram_rows(tokens, buckets, mul_prev, mul_cur):
    """Row of the bigram table per token; a first token has the row behind the hashed ones."""
    rows, prev = [], None
    for t in tokens:
        rows.append(buckets if prev is None else (prev * mul_prev + t * mul_cur) % buckets)
        prev = t
    return rows


def embedding(tokens, w, cfg):
    x = w["embed"][torch.as_tensor(tokens)] * cfg["scale"]
    if cfg.get("bigram"):
        b = cfg["bigram"]
        x = x + w["bigram"][torch.as_tensor(bigram_rows(tokens, b["buckets"], b["mul_prev"], b["mul_cur"]))]
    return x


def decaying_memory(q, k, v, decay):
    """q, k (T, H, D), v (T, H, V), decay (H,): S <- decay S + k v^T, o = S^T q, token by token from zero."""
    s = torch.zeros(q.shape[1], q.shape[2], v.shape[2], dtype=q.dtype)
    outs = []
    for t in range(q.shape[0]):
        s = decay[:, None, None] * s + k[t][:, :, None] * v[t][:, None, :]
        outs.append((s * q[t][:, :, None]).sum(1))
    return torch.stack(outs)


def lightning(h, w, p, cfg, eps):
    n, heads = h.shape[0], cfg["heads"]
    q = silu(h @ w[p + "q"].T).view(n, heads, cfg["dim"])
    k = silu(h @ w[p + "k"].T).view(n, heads, cfg["dim"])
    v = silu(h @ w[p + "v"].T).view(n, heads, cfg["vdim"])
    o = decaying_memory(q, k, v, torch.tensor(cfg["decay"], dtype=torch.float64).to(h.dtype)).reshape(n, -1)
    return (rms(o, eps) * w[p + "norm"] * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def latent(h, w, p, eps):
    return rms(h @ w[p + "dkv"].T, eps) * w[p + "dkv.norm"]


def latent_attention(h, c, w, p, cfg):
    """Causal softmax attention of h's queries over keys and values made of the latents c (T, kv_rank)."""
    n, heads = h.shape[0], cfg["heads"]
    q = (h @ w[p + "q"].T).view(n, heads, cfg["dim"])
    k = (c @ w[p + "uk"].T).view(n, heads, cfg["dim"])
    v = (c @ w[p + "uv"].T).view(n, heads, cfg["vdim"])
    out = torch.empty(n, heads, cfg["vdim"], dtype=h.dtype)
    see = torch.arange(n)[None, :] <= torch.arange(n)[:, None]
    for i in range(heads):
        s = (q[:, i] @ k[:, i].T * cfg["scale"]).masked_fill(~see, float("-inf"))
        out[:, i] = torch.softmax(s, -1) @ v[:, i]
    return out.reshape(n, -1) @ w[p + "o"].T


def route(z, correction, cfg):
    """Experts and their weights of one token: z (E,) router logits."""
    s = torch.sigmoid(z)
    choice = s + correction
    groups = cfg.get("groups") or {"count": 1, "keep": 1}
    size = z.numel() // groups["count"]
    score = [sum(sorted(choice[g * size:(g + 1) * size].tolist(), reverse=True)[:2]) for g in range(groups["count"])]
    best = sorted(range(groups["count"]), key=lambda g: -score[g])[:groups["keep"]]
    open_ = [e for g in best for e in range(g * size, (g + 1) * size)]
    ids = sorted(open_, key=lambda e: -choice[e].item())[:cfg["top"]]
    return ids, s[ids] / (s[ids].sum() + 1e-20)


def expert(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def experts(h, w, p, cfg):
    """Mixture of experts with a shared one, token by token."""
    z = h @ w[p + "router"].T
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        ids, weights = route(z[t], w[p + "correction"], cfg["router"])
        for e, g in zip(ids, weights):
            out[t] += g * expert(h[t], w, f"{p}e{e}.")
    if cfg.get("shared"):
        out = out + torch.sigmoid(h @ w[p + "shared.sg"].T) * expert(h, w, p + "shared.")
    return out


def hyper_sublayer(xs, w, p, number, fn, eps):
    """One sublayer between the streams xs (S, T, W): a weighted sum goes in, every new stream is a mix of the old ones plus
    its share of the scaled result."""
    hc = f"{p}hc{number}."
    u = torch.einsum("s,stw->tw", w[hc + "in"], xs)
    y = fn(rms(u, eps) * w[f"{p}norm{number}"]) * w[f"{p}ls{number}"]
    return torch.einsum("st,snw->tnw", w[hc + "mix"], xs) + w[hc + "out"][:, None, None] * y


def forward(tokens, weights, config, dtype=torch.float64, layer_outputs=None):
    """Logits (T, vocab) of one sequence; ``layer_outputs`` (a list) collects the sum of the streams after every layer."""
    w = {k: (t.to(dtype) if t.is_floating_point() else t) for k, t in weights.items()}
    eps = config["norm"]["eps"]
    xs = embedding(tokens, w, config["embedding"]).expand(config["streams"], -1, -1).clone()
    latents = {}
    for i, entry in enumerate(config["layers"]):
        p, m = f"l{i}.", entry["mixer"]

        def mixer(h):
            if entry["type"] == "lightning":
                return lightning(h, w, p + "mix.", m, eps)
            if m.get("kv_from") is None:
                latents[i] = latent(h, w, p + "mix.", eps)
            return latent_attention(h, latents[i if m.get("kv_from") is None else m["kv_from"]], w, p + "mix.", m)

        xs = hyper_sublayer(xs, w, p, 1, mixer, eps)
        if entry.get("mlp") is not None:
            xs = hyper_sublayer(xs, w, p, 2, lambda h: experts(h, w, p + "mlp.", entry["mlp"]), eps)
        if layer_outputs is not None:
            layer_outputs.append(xs.sum(0))
    return (rms(xs.sum(0), eps) * w["final.norm"]) @ w["embed"].T


def random_weights(config, seed=0, dtype=torch.bfloat16):
    """Checkpoint tensors of a configuration, drawn so that every gain, stream weight and correction takes part."""
    g = torch.Generator().manual_seed(seed)
    width, streams = config["width"], config["streams"]

    def normal(*shape, std=1.0, mean=0.0):
        return (torch.randn(shape, generator=g) * std + mean).to(dtype)

    def linear(rows, columns):
        return normal(rows, columns, std=columns ** -0.5)

    w = {"embed": linear(config["vocab"], width), "final.norm": normal(width, std=0.2, mean=1.0)}
    if config["embedding"].get("bigram"):
        w["bigram"] = normal(config["embedding"]["bigram"]["buckets"] + 1, width, std=0.7)
    for i, entry in enumerate(config["layers"]):
        p, c, e = f"l{i}.", entry["mixer"], entry.get("mlp")
        for s in ("1", "2") if e is not None else ("1",):
            w[f"{p}norm{s}"] = normal(width, std=0.2, mean=1.0)
            w[f"{p}ls{s}"] = normal(width, std=0.2, mean=0.7)
            w[f"{p}hc{s}.in"] = normal(streams, std=0.3, mean=1.0 / streams)
            w[f"{p}hc{s}.out"] = normal(streams, std=0.3, mean=1.0)
            w[f"{p}hc{s}.mix"] = (torch.eye(streams) + torch.randn(streams, streams, generator=g) * 0.2).to(dtype)
        m, heads = p + "mix.", c["heads"]
        w[m + "q"] = linear(heads * c["dim"], width)
        w[m + "o"] = linear(width, heads * c["vdim"])
        if entry["type"] == "lightning":
            w[m + "k"], w[m + "v"], w[m + "g"] = linear(heads * c["dim"], width), linear(heads * c["vdim"], width), linear(heads * c["vdim"], width)
            w[m + "norm"] = normal(heads * c["vdim"], std=0.2, mean=1.0)
        else:
            w[m + "uk"], w[m + "uv"] = linear(heads * c["dim"], c["kv_rank"]), linear(heads * c["vdim"], c["kv_rank"])
            if c.get("kv_from") is None:
                w[m + "dkv"], w[m + "dkv.norm"] = linear(c["kv_rank"], width), normal(c["kv_rank"], std=0.2, mean=1.0)
        if e is not None:
            forms = [(f"{p}mlp.e{j}.", e["expert"]["ff"]) for j in range(e["router"]["experts"])]
            if e.get("shared"):
                forms.append((p + "mlp.shared.", e["shared"]["ff"]))
                w[p + "mlp.shared.sg"] = linear(1, width)
            for name, ff in forms:
                w[name + "gate"], w[name + "up"], w[name + "down"] = linear(ff, width), linear(ff, width), linear(width, ff)
            w[p + "mlp.router"] = normal(e["router"]["experts"], width, std=2 * width ** -0.5)
            w[p + "mlp.correction"] = normal(e["router"]["experts"], std=0.5, mean=-0.3)     # choice scores of both signs
    return w
