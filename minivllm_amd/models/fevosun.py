"""Fevosun: a decoder of parallel layers: one norm, a windowed mixer and a feed-forward on its output, their sum into the residual.

Mixers are attention whose values are its keys (distance bias, query temperature, a gate per channel) and two kinds of latent
attention with a rotated part; feed-forwards are dense or mixtures of clamped experts, some of which hand their input on, with a
shared one.  Since both sublayers read the same rows and end in the same sum, a layer has one projection in front (everything
that reads the norm's output but the router and the experts) and one behind (mixer, dense feed-forward and shared expert side by
side), and one launch adds what the experts leave and makes the next layer's norm.  The residual is fp32.

The model runs ragged steps only: ``forward`` reads the step from the ``Context``.  Constants and sizes come from the
checkpoint's config.json; tensors keep its names."""
from __future__ import annotations

import os

import torch
import torch.nn as nn

from minivllm_amd.engine.windows import SlidingWindow
from minivllm_amd.layers.basic import Linear, rotary_pair_table
from minivllm_amd.layers.experts import SparseExperts
from minivllm_amd.layers.fused import gated_unit, stream_embed_norm, stream_norm
from minivllm_amd.layers.mixers import RotaryLatentAttention, SharedKeyAttention, distance_slopes
from minivllm_amd.utils.context import get_context
from minivllm_amd.utils.padding import pad_to, round_up
from minivllm_amd.utils.safetensors_io import read_safetensors

ALPHA, SHIFT = 1.702, 1.0              # of the clamped experts: g sigmoid(ALPHA g) (u + SHIFT)
LATENT = ("latent_attention", "latent_attention_2")


def engine_config(config: dict) -> dict:
    """config.json keys as they are, plus the engine's names for what the runner needs."""
    return {**config, "vocab_size": config["vocab"], "hidden_size": config["width"], "num_layers": len(config["layers"])}


def kernel_sources(config: dict) -> list[str]:
    """The csrc files a model of this configuration runs on."""
    layers = config["layers"]
    sources = ["capi.hip", "activation.hip", "linear_small.hip", "stream_norm.hip", "head_rope.hip", "ring_rows.hip", "window_prefill.hip",
               "window_decode.hip"]
    if any(e["type"] in LATENT for e in layers):
        sources += ["latent.hip", "window_prefill_latent.hip"]
    if any((e.get("mlp") or {}).get("kind") == "moe" for e in layers):
        sources += ["moe.hip", "gate_linear.hip"]
    return sources


def _window(mixer: dict) -> SlidingWindow:
    return SlidingWindow(int((mixer.get("mask") or {}).get("size") or 0))


def _mixer(kind: str, m: dict, windows: list, block_size: int, dtype, eps: float, small_rows: int):
    view = _window(m)
    where = (windows.index(view), view, block_size, dtype)
    if kind == "attention":
        if m.get("vdim", m["dim"]) != m["dim"]:
            raise ValueError(f"values are keys: they cannot have {m['vdim']} and {m['dim']} channels")
        t = m.get("q_temp")
        return SharedKeyAttention(m["heads"], m["kv_heads"], m["dim"], m["scale"], *where, (t["coef"], t["every"]) if t else (0.0, 0),
                                  distance_slopes(m["heads"]))
    if kind in LATENT:
        second = kind == LATENT[1]
        return RotaryLatentAttention(m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], m["scale"], *where, eps,
                                     interleaved=second, q_rank=m["q_rank"] if second else 0, small_rows=small_rows)
    raise ValueError(f"unknown mixer type {kind!r}")


class FevosunLayer(nn.Module):
    is_attention = True

    def __init__(self, entry: dict, width: int, inputs: int, windows: list, block_size: int, dtype, eps: float, small_rows: int):
        super().__init__()
        self.mixer = _mixer(entry["type"], entry["mixer"], windows, block_size, dtype, eps, small_rows)
        self.width, self.inputs, self.experts, self.unit, self.dense_names, ff = width, inputs, None, {}, None, 0
        if entry.get("mlp") is not None:
            c = entry["mlp"]
            if c.get("kind") == "dense":
                self.dense_names, ff = "mlp.", c["ff"]
            elif c.get("kind") == "moe":
                r, shared, clamped = c["router"], c.get("shared"), lambda form: (ALPHA, form["limit"], SHIFT)
                self.experts = SparseExperts(width, inputs, r["experts"], r["top"], c["expert"]["ff"], softmax=True,
                                             identity=r.get("identity", 0), glu=clamped(c["expert"]))
                if shared:
                    self.dense_names, ff, self.unit = "mlp.shared.", shared["ff"], dict(zip(("alpha", "limit", "shift"), clamped(shared)))
            else:
                raise ValueError(f"unknown feed-forward kind {c.get('kind')!r}")
        self.ff = round_up(ff, 16)                      # channels of what runs for every row: dense feed-forward or shared expert
        front, behind = self.mixer.sizes
        with torch.device("meta"):
            self.front = Linear(inputs, front + 2 * self.ff, bias=False, small_rows=small_rows)
            self.behind = Linear(behind + self.ff, width, bias=False, small_rows=small_rows)

    @torch.no_grad()
    def load(self, tensors: dict, prefix: str, dtype, device):
        def matrix(t):
            return t.to(device=device, dtype=dtype).contiguous()

        get = lambda name: tensors[prefix + name]
        self.gain = 1.0 + get("norm1").to(device=device, dtype=torch.float32)           # the checkpoint holds gain - 1
        rows, columns = self.mixer.load(lambda name: get("mix." + name), matrix, self.inputs)
        rows, columns = [rows], [columns]
        if self.dense_names:
            rows += [pad_to(matrix(get(self.dense_names + n)), self.ff, self.inputs) for n in ("gate", "up")]
            columns.append(pad_to(matrix(get(self.dense_names + "down")), None, self.ff))
        self.front.weight = nn.Parameter(torch.cat(rows), requires_grad=False)
        self.behind.weight = nn.Parameter(torch.cat(columns, 1).contiguous(), requires_grad=False)
        if self.experts is not None:
            self.experts.load(lambda name: get("mlp." + name), matrix)

    def forward(self, h, step):
        front, behind = self.mixer.sizes
        proj = self.front(h)
        z = torch.empty((h.shape[0], behind + self.ff), dtype=h.dtype, device=h.device)
        self.mixer(h, proj[:, :front], z[:, :behind], step)
        if self.ff:
            gated_unit(proj[:, front:], z[:, behind:], **self.unit)
        y = self.behind(z)
        if self.experts is None:
            return y
        out = self.experts(h)
        out.shared = y                                  # what every row has, beside the experts' rows
        return out


class FevosunForCausalLM(nn.Module):
    latent_views = False                                # its windows are sliding ones (engine/windows.py)
    memory_units = 0                                    # no recurrence

    def __init__(self, config: dict, block_size: int, dtype: torch.dtype, device: torch.device):
        super().__init__()
        self.config, self.dtype, self.device, self.block_size = config, dtype, device, block_size
        self.eps, self.width = config["norm"]["eps"], config["width"]
        self.inputs = round_up(self.width, SparseExperts.ALIGN)          # columns of a layer's input, zeros past the width
        layers = config["layers"]
        self.windows = sorted({_window(e["mixer"]) for e in layers})
        self.layer_stack = nn.ModuleList(FevosunLayer(e, self.width, self.inputs, self.windows, block_size, dtype, self.eps,
                                                      config.get("linear_small_rows", 64)) for e in layers)
        max_position, tables = config.get("max_position", 4096), {}
        for layer, entry in zip(self.layer_stack, layers):
            if entry["type"] not in LATENT:
                continue
            rot = entry["mixer"]["rot"]
            if rot["dims"] > entry["mixer"]["rot_dim"]:
                raise ValueError(f"{rot['dims']} rotated dimensions of {entry['mixer']['rot_dim']}")
            key = (rot["base"], rot["dims"], tuple(sorted((rot.get("scaling") or {}).items())))
            if key not in tables:
                tables[key] = rotary_pair_table(rot["base"], rot["dims"], max_position, rot.get("scaling") or None).to(device)
            layer.mixer.table = tables[key]
        self.one = torch.ones(1, dtype=torch.float32, device=device)     # one residual stream

    # ---- weights ----
    def load_weights(self, tensors: dict) -> None:
        dev = dict(device=self.device, dtype=self.dtype)
        self.embedding, self.lm_head_weight = (tensors[n].to(**dev).contiguous() for n in ("embed", "head"))
        self.final_gain = 1.0 + tensors["final.norm"].to(device=self.device, dtype=torch.float32)
        for i, layer in enumerate(self.layer_stack):
            layer.load(tensors, f"l{i}.", self.dtype, self.device)

    def load_checkpoint(self, model_dir: str) -> None:
        self.load_weights(read_safetensors(os.path.join(model_dir, "model.safetensors")))

    def reset_parameters(self, seed: int = 0) -> None:
        """Random tensors of the configuration's shapes, scaled so that activations keep their size."""
        g = torch.Generator(device=self.device).manual_seed(seed)
        c, width = self.config, self.width

        def normal(*shape, std=1.0, mean=0.0):
            return (torch.randn(shape, generator=g, device=self.device) * std + mean).to(torch.bfloat16)

        def linear(rows, columns):
            return normal(rows, columns, std=columns ** -0.5)

        t = {"embed": normal(c["vocab"], width), "head": linear(c["vocab"], width), "final.norm": normal(width, std=0.0)}
        for i, entry in enumerate(c["layers"]):
            m, p, f = entry["mixer"], f"l{i}.mix.", entry.get("mlp")
            heads = m["heads"]
            t[f"l{i}.norm1"] = normal(width, std=0.0)
            if entry["type"] == "attention":
                q, kv = heads * m["dim"], m["kv_heads"] * m["dim"]
                t.update({p + "q": linear(q, width), p + "k": linear(kv, width), p + "g": linear(q, width), p + "o": linear(width, q)})
            else:
                q, rank = heads * (m["dim"] + m["rot_dim"]), m["kv_rank"]
                t.update({p + "dkv": linear(rank + m["rot_dim"], width), p + "dkv.norm": normal(rank, std=0.0, mean=1.0),
                          p + "uk": linear(heads * m["dim"], rank), p + "uv": linear(heads * m["vdim"], rank),
                          p + "o": linear(width, heads * m["vdim"])})
                if entry["type"] == LATENT[1]:
                    t.update({p + "dq": linear(m["q_rank"], width), p + "dq.norm": normal(m["q_rank"], std=0.0, mean=1.0),
                              p + "uq": linear(q, m["q_rank"])})
                else:
                    t[p + "q"] = linear(q, width)
            if f is None:
                continue
            n, forms = f"l{i}.mlp.", []
            if f["kind"] == "dense":
                forms.append((n, f["ff"]))
            else:
                r = f["router"]
                outputs = r["experts"] + r.get("identity", 0)
                forms += [(f"{n}e{j}.", f["expert"]["ff"]) for j in range(r["experts"])]
                forms += [(n + "shared.", f["shared"]["ff"])] if f.get("shared") else []
                t.update({n + "router": linear(outputs, width), n + "correction": normal(outputs, std=0.01)})
            for name, ff in forms:
                t.update({name + "gate": linear(ff, width), name + "up": linear(ff, width), name + "down": linear(width, ff)})
        self.load_weights(t)

    # ---- caches ----
    def allocate_state(self, num_blocks: int, num_slots: int) -> None:
        """A pool of ``num_blocks`` blocks per layer; nothing is kept per slot."""
        for layer in self.layer_stack:
            layer.mixer.allocate(num_blocks, self.device)

    def forward(self, input_ids, positions, layer_outputs: list | None = None):
        """Final hidden states (T, width) of the context's ragged step; ``layer_outputs`` collects the residual after every layer
        (tests)."""
        step, layers, one = get_context().ragged, self.layer_stack, self.one
        h, x = stream_embed_norm(step, input_ids, self.embedding, self.config["embedding"]["scale"], 1, layers[0].gain, self.eps,
                                 padded=self.inputs)
        for i, layer in enumerate(layers):
            y, last = layer(h, step), i + 1 == len(layers)
            h, x = stream_norm(x, y, one, one.view(1, 1), self.final_gain if last else layers[i + 1].gain, self.eps,
                               padded=0 if last else self.inputs, want_x=not last or layer_outputs is not None)
            if layer_outputs is not None:
                layer_outputs.append(x[:, 0].clone())
        return h

    def compute_logits(self, hidden):
        return torch.nn.functional.linear(hidden, self.lm_head_weight)
