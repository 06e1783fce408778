"""Sokevik: a decoder of chunked-attention and matrix-memory (mLSTM) layers.

Every sublayer stands between two norms with a single gain, behind a short causal convolution over time:
``x + norm_b(f(h + conv(h)))``, ``h = norm(x)``.  Attention layers see their own chunk of the sequence only, with a sink in
the softmax, rotated values and a gate per head; a layer may have a gated feed-forward or none, and may share the weights
of another layer (its caches are its own).  The residual stream, norms, convolution state and recurrence are fp32.

The model runs ragged steps only: ``forward`` reads the step from the ``Context``.  Constants and sizes come from the
checkpoint's config.json; tensors keep its names."""
from __future__ import annotations

import os

import torch
import torch.nn as nn

from minivllm_amd.layers.basic import Linear, rotary_pair_table
from minivllm_amd.layers.fused import norm_conv
from minivllm_amd.layers.mixers import MatrixMemory, RaggedAttention, attention_head_dim
from minivllm_amd.layers.recurrent import MlstmState
from minivllm_amd.models.qwen3 import Qwen3MLP
from minivllm_amd.utils.context import get_context
from minivllm_amd.utils.safetensors_io import read_safetensors


def engine_config(config: dict) -> dict:
    """config.json keys as they are, plus the engine's names for what the runner needs."""
    return {**config, "vocab_size": config["vocab"], "hidden_size": config["width"], "num_layers": len(config["layers"])}


def _owner(layers, i):
    """The layer whose weights layer i uses."""
    seen = set()
    while layers[i].get("weights_of") is not None:
        if i in seen:
            raise ValueError(f"layer {i}: weights_of runs in a circle")
        seen.add(i)
        i = layers[i]["weights_of"]
    return i


def _window(mixer: dict) -> int:
    return int((mixer.get("mask") or {}).get("size") or 0)


def kernel_sources(config: dict) -> list[str]:
    """The csrc files a model of this configuration runs on."""
    sources = ["capi.hip", "activation.hip", "linear_small.hip", "norm_conv.hip"]
    if any(e["type"] == "mlstm" for e in config["layers"]):
        sources += ["gate_linear.hip", "mlstm.hip", "mlstm_chunk.hip"]
    attention = [e["mixer"] for e in config["layers"] if e["type"] == "attention"]
    if attention:
        sources += ["head_rope.hip", "store_kvcache.hip", "paged_decode.hip", "prefill_varlen.hip", "prefill_split.hip",
                    "prefill_f32.hip"]
        if any(attention_head_dim(m["dim"], m["vdim"], torch.bfloat16) not in (64, 128) for m in attention):
            sources.append("prefill_other_dims.hip")
    return sources


def _pad_rows(t, multiple):
    extra = -t.shape[0] % multiple
    return torch.cat([t, t.new_zeros(extra, *t.shape[1:])]) if extra else t


class LayerWeights(nn.Module):
    """Tensors of one layer, for it and every layer that shares them."""

    def __init__(self, entry: dict, width: int, small_rows: int):
        super().__init__()
        self.entry, m = entry, entry["mixer"]
        heads = m["heads"]
        if entry["type"] == "attention":
            self.columns = heads * m["dim"] + m["kv_heads"] * (m["dim"] + m["vdim"])     # where the gates start
            total = self.columns + heads
        elif entry["type"] == "mlstm":
            self.columns = heads * (2 * m["dim"] + m["vdim"])
            total = self.columns + heads * m["vdim"]
        else:
            raise ValueError(f"unknown mixer type {entry['type']!r}")
        self.proj = Linear(width, -(-total // 16) * 16, bias=False, small_rows=small_rows)
        self.out = Linear(heads * m["vdim"], width, bias=False, small_rows=small_rows)
        self.mlp = None
        if entry.get("mlp") is not None:
            if entry["mlp"].get("kind", "dense") != "dense":
                raise ValueError(f"unknown feed-forward kind {entry['mlp']['kind']!r}")
            self.mlp = Qwen3MLP(width, -(-entry["mlp"]["ff"] // 16) * 16, False, True, small_rows)
        self.f32 = {}                                   # gains, taps, gate biases and the like: fp32 whatever the model's type

    @torch.no_grad()
    def load(self, tensors: dict, prefix: str, dtype, device):
        def get(name):
            return tensors[prefix + name]

        def matrix(t):
            return nn.Parameter(t.to(device=device, dtype=dtype).contiguous(), requires_grad=False)

        def f32(name):
            return get(name).to(device=device, dtype=torch.float32).contiguous()

        kind = self.entry["type"]
        self.proj.weight = matrix(_pad_rows(torch.cat([get("mix.q"), get("mix.k"), get("mix.v"), get("mix.g")]), 16))
        self.out.weight = matrix(get("mix.o"))
        self.f32 = {n: f32(n) for n in ("norm1", "norm1b")}
        self.f32["canon1"] = f32("canon1").t().contiguous()                    # (taps, width)
        if kind == "attention":
            self.f32.update(q_norm=f32("mix.q.norm"), k_norm=f32("mix.k.norm"), sink=f32("mix.sink"))
        else:
            self.gate_weight = matrix(torch.cat([get("mix.i"), get("mix.f")]))
            self.f32.update(gate_bias=torch.cat([f32("mix.i.b"), f32("mix.f.b")]), norm=f32("mix.norm"))
        if self.mlp is not None:
            self.f32.update({n: f32(n) for n in ("norm2", "norm2b")})
            self.f32["canon2"] = f32("canon2").t().contiguous()
            self.mlp.gate_up.weight = matrix(torch.cat([_pad_rows(get("mlp.gate"), 16), _pad_rows(get("mlp.up"), 16)]))
            self.mlp.gate_down.weight = matrix(_pad_rows(get("mlp.down").t(), 16).t())


class SokevikLayer(nn.Module):
    def __init__(self, weights: LayerWeights, entry: dict, windows: list, block_size: int, dtype, eps: float):
        super().__init__()
        self.weights, m = weights, entry["mixer"]
        self.is_attention = entry["type"] == "attention"
        if self.is_attention:
            self.mixer = RaggedAttention(m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"],
                                         windows.index(_window(m)), block_size, dtype, eps, gate_col=weights.columns)
        else:
            self.mixer = MatrixMemory(m["heads"], m["dim"], m["vdim"], m["gate_cap"], eps)
        self.conv_state = None                          # (banks, taps - 1, width) per sublayer, assigned from outside
        self.tables = (None, None)                      # rotary tables of q / k and of the values

    def mix(self, h, step):
        w = self.weights
        proj = w.proj(h)
        if self.is_attention:
            o = self.mixer(proj, step, w.f32["q_norm"], w.f32["k_norm"], *self.tables, w.f32["sink"])
        else:
            o = self.mixer(h, proj, step, w.gate_weight, w.f32["gate_bias"], w.f32["norm"])
        return w.out(o)


class SokevikForCausalLM(nn.Module):
    latent_views = False                                # its attention layers cache keys and values

    def __init__(self, config: dict, block_size: int, dtype: torch.dtype, device: torch.device):
        super().__init__()
        self.config, self.dtype, self.device, self.block_size = config, dtype, device, block_size
        self.eps, self.taps = config["norm"]["eps"], config["canon"]["taps"]
        layers, width = config["layers"], config["width"]
        self.owners = [_owner(layers, i) for i in range(len(layers))]
        small_rows = config.get("linear_small_rows", 64)
        with torch.device("meta"):
            shared = {j: LayerWeights(layers[j], width, small_rows) for j in sorted(set(self.owners))}
        self.shared = nn.ModuleDict({str(j): w for j, w in shared.items()})
        # attention windows: layers of one window share a block table
        self.windows = sorted({_window(e["mixer"]) for e in layers if e["type"] == "attention"})
        self.layer_stack = nn.ModuleList([
            SokevikLayer(shared[j], layers[i], self.windows, block_size, dtype, self.eps) for i, j in enumerate(self.owners)])
        # workgroups per segment of the block form of the matrix memory (0: no such layer): how far portions are cut
        self.memory_units = min((e["mixer"]["heads"] * -(-e["mixer"]["vdim"] // 128) for e in layers if e["type"] == "mlstm"),
                                default=0)
        max_position, tables = config.get("max_position", 4096), {}

        def table(base, dims, scaling):
            key = (base, dims, tuple(sorted(scaling.items())) if scaling else None)
            if key not in tables:
                tables[key] = rotary_pair_table(base, dims, max_position, scaling).to(device)
            return tables[key]

        for layer, entry in zip(self.layer_stack, layers):
            if layer.is_attention:
                m = entry["mixer"]
                rot = m["rot"]
                layer.tables = (table(rot["base"], rot["dims"], rot.get("scaling")) if rot["dims"] else None,
                                table(rot["base"], m["vdim"], None))

    # ---- weights ----
    def load_weights(self, tensors: dict) -> None:
        dev = dict(device=self.device, dtype=self.dtype)
        self.embedding = tensors["embed"].to(**dev).contiguous()
        self.lm_head_weight = tensors["head"].to(**dev).contiguous()
        self.final_norm = tensors["final.norm"].to(device=self.device, dtype=torch.float32)
        for name, weights in self.shared.items():
            weights.load(tensors, f"l{name}.", self.dtype, self.device)

    def load_checkpoint(self, model_dir: str) -> None:
        self.load_weights(read_safetensors(os.path.join(model_dir, "model.safetensors")))

    def reset_parameters(self, seed: int = 0) -> None:
        """Random tensors of the configuration's shapes, scaled so that activations keep their size."""
        g = torch.Generator(device=self.device).manual_seed(seed)
        c = self.config
        width = c["width"]

        def normal(*shape, std=1.0, mean=0.0):
            return (torch.randn(shape, generator=g, device=self.device) * std + mean).to(torch.bfloat16)

        t = {"embed": normal(c["vocab"], width), "head": normal(c["vocab"], width, std=width ** -0.5),
             "final.norm": normal(mean=1.0, std=0.0)}
        for j in sorted(set(self.owners)):
            entry = c["layers"][j]
            m, p = entry["mixer"], f"l{j}."
            heads, kv = m["heads"], m.get("kv_heads", m["heads"])
            for s in ("1", "2") if entry.get("mlp") is not None else ("1",):
                t.update({f"{p}norm{s}": normal(mean=1.0, std=0.0), f"{p}norm{s}b": normal(mean=0.5, std=0.0),
                          f"{p}canon{s}": normal(width, self.taps, std=0.1)})
            for n, rows in (("q", heads * m["dim"]), ("k", kv * m["dim"]), ("v", kv * m["vdim"])):
                t[f"{p}mix.{n}"] = normal(rows, width, std=width ** -0.5)
            t[p + "mix.o"] = normal(width, heads * m["vdim"], std=(heads * m["vdim"]) ** -0.5)
            if entry["type"] == "attention":
                t.update({p + "mix.q.norm": normal(m["dim"], mean=1.0, std=0.0), p + "mix.k.norm": normal(m["dim"], mean=1.0, std=0.0),
                          p + "mix.sink": normal(heads), p + "mix.g": normal(heads, width, std=width ** -0.5)})
            else:
                t.update({p + "mix.g": normal(heads * m["vdim"], width, std=width ** -0.5),
                          p + "mix.norm": normal(heads * m["vdim"], mean=1.0, std=0.0),
                          p + "mix.i": normal(heads, width, std=width ** -0.5), p + "mix.i.b": normal(heads),
                          p + "mix.f": normal(heads, width, std=width ** -0.5), p + "mix.f.b": normal(heads, mean=4.0)})
            if entry.get("mlp") is not None:
                ff = entry["mlp"]["ff"]
                t.update({p + "mlp.gate": normal(ff, width, std=width ** -0.5), p + "mlp.up": normal(ff, width, std=width ** -0.5),
                          p + "mlp.down": normal(width, ff, std=ff ** -0.5)})
        self.load_weights(t)

    # ---- caches and states ----
    def allocate_state(self, num_blocks: int, num_slots: int) -> None:
        """Key / value pools of ``num_blocks`` blocks per attention layer, recurrent state and two convolution banks per
        slot and sublayer (an entry of several rows reads one and writes the other), one bank for padding rows."""
        dev, c = self.device, self.config
        for layer, entry in zip(self.layer_stack, c["layers"]):
            mixer, m = layer.mixer, entry["mixer"]
            if layer.is_attention:
                shape = (num_blocks, self.block_size, m["kv_heads"], mixer.head_dim)
                mixer.k_cache = torch.zeros(shape, dtype=self.dtype, device=dev)
                mixer.v_cache = torch.zeros(shape, dtype=self.dtype, device=dev)
            else:
                mixer.state = MlstmState.allocate(num_slots, m["heads"], m["dim"], m["vdim"], dev)
            subs = 1 if entry.get("mlp") is None else 2
            layer.conv_state = [torch.zeros(2 * num_slots + 1, max(self.taps - 1, 1), c["width"], dtype=torch.float32,
                                            device=dev) for _ in range(subs)]

    def forward(self, input_ids, positions, layer_outputs: list | None = None):
        """Final hidden states (T, width) of the context's ragged step; ``layer_outputs`` collects the residual stream
        after every layer (tests)."""
        step = get_context().ragged
        x, y, post = None, None, None                   # residual stream, output of the sublayer before, its norm's gain
        embed = dict(tokens=input_ids, embed=self.embedding)
        for layer in self.layer_stack:
            w = layer.weights
            h, x = norm_conv(step, w.f32["norm1"], self.eps, self.dtype, x=x, y=y, post=post, conv=w.f32["canon1"],
                             state=layer.conv_state[0], **embed)
            embed = {}
            if layer_outputs is not None:
                layer_outputs.append(x)
            y, post = layer.mix(h, step), w.f32["norm1b"]
            if w.mlp is not None:
                h, x = norm_conv(step, w.f32["norm2"], self.eps, self.dtype, x=x, y=y, post=post, conv=w.f32["canon2"],
                                 state=layer.conv_state[1])
                y, post = w.mlp(h), w.f32["norm2b"]
        h, x = norm_conv(step, self.final_norm, self.eps, self.dtype, x=x, y=y, post=post, want_x=layer_outputs is not None)
        if layer_outputs is not None:
            layer_outputs.append(x)
            del layer_outputs[0]                        # the embedding
        return h

    def compute_logits(self, hidden):
        return torch.nn.functional.linear(hidden, self.lm_head_weight)
