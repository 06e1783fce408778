"""Lenuzen: a decoder that norms what its sublayers return and nothing else: x + norm(mixer(x)), then x + norm(ff(x)).

Mixers are windowed attention over unit heads (biases, a factor per head on the scores, a gate per head) and chunked attention
whose heads' scores are mixed, with a sink; the feed-forward is dense with gelu, or absent.  One launch adds a sublayer's normed
result to the residual and hands the new residual on.  The residual is fp32; the head is the embedding table.

The model runs ragged steps only: ``forward`` reads the step from the ``Context``.  Constants and sizes come from the
checkpoint's config.json; tensors keep its names."""
from __future__ import annotations

import os

import torch
import torch.nn as nn

from minivllm_amd.engine.windows import SlidingWindow, places
from minivllm_amd.layers.basic import Linear, rotary_pair_table
from minivllm_amd.layers.fused import embed_rows, post_norm
from minivllm_amd.layers.mixers import TalkingAttention, UnitHeadAttention
from minivllm_amd.utils.context import get_context
from minivllm_amd.utils.padding import pad_to, round_up
from minivllm_amd.utils.safetensors_io import read_safetensors

SINK = 0.0                              # of the mixed heads: one more exp(SINK) in a softmax's denominator
UNIT, TALKING = "attention", "attention_2"


def engine_config(config: dict) -> dict:
    """config.json keys as they are, plus the engine's names for what the runner needs."""
    return {**config, "vocab_size": config["vocab"], "hidden_size": config["width"], "num_layers": len(config["layers"])}


def kernel_sources(config: dict) -> list[str]:
    """The csrc files a model of this configuration runs on."""
    kinds = {e["type"] for e in config["layers"]}
    sources = ["capi.hip", "activation.hip", "linear_small.hip", "post_norm.hip", "head_rope.hip"]
    if UNIT in kinds:
        sources += ["ring_rows.hip", "window_prefill.hip", "window_prefill_heads.hip", "window_decode.hip", "window_decode_split.hip"]
    if TALKING in kinds:
        sources += ["store_kvcache.hip", "talk.hip", "talk_prefill.hip", "talk_decode.hip"]
    return sources


def _window(entry: dict):
    """A sliding window, or a plain number: the size of chunks."""
    size = int((entry["mixer"].get("mask") or {}).get("size") or 0)
    return SlidingWindow(size) if entry["type"] == UNIT else size


class LenuzenLayer(nn.Module):
    is_attention = True

    def __init__(self, entry: dict, width: int, inputs: int, windows: list, block_size: int, dtype, eps: float, small_rows: int):
        super().__init__()
        m, kind, view = entry["mixer"], entry["type"], _window(entry)
        sizes = (m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"], windows.index(view))
        if kind == UNIT:
            self.mixer = UnitHeadAttention(inputs, *sizes, view, block_size, dtype, eps, small_rows=small_rows)
        elif kind == TALKING:
            self.mixer = TalkingAttention(inputs, *sizes, block_size, dtype, eps, sink=SINK, small_rows=small_rows)
        else:
            raise ValueError(f"unknown mixer type {kind!r}")
        self.width, self.inputs, self.ff = width, inputs, 0
        if entry.get("mlp") is not None:
            if entry["mlp"].get("kind", "dense") != "dense":
                raise ValueError(f"unknown feed-forward kind {entry['mlp']['kind']!r}")
            self.ff = round_up(entry["mlp"]["ff"], 64)
            with torch.device("meta"):
                self.up = Linear(inputs, self.ff, bias=False, small_rows=small_rows)
                self.down = Linear(self.ff, width, bias=False, small_rows=small_rows)

    @torch.no_grad()
    def load(self, tensors: dict, prefix: str, dtype, device):
        def matrix(t):
            return t.to(device=device, dtype=dtype).contiguous()

        get = lambda name: tensors[prefix + name]
        f32 = lambda name: get(name).to(device=device, dtype=torch.float32).contiguous()
        self.mixer.load(lambda name: get("mix." + name), matrix, self.inputs)
        self.gains = [f32("norm1")]
        if self.ff:
            self.gains.append(f32("norm2"))
            self.up.weight = nn.Parameter(pad_to(matrix(get("mlp.up")), self.ff, self.inputs), requires_grad=False)
            self.down.weight = nn.Parameter(pad_to(matrix(get("mlp.down")), None, self.ff), requires_grad=False)

    def feed_forward(self, h):
        return self.down(self.up(h, gelu=True))


class LenuzenForCausalLM(nn.Module):
    latent_views = False                                # its windows are sliding ones (engine/windows.py) and chunks
    memory_units = 0                                    # no recurrence

    def __init__(self, config: dict, block_size: int, dtype: torch.dtype, device: torch.device):
        super().__init__()
        self.config, self.dtype, self.device, self.block_size = config, dtype, device, block_size
        self.eps, self.width = config["norm"]["eps"], config["width"]
        self.inputs = round_up(self.width, 64)          # columns of what a sublayer reads, zeros past the width
        layers = config["layers"]
        self.windows = sorted({_window(e) for e in layers}, key=lambda w: (isinstance(w, SlidingWindow), places(w)))
        self.layer_stack = nn.ModuleList(LenuzenLayer(e, self.width, self.inputs, self.windows, block_size, dtype, self.eps,
                                                      config.get("linear_small_rows", 64)) for e in layers)
        max_position, tables = config.get("max_position", 4096), {}
        for layer, entry in zip(self.layer_stack, layers):
            rot = entry["mixer"].get("rot") or {}
            if not rot.get("dims"):
                continue
            if rot["dims"] > entry["mixer"]["dim"]:
                raise ValueError(f"{rot['dims']} rotated dimensions of {entry['mixer']['dim']}")
            key = (rot["base"], rot["dims"], tuple(sorted((rot.get("scaling") or {}).items())))
            if key not in tables:
                tables[key] = rotary_pair_table(rot["base"], rot["dims"], max_position, rot.get("scaling") or None).to(device)
            layer.mixer.table = tables[key]

    # ---- weights ----
    def load_weights(self, tensors: dict) -> None:
        self.embedding = tensors["embed"].to(device=self.device, dtype=self.dtype).contiguous()
        self.lm_head_weight = self.embedding
        # the factor on the logits is one on the rows they are made of
        self.final_gain = (tensors["final.norm"].to(device=self.device, dtype=torch.float32) * self.config["logit_scale"]).contiguous()
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

        t = {"embed": normal(c["vocab"], width), "final.norm": normal(width, std=0.0, mean=1.0)}
        for i, entry in enumerate(c["layers"]):
            m, p, f = entry["mixer"], f"l{i}.mix.", entry.get("mlp")
            heads, rows = m["heads"], {"q": m["heads"] * m["dim"], "k": m["kv_heads"] * m["dim"], "v": m["kv_heads"] * m["vdim"]}
            t[f"l{i}.norm1"] = normal(width, std=0.0, mean=1.0)
            t.update({p + n: linear(r, width) for n, r in rows.items()})
            t[p + "o"] = linear(width, heads * m["vdim"])
            if entry["type"] == UNIT:
                t.update({f"{p}{n}.b": normal(r, std=0.1) for n, r in rows.items()})
                t.update({p + "temp": normal(heads, std=0.0, mean=1.0), p + "g": linear(heads, width)})
            else:
                t.update({f"{p}{n}.norm": normal(rows[n], std=0.0, mean=1.0) for n in ("q", "k")})
                t[p + "talk"] = (torch.eye(heads, device=self.device) + 0.1 * normal(heads, heads).float()).to(torch.bfloat16)
            if f is not None:
                t.update({f"l{i}.norm2": normal(width, std=0.0, mean=1.0), f"l{i}.mlp.up": linear(f["ff"], width),
                          f"l{i}.mlp.down": linear(width, f["ff"])})
        self.load_weights(t)

    # ---- caches ----
    def allocate_state(self, num_blocks: int, num_slots: int) -> None:
        """A pool of ``num_blocks`` blocks per layer; nothing is kept per slot."""
        for layer in self.layer_stack:
            layer.mixer.allocate(num_blocks, self.device)

    def forward(self, input_ids, positions, layer_outputs: list | None = None):
        """Final hidden states (T, width) of the context's ragged step; ``layer_outputs`` collects the residual after every layer
        (tests)."""
        step, layers = get_context().ragged, self.layer_stack
        h, x = embed_rows(input_ids, self.embedding, self.config["embedding"]["scale"], padded=self.inputs)
        for layer in layers:
            for sublayer, gain in zip((lambda h: layer.mixer(h, step), layer.feed_forward), layer.gains):
                last = layer is layers[-1] and gain is layer.gains[-1]
                h, x = post_norm(x, sublayer(h), gain, self.eps, final_gain=self.final_gain if last else None,
                                 padded=0 if last else self.inputs, want_x=not last or layer_outputs is not None)
            if layer_outputs is not None:
                layer_outputs.append(x.clone())
        return h

    def compute_logits(self, hidden):
        return torch.nn.functional.linear(hidden, self.lm_head_weight)
