"""Niridra: a decoder of lightning-attention and latent-attention layers with mixtures of experts.

The residual is several fp32 streams (hyper-connections): a weighted sum of them goes into a sublayer, and every stream
becomes a mix of all of them plus its share of the scaled result.  Lightning layers keep a matrix memory with a constant
decay per head; latent layers attend to one cached latent per token, their own or an earlier layer's.  The embedding adds a
row chosen by a hash of the token and the one before it; the LM head is the embedding table.

The model runs ragged steps only: ``forward`` reads the step from the ``Context``.  Constants and sizes come from the
checkpoint's config.json; tensors keep its names."""
from __future__ import annotations

import os

import torch
import torch.nn as nn

from minivllm_amd.layers.basic import Linear
from minivllm_amd.layers.experts import SparseExperts
from minivllm_amd.layers.fused import stream_embed_norm, stream_norm
from minivllm_amd.layers.mixers import DecayMemory, LatentAttention, attention_head_dim
from minivllm_amd.layers.recurrent import DecayMemoryState
from minivllm_amd.utils.context import get_context
from minivllm_amd.utils.padding import pad_to, round_up
from minivllm_amd.utils.safetensors_io import read_safetensors


def engine_config(config: dict) -> dict:
    """config.json keys as they are, plus the engine's names for what the runner needs."""
    return {**config, "vocab_size": config["vocab"], "hidden_size": config["width"], "num_layers": len(config["layers"])}


def kernel_sources(config: dict) -> list[str]:
    """The csrc files a model of this configuration runs on."""
    sources = ["capi.hip", "activation.hip", "linear_small.hip", "stream_norm.hip"]
    if any(e["type"] == "lightning" for e in config["layers"]):
        sources.append("decay_memory.hip")
    latent = [e["mixer"] for e in config["layers"] if e["type"] == "latent_attention"]
    if latent:
        sources += ["latent.hip", "paged_decode.hip", "prefill_varlen.hip", "prefill_split.hip", "prefill_f32.hip"]
        if any(attention_head_dim(m["dim"], m["vdim"], torch.bfloat16) not in (64, 128) for m in latent):
            sources.append("prefill_other_dims.hip")
    if any(e.get("mlp") is not None for e in config["layers"]):
        sources += ["moe.hip", "gate_linear.hip"]
    return sources


class NiridraLayer(nn.Module):
    def __init__(self, index: int, entry: dict, sources: list, width: int, inputs: int, block_size: int, dtype, eps: float,
                 small_rows: int):
        super().__init__()
        m = entry["mixer"]
        self.kind, self.inputs = entry["type"], inputs
        self.is_attention = self.kind == "latent_attention"
        if self.kind == "lightning":
            if len(m["decay"]) != m["heads"]:
                raise ValueError(f"layer {index}: {m['heads']} heads and {len(m['decay'])} decays")
            self.mixer = DecayMemory(m["heads"], m["dim"], m["vdim"], eps)
            total = 2 * m["heads"] * (m["dim"] + m["vdim"])
            with torch.device("meta"):
                self.proj = Linear(inputs, round_up(total, 16), bias=False, small_rows=small_rows)
                self.out = Linear(m["heads"] * m["vdim"], width, bias=False, small_rows=small_rows)
        elif self.is_attention:
            source = None
            if m.get("kv_from") is not None:
                source = sources[m["kv_from"]].mixer if 0 <= m["kv_from"] < index else None
                if not isinstance(source, LatentAttention) or source.owner is not source or source.rank != m["kv_rank"]:
                    raise ValueError(f"layer {index}: kv_from must name an earlier layer with latents of its own and of the same rank")
            self.mixer = LatentAttention(width, m["heads"], m["dim"], m["vdim"], m["kv_rank"], m["scale"], 0, block_size, dtype, eps,
                                         source, small_rows)
        else:
            raise ValueError(f"unknown mixer type {self.kind!r}")
        self.mlp = None
        if entry.get("mlp") is not None:
            c = entry["mlp"]
            if c.get("kind", "moe") != "moe":
                raise ValueError(f"unknown feed-forward kind {c['kind']!r}")
            router, groups, shared = c["router"], c["router"].get("groups") or {}, c.get("shared") or {}
            self.mlp = SparseExperts(width, inputs, router["experts"], router["top"], c["expert"]["ff"], groups.get("count", 1),
                                     groups.get("keep", 1), shared.get("ff", 0), small_rows=small_rows)
        self.f32 = {}                                   # gains, stream weights and the like: fp32 whatever the model's type

    @torch.no_grad()
    def load(self, tensors: dict, prefix: str, dtype, device):
        def matrix(t):
            return t.to(device=device, dtype=dtype).contiguous()

        def f32(name):
            return tensors[prefix + name].to(device=device, dtype=torch.float32).contiguous()

        def parameter(t):
            return nn.Parameter(t.contiguous(), requires_grad=False)

        get = lambda name: tensors[prefix + "mix." + name]
        if self.is_attention:
            self.mixer.load(get, matrix, self.inputs)
        else:
            rows = torch.cat([matrix(get(n)) for n in ("q", "k", "v", "g")])
            self.proj.weight = parameter(pad_to(rows, self.proj.out_features, self.inputs))
            self.out.weight = parameter(matrix(get("o")))
            self.f32["mix.norm"] = f32("mix.norm")
        for s in ("1", "2") if self.mlp is not None else ("1",):
            for n in (f"norm{s}", f"ls{s}", f"hc{s}.in", f"hc{s}.out", f"hc{s}.mix"):
                self.f32[n] = f32(n)
        if self.mlp is not None:
            self.mlp.load(lambda name: tensors[prefix + "mlp." + name], matrix)

    def mix(self, h, step):
        if self.is_attention:
            return self.mixer(h, step)
        return self.out(self.mixer(self.proj(h), step, self.f32["mix.norm"]))


class NiridraForCausalLM(nn.Module):
    latent_views = True                                 # its attention layers cache latents (engine/ragged.py: LatentStep)

    def __init__(self, config: dict, block_size: int, dtype: torch.dtype, device: torch.device):
        super().__init__()
        self.config, self.dtype, self.device, self.block_size = config, dtype, device, block_size
        self.eps, self.streams, self.width = config["norm"]["eps"], config["streams"], config["width"]
        self.inputs = round_up(self.width, SparseExperts.ALIGN)          # columns of a sublayer's input, zeros past the width
        layers = config["layers"]
        self.windows = [0] if any(e["type"] == "latent_attention" for e in layers) else []
        self.layer_stack = nn.ModuleList()
        for i, entry in enumerate(layers):
            self.layer_stack.append(NiridraLayer(i, entry, self.layer_stack, self.width, self.inputs, block_size, dtype, self.eps,
                                                 config.get("linear_small_rows", 64)))
        # workgroups per segment of the block form of the memories (0: no such layer): how far portions are cut
        self.memory_units = min((e["mixer"]["heads"] * -(-e["mixer"]["vdim"] // 128) for e in layers if e["type"] == "lightning"),
                                default=0)
        bigram = config["embedding"].get("bigram")
        self.hashing = (bigram["buckets"], bigram["mul_prev"], bigram["mul_cur"]) if bigram else None

    # ---- weights ----
    def load_weights(self, tensors: dict) -> None:
        dev = dict(device=self.device, dtype=self.dtype)
        self.embedding = self.lm_head_weight = tensors["embed"].to(**dev).contiguous()
        self.bigram = tensors["bigram"].to(**dev).contiguous() if self.hashing else None
        self.final_norm = tensors["final.norm"].to(device=self.device, dtype=torch.float32).contiguous()
        for i, layer in enumerate(self.layer_stack):
            layer.load(tensors, f"l{i}.", self.dtype, self.device)

    def load_checkpoint(self, model_dir: str) -> None:
        self.load_weights(read_safetensors(os.path.join(model_dir, "model.safetensors")))

    def reset_parameters(self, seed: int = 0) -> None:
        """Random tensors of the configuration's shapes, scaled so that activations keep their size."""
        g = torch.Generator(device=self.device).manual_seed(seed)
        c, width, s = self.config, self.width, self.streams

        def normal(*shape, std=1.0, mean=0.0):
            return (torch.randn(shape, generator=g, device=self.device) * std + mean).to(torch.bfloat16)

        def linear(rows, columns):
            return normal(rows, columns, std=columns ** -0.5)

        t = {"embed": linear(c["vocab"], width), "final.norm": normal(width, std=0.0, mean=1.0)}
        if self.hashing:
            t["bigram"] = normal(self.hashing[0] + 1, width, std=0.1)
        for i, entry in enumerate(c["layers"]):
            m, p = entry["mixer"], f"l{i}."
            for q in ("1", "2") if entry.get("mlp") is not None else ("1",):
                t.update({f"{p}norm{q}": normal(width, std=0.0, mean=1.0), f"{p}ls{q}": normal(width, std=0.0, mean=0.5),
                          f"{p}hc{q}.in": normal(s, std=0.1, mean=1.0 / s), f"{p}hc{q}.out": normal(s, std=0.1, mean=1.0),
                          f"{p}hc{q}.mix": normal(s, s, std=0.05) + torch.eye(s, device=self.device).bfloat16()})
            heads, dim, vdim = m["heads"], m["dim"], m["vdim"]
            t[p + "mix.q"], t[p + "mix.o"] = linear(heads * dim, width), linear(width, heads * vdim)
            if entry["type"] == "lightning":
                t.update({p + "mix.k": linear(heads * dim, width), p + "mix.v": linear(heads * vdim, width),
                          p + "mix.g": linear(heads * vdim, width), p + "mix.norm": normal(heads * vdim, std=0.0, mean=1.0)})
            else:
                rank = m["kv_rank"]
                t.update({p + "mix.uk": linear(heads * dim, rank), p + "mix.uv": linear(heads * vdim, rank)})
                if m.get("kv_from") is None:
                    t.update({p + "mix.dkv": linear(rank, width), p + "mix.dkv.norm": normal(rank, std=0.0, mean=1.0)})
            if entry.get("mlp") is not None:
                e, n = entry["mlp"], p + "mlp."
                forms = [(f"{n}e{j}.", e["expert"]["ff"]) for j in range(e["router"]["experts"])]
                if e.get("shared"):
                    forms.append((n + "shared.", e["shared"]["ff"]))
                    t[n + "shared.sg"] = linear(1, width)
                for name, ff in forms:
                    t.update({name + "gate": linear(ff, width), name + "up": linear(ff, width), name + "down": linear(width, ff)})
                t.update({n + "router": linear(e["router"]["experts"], width), n + "correction": normal(e["router"]["experts"], std=0.1)})
        self.load_weights(t)

    # ---- caches and states ----
    def allocate_state(self, num_blocks: int, num_slots: int) -> None:
        """A pool of ``num_blocks`` blocks of latents per layer that has latents of its own, a memory per slot and lightning
        layer, and two banks per slot for the token before a step (an entry of several rows reads one and writes the other),
        one for padding rows."""
        for layer, entry in zip(self.layer_stack, self.config["layers"]):
            m = layer.mixer
            if not layer.is_attention:
                m.state = DecayMemoryState.allocate(num_slots, entry["mixer"]["decay"], m.dim, m.vdim, self.device)
            elif m.owner is m:
                m.cache = torch.zeros(num_blocks, self.block_size, m.latent_width, dtype=self.dtype, device=self.device)
        self.prev_tokens = torch.zeros(2 * num_slots + 1, dtype=torch.int64, device=self.device)

    def forward(self, input_ids, positions, layer_outputs: list | None = None):
        """Final hidden states (T, width) of the context's ragged step; ``layer_outputs`` collects the sum of the residual
        streams after every layer (tests)."""
        step, layers = get_context().ragged, self.layer_stack
        h, x = stream_embed_norm(step, input_ids, self.embedding, self.config["embedding"]["scale"], self.streams,
                                 layers[0].f32["norm1"], self.eps, layers[0].f32["hc1.in"], self.bigram, self.hashing or (1, 0, 0),
                                 self.prev_tokens, self.inputs)
        for i, layer in enumerate(layers):
            f, y, q = layer.f32, layer.mix(h, step), "1"
            if layer.mlp is not None:
                h, x = stream_norm(x, y, f["hc1.out"], f["hc1.mix"], f["norm2"], self.eps, f["hc2.in"], f["ls1"], self.inputs)
                y, q = layer.mlp(h), "2"
            last = i + 1 == len(layers)
            after = {} if last else dict(hc_in=layers[i + 1].f32["hc1.in"], padded=self.inputs)
            h, x = stream_norm(x, y, f[f"hc{q}.out"], f[f"hc{q}.mix"], self.final_norm if last else layers[i + 1].f32["norm1"], self.eps,
                               scale=f["ls" + q], want_x=not last or layer_outputs is not None, **after)
            if layer_outputs is not None:
                layer_outputs.append(x.sum(1))
        return h

    def compute_logits(self, hidden):
        return torch.nn.functional.linear(hidden, self.lm_head_weight)
