"""Runner of models that run ragged steps and keep recurrent state (models/sokevik.py, models/niridra.py, models/fevosun.py,
models/lenuzen.py): portions of prompts and decoded tokens in one batch, a cache manager of its own, and the captured decode step
of ``ModelRunner`` over more static buffers.

Engine keys as for ``ModelRunner``; ``max_cached_blocks`` counts the blocks of each attention window's pool,
``max_num_sequences`` the slots of recurrent state, ``model_dir`` names a checkpoint folder (absent: random weights)."""
from __future__ import annotations

import torch

from minivllm_amd.engine.hybrid_cache import HybridCacheManager
from minivllm_amd.engine.model_runner import _DTYPES, ModelRunner
from minivllm_amd.engine.ragged import LatentStep, RaggedStep, RingStep, WindowStep, ragged_step
from minivllm_amd.engine.windows import SlidingWindow, places
from minivllm_amd.layers.fused import chunk_decode_step, lm_head_sample, lm_head_sample_takes, sample_tokens
from minivllm_amd.utils.context import reset_context, set_context


class HybridModelRunner(ModelRunner):
    def __init__(self, config: dict, model_class, device: str = "cuda:0"):
        if config.get("kv_cache_dtype", "auto") != "auto" or config.get("dtype", "bf16") in ("fp16", "float16"):
            raise ValueError("this model runs in bf16 or fp32 with a cache of that type")
        if config.get("block_size", 256) % 16:
            raise ValueError("block_size must be a multiple of 16")
        self.model_class = model_class
        super().__init__(config, device)

    def build_model(self):
        torch.backends.cuda.matmul.allow_tf32 = False            # fp32 means fp32
        model = self.model_class(self.config, self.block_size, _DTYPES[self.config.get("dtype", "bf16")], self.device)
        if self.config.get("model_dir"):
            model.load_checkpoint(self.config["model_dir"])
        else:
            model.reset_parameters(self.config.get("seed", 0))
        return model.eval()

    def allocate_kv_cache(self):
        slots = self.config.get("max_num_sequences", 16)
        self.cache_manager = HybridCacheManager(self.model.windows, self.num_blocks, self.block_size, slots)
        self.model.allocate_state(self.num_blocks, slots)
        self._dummy_bank = 2 * slots

    # ---- ragged steps ----
    @torch.inference_mode()
    def forward_step(self, seqs, layer_outputs=None):
        """Run every sequence's scheduled tokens; returns (hidden rows, the step)."""
        step = ragged_step(seqs, self.model.windows, self.block_size, self.device, self.model.memory_units,
                           self.model.latent_views)
        set_context(step.multi_rows > 0, ragged=step)
        try:
            hidden = self.model(step.input_ids, step.positions, layer_outputs)
        finally:
            reset_context()
        self._last_sampled = self._steady = None
        return hidden, step

    @torch.inference_mode()
    def step_logits(self, seqs, wanted):
        """Logits of places among the scheduled tokens (``wanted[i]`` of sequence i, in that order): float32 (n, vocab)."""
        hidden, step = self.forward_step(seqs)
        rows = [step.starts[i] + p for i, places in enumerate(wanted) for p in places]
        if not rows:
            return None
        return self.model.compute_logits(hidden[self._to_device(rows, torch.int64)]).float()

    @torch.inference_mode()
    def run(self, seqs, is_prefill: bool) -> list:
        if not is_prefill and self.can_launch_decode(seqs):
            return super().run(seqs, is_prefill)
        hidden, step = self.forward_step(seqs)
        # sequences whose last token the step brought are sampled; the others have prompt tokens to come
        done = [i for i, s in enumerate(seqs) if s.num_computed_tokens + s.num_scheduled_tokens == len(s)]
        out = [None] * len(seqs)
        if not done:
            return out
        rows = self._to_device([step.starts[i] + seqs[i].num_scheduled_tokens - 1 for i in done], torch.int64)
        temperatures = self._to_device([seqs[i].temperature for i in done], torch.float32)
        weight = self.model.lm_head_weight
        if self.fused_lm_head and lm_head_sample_takes(hidden, weight, len(done)):
            ids = lm_head_sample(hidden, weight, temperatures, self.seed, self.sample_calls, row_index=rows)
        elif self.fused_sampler:
            ids = sample_tokens(self.model.compute_logits(hidden[rows]), temperatures, self.seed, self.sample_calls)
        else:
            ids = self.sampler(self.model.compute_logits(hidden[rows]), temperatures, self.generator)
        self.sample_calls += 1
        for i, token in zip(done, ids.tolist()):
            out[i] = token
        return out

    # ---- captured decode ----
    def _table_widths(self):
        longest = self.config.get("max_model_length", self.config.get("max_position", 4096))
        return [self.cache_manager.blocks_for(w, longest) for w in self.model.windows]

    def _own_decode_workspace(self, buckets, max_blocks):
        need, widths = 16, self._table_widths()
        for layer in self.model.layer_stack:
            if layer.is_attention:
                need = max([need] + [layer.mixer.workspace_bytes(b, widths[layer.mixer.window]) for b in buckets])
        self.decode_workspace = torch.empty(need, dtype=torch.uint8, device=self.device)
        for layer in self.model.layer_stack:
            if layer.is_attention:
                layer.mixer.decode_workspace = self.decode_workspace
        # the static buffers a captured step reads beside the base class's
        n, dev = max(buckets), self.device
        self.graph_vars.update(
            cu_seqlens=torch.arange(n + 1, dtype=torch.int32, device=dev), row_entry=torch.arange(n, dtype=torch.int32, device=dev),
            banks=torch.full((n,), self._dummy_bank, dtype=torch.int32, device=dev),
            state_slots=torch.full((n,), -1, dtype=torch.int32, device=dev),
            tables=[torch.full((n, w), -1, dtype=torch.int32, device=dev) for w in self._table_widths()],
            chunk_lens=[torch.zeros(n, dtype=torch.int64, device=dev) for _ in self.model.windows],
            chunk_slots=[torch.full((n,), -1, dtype=torch.int64, device=dev) for _ in self.model.windows])

    def _captured_context(self, bs):
        v = self.graph_vars
        lens, slots = [t[:bs] for t in v["chunk_lens"]], [t[:bs] for t in v["chunk_slots"]]
        tables = [t[:bs] for t in v["tables"]]

        def view(w, s, n, t):
            if isinstance(w, SlidingWindow):
                return RingStep(absorbed=bs, slots=s, lens=v["context_lens"][:bs], tables=t)
            if self.model.latent_views:
                return LatentStep(absorbed=bs, slots=s, lens=n, tables=t)
            return WindowStep(num_decode=bs, slots=s, chunk_lens=n, decode_tables=t)

        windows = [view(*of) for of in zip(self.model.windows, slots, lens, tables)]
        step = RaggedStep(num_tokens=bs, num_entries=bs, num_single=bs, num_short=bs, input_ids=v["input_ids"][:bs],
                          positions=v["positions"][:bs], cu_seqlens=v["cu_seqlens"][:bs + 1], row_entry=v["row_entry"][:bs],
                          bank_in=v["banks"][:bs], bank_out=v["banks"][:bs], state_slots=v["state_slots"][:bs], windows=windows)
        set_context(False, ragged=step)

        def prepare():
            # where the rows' tokens lie in their chunks (rings) follows from the context lengths the step before left behind
            for w, t, n, s in zip(self.model.windows, tables, lens, slots):
                chunk_decode_step(v["context_lens"][:bs], t, places(w), self.block_size, n, s)
        return prepare

    def _fill_decode_buffers(self, seqs, gbs):
        bs, v = len(seqs), self.graph_vars
        pad = gbs - bs
        v["input_ids"][:bs].copy_(self._to_device([s.last_token for s in seqs], torch.int64))
        v["positions"][:gbs].copy_(self._to_device([len(s) - 1 for s in seqs] + [0] * pad, torch.int64))
        v["context_lens"][:gbs].copy_(self._to_device([len(s) for s in seqs] + [0] * pad, torch.int64))
        v["temperatures"][:gbs].copy_(self._to_device([s.temperature for s in seqs] + [1.0] * pad, torch.float32))
        v["banks"][:gbs].copy_(self._to_device([2 * s.state_slot + s.state_bank for s in seqs] + [self._dummy_bank] * pad, torch.int32))
        v["state_slots"][:gbs].copy_(self._to_device([s.state_slot for s in seqs] + [-1] * pad, torch.int32))
        for g, table in enumerate(v["tables"]):
            width = max(len(s.group_tables[g]) for s in seqs)
            rows = [s.group_tables[g] + [-1] * (width - len(s.group_tables[g])) for s in seqs]
            table[:bs, :width].copy_(self._to_device(rows, torch.int32))
        self._steady = dict(key=tuple(s.seq_id for s in seqs), lens=[len(s) for s in seqs],
                            held=[[len(t) for t in s.group_tables] for s in seqs])

    def _advance_decode_buffers(self, seqs) -> bool:
        if not self.continues_last_decode(seqs):
            return False
        st = self._steady
        for g, table in enumerate(self.graph_vars["tables"]):
            fresh = [i for i, s in enumerate(seqs) if len(s.group_tables[g]) > st["held"][i][g]]
            if fresh:
                rows = self._to_device(fresh, torch.int64)
                cols = self._to_device([len(seqs[i].group_tables[g]) - 1 for i in fresh], torch.int64)
                table[rows, cols] = self._to_device([seqs[i].group_tables[g][-1] for i in fresh], torch.int32)
        st["lens"] = [len(s) for s in seqs]
        st["held"] = [[len(t) for t in s.group_tables] for s in seqs]
        return True
