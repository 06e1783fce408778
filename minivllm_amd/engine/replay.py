"""Replay of a step trace: given token ids run through a model step by step, logits of chosen places written to files.

Steps are JSON objects, one a line:
    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}
All entries of a step are one ragged batch; a request is admitted at its first entry and gives its cache and state back
when ``end`` names it.  The steps run on the engine's own runner and cache manager; nothing is sampled."""
from __future__ import annotations

import json
import os

from minivllm_amd.engine.llm_engine import LLMEngine
from minivllm_amd.engine.sequence import Sequence


class TraceReplay:
    def __init__(self, engine: LLMEngine):
        self.runner = engine.model_runner
        self.cache = engine.scheduler.block_manager
        self.block_size = engine.block_size
        self.live: dict[str, Sequence] = {}

    def run_step(self, step: dict):
        """float32 logits (wanted, vocab) of the step, None if nothing is wanted."""
        seqs, wanted = [], []
        for entry in step["entries"]:
            tokens = entry["tokens"]
            if not tokens:
                if entry["want"]:
                    raise ValueError("an entry without tokens has no places to ask for")
                continue
            seq = self.live.get(entry["id"])
            if seq is None:
                seq = Sequence(list(tokens), block_size=self.block_size)
                if not self.cache.can_allocate(seq):
                    raise RuntimeError("no room for another request")
                self.cache.allocate(seq)
                self.live[entry["id"]] = seq
            else:
                for token in tokens:
                    seq.append_token(token)
                if not self.cache.can_append(seq):
                    raise RuntimeError("the cache pool is too small for the live requests")
                self.cache.append(seq)
            seq.num_scheduled_tokens = len(tokens)
            seqs.append(seq)
            wanted.append(entry["want"])
        logits = self.runner.step_logits(seqs, wanted) if seqs else None
        for seq in seqs:
            seq.num_computed_tokens += seq.num_scheduled_tokens
        for name in step.get("end", []):
            seq = self.live.pop(name, None)
            if seq is not None:
                self.cache.deallocate(seq)
        return logits


def replay(model_dir: str, dtype: str, out_dir: str, max_tokens: int, lines, emit) -> None:
    """Replay ``lines`` (JSON steps); logits go to ``out_dir``/<step>.f32, ``emit`` gets a line after every step."""
    block_size = 16
    engine = LLMEngine.from_pretrained(
        model_dir, dtype=dtype, block_size=block_size, max_cached_blocks=-(-max_tokens // block_size), max_num_sequences=4,
        max_position=max(max_tokens, 64), enforce_eager=True)
    trace = TraceReplay(engine)
    for line in lines:
        if not line.strip():
            continue
        step = json.loads(line)
        logits = trace.run_step(step)
        if logits is not None:
            path = os.path.join(out_dir, f"{step['step']}.f32")
            logits.cpu().numpy().astype("<f4").tofile(path)
        else:
            import torch
            torch.cuda.synchronize()                     # the step has run when its line says so
        emit(f"done {step['step']}")
