"""Command line: ``python -m minivllm_amd generate`` runs prompts of token ids through a checkpoint folder,
``python -m minivllm_amd replay`` replays a step trace from standard input (also installed as ``bin/trace_run``)."""
from __future__ import annotations

import argparse
import json
import os
import sys


def _add_model(parser):
    parser.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    parser.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")


def _ensure_kernels(model_dir):
    """Kernels for this model, compiled if the checkout has no library yet."""
    from minivllm_amd import _build
    from minivllm_amd.models.registry import design_of, read_model_config
    config = read_model_config(model_dir)
    sources = design_of(config).kernel_sources
    _build.ensure_library(sources(config) if sources else _build.SOURCES)


def _replay(args):
    _ensure_kernels(args.model)
    os.makedirs(args.out, exist_ok=True)
    from minivllm_amd.engine.replay import replay
    replay(args.model, args.dtype, args.out, args.max_tokens, sys.stdin, lambda text: print(text, flush=True))


def _generate(args):
    from minivllm_amd import _build
    if not os.path.exists(_build.LIB_PATH):
        _build.build_library(verbose=False)
    from minivllm_amd.engine.llm_engine import LLMEngine
    from minivllm_amd.sampling_parameters import SamplingParams
    prompts = [[int(t) for t in p.replace(",", " ").split()] for p in args.prompt]
    params = SamplingParams(temperature=args.temperature, max_tokens=args.max_tokens, ignore_eos=args.eos is None,
                            greedy=args.greedy)
    longest = max(len(p) for p in prompts) + args.max_tokens
    engine = LLMEngine.from_pretrained(
        args.model, dtype=args.dtype, block_size=args.block_size, max_num_sequences=args.max_num_sequences,
        max_cached_blocks=args.max_num_sequences * -(-longest // args.block_size), max_position=longest,
        max_num_batched_tokens=args.max_num_batched_tokens, enforce_eager=args.enforce_eager, seed=args.seed,
        eos=-1 if args.eos is None else args.eos)
    print(json.dumps(engine.generate(prompts, params)))


def main(argv=None):
    parser = argparse.ArgumentParser(prog="minivllm_amd", description=__doc__)
    sub = parser.add_subparsers(dest="command", required=True)
    gen = sub.add_parser("generate", help="generate from prompts of token ids")
    _add_model(gen)
    gen.add_argument("--prompt", action="append", required=True, help="token ids with commas or spaces (repeatable)")
    gen.add_argument("--max-tokens", type=int, default=64, help="new tokens per prompt")
    gen.add_argument("--temperature", type=float, default=1.0)
    gen.add_argument("--greedy", action="store_true")
    gen.add_argument("--eos", type=int, default=None)
    gen.add_argument("--seed", type=int, default=0)
    gen.add_argument("--block-size", type=int, default=16)
    gen.add_argument("--max-num-sequences", type=int, default=16)
    gen.add_argument("--max-num-batched-tokens", type=int, default=8192)
    gen.add_argument("--enforce-eager", action="store_true", help="no captured decode graphs")
    gen.set_defaults(run=_generate)
    rep = sub.add_parser("replay", help="replay a step trace from standard input")
    _add_model(rep)
    rep.add_argument("--out", required=True, help="folder for <step>.f32")
    rep.add_argument("--max-tokens", type=int, required=True, help="the most tokens live requests hold at any time")
    rep.set_defaults(run=_replay)
    args = parser.parse_args(argv)
    args.run(args)


if __name__ == "__main__":
    main()
