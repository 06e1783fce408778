"""Model designs by the ``architecture`` key of their configuration (absent: the Qwen3-style decoder).

An entry names the runner that serves the design, how a checkpoint's config.json turns into the engine's configuration,
and which kernel sources it runs on (for ``_build.ensure_library`` in a checkout without a built library)."""
from __future__ import annotations

import json
import os
from dataclasses import dataclass
from typing import Callable, Optional


@dataclass(frozen=True)
class Design:
    make_runner: Callable
    normalize: Callable = dict
    kernel_sources: Optional[Callable] = None      # (config) -> list of csrc files; None: the full library


def _qwen3_runner(config):
    from minivllm_amd.engine.model_runner import ModelRunner
    return ModelRunner(config)


def _sokevik_runner(config):
    from minivllm_amd.engine.hybrid_runner import HybridModelRunner
    from minivllm_amd.models.sokevik import SokevikForCausalLM
    return HybridModelRunner(config, SokevikForCausalLM)


def _sokevik_normalize(config):
    from minivllm_amd.models.sokevik import engine_config
    return engine_config(config)


def _sokevik_sources(config):
    from minivllm_amd.models.sokevik import kernel_sources
    return kernel_sources(config)


def _niridra_runner(config):
    from minivllm_amd.engine.hybrid_runner import HybridModelRunner
    from minivllm_amd.models.niridra import NiridraForCausalLM
    return HybridModelRunner(config, NiridraForCausalLM)


def _niridra_normalize(config):
    from minivllm_amd.models.niridra import engine_config
    return engine_config(config)


def _niridra_sources(config):
    from minivllm_amd.models.niridra import kernel_sources
    return kernel_sources(config)


def _fevosun_runner(config):
    from minivllm_amd.engine.hybrid_runner import HybridModelRunner
    from minivllm_amd.models.fevosun import FevosunForCausalLM
    return HybridModelRunner(config, FevosunForCausalLM)


def _fevosun_normalize(config):
    from minivllm_amd.models.fevosun import engine_config
    return engine_config(config)


def _fevosun_sources(config):
    from minivllm_amd.models.fevosun import kernel_sources
    return kernel_sources(config)


def _lenuzen_runner(config):
    from minivllm_amd.engine.hybrid_runner import HybridModelRunner
    from minivllm_amd.models.lenuzen import LenuzenForCausalLM
    return HybridModelRunner(config, LenuzenForCausalLM)


def _lenuzen_normalize(config):
    from minivllm_amd.models.lenuzen import engine_config
    return engine_config(config)


def _lenuzen_sources(config):
    from minivllm_amd.models.lenuzen import kernel_sources
    return kernel_sources(config)


DESIGNS = {"Qwen3": Design(_qwen3_runner), "Sokevik": Design(_sokevik_runner, _sokevik_normalize, _sokevik_sources),
           "Niridra": Design(_niridra_runner, _niridra_normalize, _niridra_sources),
           "Fevosun": Design(_fevosun_runner, _fevosun_normalize, _fevosun_sources),
           "Lenuzen": Design(_lenuzen_runner, _lenuzen_normalize, _lenuzen_sources)}


def design_of(config: dict) -> Design:
    name = config.get("architecture", "Qwen3")
    if name not in DESIGNS:
        raise ValueError(f"unknown architecture {name!r}; known: {', '.join(sorted(DESIGNS))}")
    return DESIGNS[name]


def read_model_config(model_dir: str) -> dict:
    with open(os.path.join(model_dir, "config.json")) as f:
        return json.load(f)


def make_runner(config: dict):
    design = design_of(config)
    return design.make_runner(design.normalize(config))
