"""Host side of the Niridra design: registry, configuration, what a checkpoint must hold, metadata of latent layers, padding,
scheduling; and the oracle against itself."""
import random

import numpy as np
import pytest
import torch

from minivllm_amd.engine.ragged import LONG_ROWS, ragged_arrays, ragged_step
from minivllm_amd.engine.sequence import Sequence
from minivllm_amd.layers.experts import SparseExperts, interleave_gate_up
from minivllm_amd.layers.latent import latent_width
from minivllm_amd.layers.recurrent import DecayMemoryState
from minivllm_amd.models import registry
from minivllm_amd.models.niridra import NiridraForCausalLM, engine_config
from minivllm_amd.utils.padding import pad_heads, pad_to
from niridra_cases import CONFIGS, config, latent_layer, lightning_layer, mixed_config, moe
from oracle import niridra_oracle as ref
from sokevik_cases import manager, tokens

CPU = torch.device("cpu")


# ---- registry and configuration ----
def test_registry_has_the_design():
    assert registry.design_of({"architecture": "Niridra"}) is registry.DESIGNS["Niridra"]
    full = registry.DESIGNS["Niridra"].normalize(mixed_config())
    assert (full["vocab_size"], full["hidden_size"], full["num_layers"]) == (150, 80, 6)


def test_kernel_sources_follow_the_configuration():
    sources = registry.DESIGNS["Niridra"].kernel_sources
    only_memory = sources(config([lightning_layer()]))
    assert "decay_memory.hip" in only_memory and "latent.hip" not in only_memory and "moe.hip" not in only_memory
    only_latent = sources(config([latent_layer(dim=64, vdim=64, mlp=moe())]))
    assert "latent.hip" in only_latent and "moe.hip" in only_latent and "decay_memory.hip" not in only_latent
    assert "prefill_other_dims.hip" not in only_latent and "prefill_other_dims.hip" in sources(config([latent_layer(dim=96)]))


def build(cfg):
    return NiridraForCausalLM(engine_config(cfg), 16, torch.float32, CPU)


def test_configurations_that_make_no_sense_are_refused():
    for bad in (latent_layer(kv_from=1), latent_layer(kv_from=0), latent_layer(kv_from=7)):       # itself; no latents; nothing
        with pytest.raises(ValueError, match="kv_from"):
            build(config([lightning_layer(), bad]))
    with pytest.raises(ValueError, match="kv_from"):                                              # latents of another rank
        build(config([latent_layer(rank=72), latent_layer(rank=40, kv_from=0)]))
    with pytest.raises(ValueError, match="kv_from"):                                              # a layer that reads another's
        build(config([latent_layer(), latent_layer(kv_from=0), latent_layer(kv_from=1)]))
    with pytest.raises(ValueError, match="decays"):
        build(config([lightning_layer(heads=3, decay=[0.5, 0.5])]))
    with pytest.raises(ValueError, match="mixer type"):
        build(config([{**lightning_layer(), "type": "nothing"}]))
    with pytest.raises(ValueError, match="feed-forward"):
        build(config([lightning_layer(mlp={**moe(), "kind": "dense"})]))


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_checkpoint_names_and_shapes(name):
    """Every tensor of a checkpoint finds its place, and the model's own random weights are a checkpoint of the same names."""
    cfg = CONFIGS[name]()
    weights = ref.random_weights(cfg)
    seen = set()

    class Watched(dict):
        def __getitem__(self, key):
            seen.add(key)
            return super().__getitem__(key)

    model = build(cfg)
    model.load_weights(Watched(weights))
    assert seen == set(weights)
    drawn = {}
    model.load_weights = drawn.update
    model.reset_parameters()
    assert {k: tuple(t.shape) for k, t in drawn.items()} == {k: tuple(t.shape) for k, t in weights.items()}
    with pytest.raises(KeyError):
        build(cfg).load_weights({k: t for k, t in weights.items() if not k.endswith("hc1.mix")})


def test_states_are_allocated_per_layer():
    model = build(mixed_config())
    model.allocate_state(12, 3)
    caches = [l.mixer.cache.shape for l in model.layer_stack if l.is_attention]
    assert caches[0] == (12, 16, latent_width(72)) and caches[2] == (12, 16, latent_width(40))
    assert caches[1] == caches[3] == (0,)                                     # they read layer 1's
    assert model.layer_stack[0].mixer.state.s.shape == (3, 3, 24, 40) and model.layer_stack[0].mixer.state.s.dtype == torch.float32
    assert model.prev_tokens.shape == (7,) and model.windows == [0]
    assert build(config([lightning_layer()])).windows == []


def test_decays_at_the_ends():
    s = DecayMemoryState.allocate(1, [0.0, 1.0, 0.5], 4, 4, CPU)
    assert s.log_decay.exp().tolist() == [0.0, 1.0, 0.5] and s.decay.tolist() == [0.0, 1.0, 0.5]
    for bad in (1.5, -0.1, float("nan")):
        with pytest.raises(ValueError, match="between"):
            DecayMemoryState.allocate(1, [bad], 4, 4, CPU)


# ---- padding ----
def test_padding():
    t = torch.arange(12.0).view(4, 3)
    p = pad_heads(t, 2, 5, 4)
    assert p.shape == (10, 4) and torch.equal(p[:2, :3], t[:2]) and torch.equal(p[5:7, :3], t[2:]) and p.sum() == t.sum()
    assert torch.equal(pad_to(t, None, None), t) and pad_to(t, 6, 8).shape == (6, 8) and pad_to(t, 6, 8).sum() == t.sum()
    gate, up = torch.arange(64.0).view(64, 1), -torch.arange(64.0).view(64, 1)
    both = interleave_gate_up(gate, up)[:, 0]
    assert both[:32].tolist() == list(range(32)) and both[32:64].tolist() == [-float(i) for i in range(32)] and both[64] == 32
    assert latent_width(1) == 32 and latent_width(96) == 96 and latent_width(97) == 128 and latent_width(513) == 544
    with pytest.raises(ValueError):
        latent_width(2049)


def test_padded_experts_are_the_experts():
    """Sizes filled up with zeros change nothing."""
    cfg = moe(experts=4, ff=40, shared=30)
    w = {k[len("l0.mlp."):]: t.float() for k, t in ref.random_weights(config([lightning_layer(mlp=cfg)])).items() if k.startswith("l0.mlp.")}
    m = SparseExperts(80, 128, 4, 3, 40, 2, 1, 30)
    m.load(lambda n: w[n], lambda t: t.contiguous())
    h = torch.randn(5, 80)
    padded = torch.nn.functional.pad(h, (0, 48))
    z = (padded @ m.gate_up[2].T).view(5, -1, 2, 32)
    got = (torch.nn.functional.silu(z[:, :, 0]) * z[:, :, 1]).reshape(5, -1) @ m.down[2].T
    assert torch.allclose(got[:, :80], ref.expert(h, w, "e2."), atol=1e-5) and not got[:, 80:].any()
    assert torch.allclose(padded @ m.router.T, torch.cat([h @ w["router"].T, h @ w["shared.sg"].T], 1), atol=1e-5)


# ---- metadata of layers that cache latents ----
@pytest.mark.parametrize("seed", range(12))
def test_latent_arrays_against_row_by_row(seed):
    rng, bs = random.Random(seed), 16
    m = manager([0], 400, bs, 8)
    seqs = []
    for _ in range(rng.randint(1, 7)):
        total = rng.randint(1, 150)
        s = Sequence(tokens(seed, total, 99), block_size=bs)
        m.allocate(s)
        s.num_scheduled_tokens = min(rng.choice([1, 1, 2, 3, LONG_ROWS - 1, LONG_ROWS, 40, total]), total)
        s.num_computed_tokens = total - s.num_scheduled_tokens
        seqs.append(s)
    arrays, (view,), (counts,), facts = ragged_arrays(seqs, [0], bs, latent=True)
    packed = [seqs[i] for i in facts["order"]]
    kind = lambda s: 0 if s.num_scheduled_tokens < LONG_ROWS else 1 if s.num_computed_tokens else 2
    assert [kind(s) for s in packed] == sorted(kind(s) for s in packed)
    total = facts["num_tokens"]
    a, b = counts["absorbed"], counts["absorbed"] + counts["num_prefixed"]
    assert b + counts["num_fresh"] == total == len(view["slots"])
    pre = fresh = 0
    for e, s in enumerate(packed):
        lo, p0, n, table = int(arrays["cu_seqlens"][e]), s.num_computed_tokens, s.num_scheduled_tokens, s.group_tables[0]
        for j in range(n):
            assert view["slots"][lo + j] == table[(p0 + j) // bs] * bs + (p0 + j) % bs
        assert view["tables"][e][:len(table)].tolist() == table and (view["tables"][e][len(table):] == -1).all()
        if kind(s) == 0:
            assert lo + n <= a and view["lens"][lo:lo + n].tolist() == list(range(p0 + 1, p0 + n + 1))
        elif kind(s) == 1:
            assert view["prefixed_cu_q"][pre] == lo - a and view["prefixed_cu_q"][pre + 1] == lo - a + n
            assert view["prefixed_cu_k"][pre + 1] - view["prefixed_cu_k"][pre] == p0 + n <= counts["prefixed_max_k"]
            used = -(-(p0 + n) // bs)
            assert view["gather"][view["scratch_tables"][pre][:used]].tolist() == table[:used]
            pre += 1
        else:
            assert view["fresh_cu"][fresh] == lo - b and view["fresh_cu"][fresh + 1] == lo - b + n
            fresh += 1
    assert ("gather" in view) == (pre > 0) and ("fresh_cu" in view) == (fresh > 0) and ("lens" in view) == (a > 0)


def test_latent_step_on_the_device():
    m = manager([0], 20)
    s = Sequence(list(range(50)), block_size=16)
    m.allocate(s)
    s.num_computed_tokens, s.num_scheduled_tokens = 13, 37
    step = ragged_step([s], [0], 16, CPU, latent=True)
    v = step.windows[0]
    assert (v.absorbed, v.num_prefixed, v.num_fresh, v.prefixed_max_k) == (0, 37, 0, 50) and v.gather.tolist() == s.group_tables[0]
    assert v.slots.dtype == torch.int64 and v.tables.dtype == torch.int32 and step.scratch == {}


# ---- oracle against itself ----
def test_oracle_memory_has_the_closed_form():
    g = torch.Generator().manual_seed(3)
    q, k, v = (torch.randn(9, 2, n, generator=g, dtype=torch.float64) for n in (4, 4, 5))
    decay = torch.tensor([0.3, 0.95], dtype=torch.float64)
    got = ref.decaying_memory(q, k, v, decay)
    for h in range(2):
        for t in range(9):
            want = sum(decay[h] ** (t - s) * (k[s, h] @ q[t, h]) * v[s, h] for s in range(t + 1))
            assert torch.allclose(got[t, h], want, atol=1e-12)


def test_oracle_latents_answer_absorbed_queries():
    """q . (U_k c) = (U_k^T q) . c, and the same for the values."""
    g = torch.Generator().manual_seed(4)
    cfg = latent_layer(heads=2, dim=6, vdim=5, rank=7)["mixer"]
    w = {k: torch.randn(s, generator=g, dtype=torch.float64) for k, s in
         {"q": (12, 9), "uk": (12, 7), "uv": (10, 7), "o": (9, 10)}.items()}
    h, c = torch.randn(8, 9, generator=g, dtype=torch.float64), torch.randn(8, 7, generator=g, dtype=torch.float64)
    want = ref.latent_attention(h, c, w, "", cfg)
    outs = []
    for head in range(2):
        qc = (h @ w["q"].T)[:, 6 * head:6 * head + 6] @ w["uk"][6 * head:6 * head + 6]
        p = torch.softmax((qc @ c.T * cfg["scale"]).masked_fill(~torch.ones(8, 8).tril().bool(), float("-inf")), -1)
        outs.append(p @ c @ w["uv"][5 * head:5 * head + 5].T)
    assert torch.allclose(torch.cat(outs, 1) @ w["o"].T, want, atol=1e-12)


def test_oracle_router():
    """Groups by the sum of their two largest choice scores; negative choice scores stay below what is closed; weights
    without the correction."""
    z = torch.tensor([4.0, -4.0, 0.5, 0.4, -1.0, -1.0])
    correction = torch.tensor([-1.0, -1.0, -1.0, -1.0, 0.9, -3.0])
    s = torch.sigmoid(z)
    ids, weights = ref.route(z, correction, {"experts": 6, "top": 2, "groups": {"count": 3, "keep": 1}})
    assert ids == [2, 3]                                  # sums of the groups: -1.0, -0.78, -1.56
    assert torch.allclose(weights, s[[2, 3]] / s[[2, 3]].sum())
    ids, _ = ref.route(z, correction, {"experts": 6, "top": 3, "groups": None})
    assert ids == [4, 0, 2]


def test_oracle_first_token_has_a_row_of_its_own():
    assert ref.bigram_rows([5, 5, 2], 37, 5, 3) == [37, (25 + 15) % 37, (25 + 6) % 37]


def test_oracle_streams_update_at_once():
    w = {"hc1.in": torch.tensor([1.0, 0.0]), "hc1.out": torch.tensor([0.0, 0.0]), "hc1.mix": torch.tensor([[0.0, 1.0], [1.0, 0.0]]),
         "norm1": torch.ones(3), "ls1": torch.ones(3)}
    xs = torch.stack([torch.ones(2, 3), torch.full((2, 3), 5.0)])
    assert torch.equal(ref.hyper_sublayer(xs, w, "", 1, lambda h: h, 1e-6), xs.flip(0))       # the streams trade places


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_oracle_runs_every_configuration(name):
    cfg = CONFIGS[name]()
    layers = []
    out = ref.forward(tokens(0, 30, cfg["vocab"]), ref.random_weights(cfg), cfg, layer_outputs=layers)
    assert out.shape == (30, cfg["vocab"]) and bool(out.isfinite().all()) and len(layers) == len(cfg["layers"])
