"""Host side of the Fevosun design: registry, configuration, what a checkpoint must hold, rings, metadata of windowed layers,
tables; and the oracle against itself."""
import math
import random

import numpy as np
import pytest
import torch

from minivllm_amd.engine.ragged import LONG_ROWS, ragged_arrays, ragged_step
from minivllm_amd.engine.sequence import Sequence
from minivllm_amd.engine.windows import SlidingWindow, places
from minivllm_amd.layers.basic import rotary_pair_table
from minivllm_amd.layers.mixers import distance_slopes
from minivllm_amd.layers.window import head_size, latent_layout, shared_part_size
from minivllm_amd.models import registry
from minivllm_amd.models.fevosun import FevosunForCausalLM, engine_config
from fevosun_cases import CONFIGS, YARN, attention_layer, config, dense, latent_layer, mixed_config, moe
from oracle import fevosun_oracle as ref
from sokevik_cases import manager, tokens

CPU = torch.device("cpu")


# ---- registry and configuration ----
def test_registry_has_the_design():
    assert registry.design_of({"architecture": "Fevosun"}) is registry.DESIGNS["Fevosun"]
    full = registry.DESIGNS["Fevosun"].normalize(mixed_config())
    assert (full["vocab_size"], full["hidden_size"], full["num_layers"]) == (150, 80, 5)


def test_kernel_sources_follow_the_configuration():
    sources = registry.DESIGNS["Fevosun"].kernel_sources
    only = sources(config([attention_layer(mlp=dense())]))
    assert "window_decode.hip" in only and "latent.hip" not in only and "moe.hip" not in only
    more = sources(config([latent_layer(mlp=moe())]))
    assert {"latent.hip", "window_prefill_latent.hip", "moe.hip", "gate_linear.hip"} <= set(more)


def build(cfg):
    return FevosunForCausalLM(engine_config(cfg), 16, torch.float32, CPU)


def test_configurations_that_make_no_sense_are_refused():
    with pytest.raises(ValueError, match="mixer type"):
        build(config([{**attention_layer(), "type": "nothing"}]))
    with pytest.raises(ValueError, match="feed-forward"):
        build(config([attention_layer(mlp={"kind": "nothing"})]))
    bad = attention_layer()
    bad["mixer"]["vdim"] = 8
    with pytest.raises(ValueError, match="values are keys"):
        build(config([bad]))
    bad = latent_layer(rot_dim=8)
    bad["mixer"]["rot"]["dims"] = 10
    with pytest.raises(ValueError, match="rotated dimensions"):
        build(config([bad]))


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
        build(cfg).load_weights({k: t for k, t in weights.items() if not k.endswith("norm1")})


def test_caches_are_allocated_per_layer():
    model = build(mixed_config())
    model.allocate_state(12, 3)
    shapes = [tuple(l.mixer.cache.shape) for l in model.layer_stack]
    assert shapes[0] == (12, 16, 1, 128) and shapes[1] == (12, 16, 2, 64) and shapes[3] == (12, 16, 4, 32)
    assert [w.size for w in model.windows] == [5, 20, 33, 47]
    assert [l.mixer.view.size for l in model.layer_stack] == [33, 20, 20, 47, 5]
    assert all(model.windows[l.mixer.window] is l.mixer.view or model.windows[l.mixer.window] == l.mixer.view for l in model.layer_stack)


def test_sizes_that_kernels_step_in():
    assert [head_size(n) for n in (1, 32, 33, 96, 97, 200, 256, 257)] == [32, 32, 64, 96, 128, 256, 256, 288]
    assert [shared_part_size(n) for n in (2, 32, 34, 64, 66)] == [32, 32, 64, 64, 96]
    assert latent_layout(80, 10) == (80, 128, 128) and latent_layout(512, 64) == (512, 576, 512) and latent_layout(500, 64) == (512, 576, 512)
    assert latent_layout(150, 20) == (160, 192, 192) and latent_layout(600, 64) == (608, 672, 672)
    with pytest.raises(ValueError):
        head_size(600)
    with pytest.raises(ValueError):
        latent_layout(2040, 8)


# ---- rings ----
def test_rings_hold_a_window_and_the_rows_of_a_short_entry():
    w = SlidingWindow(20)
    assert w.places == 20 + LONG_ROWS - 2 and places(w) == w.places and places(7) == 7 and SlidingWindow().places == 0
    m = manager([w, SlidingWindow(), 20], 30)
    assert [m.blocks_for(x, 1000) for x in m.windows] == [4, 63, 2] and [m.blocks_for(x, 17) for x in m.windows] == [2, 2, 2]
    s = Sequence([1] * 100, block_size=16)
    m.allocate(s)
    assert [len(t) for t in s.group_tables] == [4, 7, 2]
    for _ in range(40):
        s.append_token(2)
    m.append(s)
    assert [len(t) for t in s.group_tables] == [4, 9, 2]
    m.deallocate(s)
    assert all(len(p.free_block_ids) == 30 for p in m.pools)


@pytest.mark.parametrize("seed", range(12))
@pytest.mark.parametrize("size", [0, 1, 5, 40, 64])
def test_ring_arrays_against_token_by_token(seed, size):
    """A simulated cache of token numbers: what a row may read is there when it reads it, in both forms."""
    rng, bs, window = random.Random(100 * size + seed), 16, SlidingWindow(size)
    m = manager([window], 60, bs, 6)
    cache = np.full(60 * bs, -1)                                           # (sequence, position) of every slot
    seqs = [Sequence([1], block_size=bs) for _ in range(4)]
    for s in seqs:
        m.allocate(s)
    done = [0] * 4
    for _ in range(14):
        chosen = [i for i in range(4) if rng.random() < 0.8] or [0]
        for i in chosen:
            n = rng.choice([1, 1, 2, 3, LONG_ROWS - 1, LONG_ROWS, 40])
            while len(seqs[i]) < done[i] + n:
                seqs[i].append_token(1)
            m.append(seqs[i])
            seqs[i].num_computed_tokens, seqs[i].num_scheduled_tokens = done[i], n
        step = [seqs[i] for i in chosen]
        arrays, (view,), (counts,), facts = ragged_arrays(step, [window], bs)
        packed = [step[i] for i in facts["order"]]
        name = lambda s, p: 10000 * seqs.index(s) + p
        keys = np.full(counts["num_keys"], -1)
        if "past_slots" in view:
            keys[view["past_rows"]] = cache[view["past_slots"]]
        written = set()
        for e, s in enumerate(packed):
            lo, p0 = int(arrays["cu_seqlens"][e]), s.num_computed_tokens
            for j in range(s.num_scheduled_tokens):
                slot = view["slots"][lo + j]
                if slot >= 0:
                    assert slot not in written                           # no two rows of a step go to one place
                    written.add(slot)
                    cache[slot] = name(s, p0 + j)
                if "key_rows" in view and view["key_rows"][lo + j] >= 0:
                    keys[view["key_rows"][lo + j]] = name(s, p0 + j)
        long_ = 0
        for e, s in enumerate(packed):
            lo, p0, n = int(arrays["cu_seqlens"][e]), s.num_computed_tokens, s.num_scheduled_tokens
            for j in range(n):
                sees = [name(s, q) for q in range(max(0, p0 + j - size + 1) if size else 0, p0 + j + 1)]
                if lo + j < counts["absorbed"]:
                    assert n < LONG_ROWS and view["lens"][lo + j] == p0 + j + 1
                    table, found = view["tables"][e], []
                    ring = window.places
                    for at in range(min(p0 + j + 1, ring) if ring else p0 + j + 1):
                        away = (p0 + j) % ring - at if ring else p0 + j - at
                        away += ring if away < 0 else 0
                        if not size or away < size:
                            found.append(cache[table[at // bs] * bs + at % bs])
                            assert found[-1] == name(s, p0 + j - away)
                    assert sorted(found) == sees
                else:
                    first, last = view["cu_k"][long_], view["cu_k"][long_ + 1]
                    own = last - n + j
                    assert keys[max(first, own - size + 1) if size else first:own + 1].tolist() == sees
            if n >= LONG_ROWS:
                assert view["cu_q"][long_ + 1] - view["cu_q"][long_] == n
                long_ += 1
        assert counts["num_long"] == sum(s.num_scheduled_tokens for s in packed if s.num_scheduled_tokens >= LONG_ROWS)
        for i in chosen:
            done[i] += seqs[i].num_scheduled_tokens


def test_ring_step_on_the_device():
    m = manager([SlidingWindow(10), SlidingWindow(50)], 20)
    s = Sequence(list(range(80)), block_size=16)
    m.allocate(s)
    s.num_computed_tokens, s.num_scheduled_tokens = 41, 39
    a, b = ragged_step([s], m.windows, 16, CPU).windows
    assert (a.absorbed, a.num_long, a.num_keys, b.num_keys) == (0, 39, 48, 80) and a.past_slots.numel() == 9 and b.past_rows.tolist() == list(range(41))
    assert a.lens is None and a.cu_k.tolist() == [0, 48] and a.slots.dtype == torch.int64 and a.key_rows.tolist() == list(range(9, 48))


# ---- tables ----
@pytest.mark.parametrize("dims,base,scaling", [(20, 700.0, YARN), (6, 1e4, None), (64, 5e5, {"factor": 8.0, "fast": 32.0, "slow": 1.0, "original": 100}),
                                               (2, 10.0, YARN), (12, 50.0, {"factor": 2.0, "fast": 1.0, "slow": 1.0, "original": 7})])
def test_rotary_tables(dims, base, scaling):
    cos, sin = ref.rotation({"base": base, "dims": dims, "scaling": scaling}, 200)
    table = rotary_pair_table(base, dims, 200, scaling)
    assert torch.allclose(table[..., 0].double(), cos, atol=1e-6) and torch.allclose(table[..., 1].double(), sin, atol=1e-6)


def test_distance_slopes():
    assert torch.allclose(distance_slopes(8), torch.tensor([2.0 ** -(i + 1) for i in range(8)]))
    assert torch.allclose(distance_slopes(6).double(), ref.distance_slopes(6), rtol=1e-6)


# ---- oracle against itself ----
def test_oracle_rotation_keeps_distances():
    """A rotated product depends on the distance only, in both layouts; other dims stay."""
    g = torch.Generator().manual_seed(1)
    x, y = torch.randn(10, generator=g, dtype=torch.float64), torch.randn(10, generator=g, dtype=torch.float64)
    for interleaved in (False, True):
        cos, sin = ref.rotation({"base": 50.0, "dims": 8}, 40)
        q, k = (ref.rotate(v.expand(40, 10), cos, sin, interleaved) for v in (x, y))
        assert torch.allclose(q[7] @ k[3], q[29] @ k[25]) and not torch.allclose(q[7] @ k[3], q[8] @ k[3])
        assert torch.equal(q[11, 8:], x[8:])
    a, b = (ref.rotate(torch.eye(4, dtype=torch.float64)[:1].expand(3, 4), *ref.rotation({"base": 9.0, "dims": 4}, 3), i) for i in (False, True))
    assert a[2, 2] != 0 and a[2, 1] == 0 and b[2, 1] != 0 and b[2, 2] == 0


def test_oracle_yarn_ends():
    """Fast pairs keep their frequency, slow ones are divided by the factor."""
    s = {"factor": 8.0, "fast": 4.0, "slow": 1.0, "original": 1000}
    cos, sin = ref.rotation({"base": 1e6, "dims": 32, "scaling": s}, 2)
    amplitude, freq = 0.1 * math.log(8.0) + 1, torch.atan2(sin[1], cos[1])
    plain = torch.tensor([1e6 ** (-i / 16) for i in range(16)], dtype=torch.float64)
    assert torch.allclose(cos[0], torch.full((16,), amplitude, dtype=torch.float64))
    assert torch.allclose(freq[0], plain[0]) and torch.allclose(freq[-1], plain[-1] / 8)


def test_oracle_window_and_temperature():
    m = ref.window_mask(5, 2)
    assert m.sum(1).tolist() == [1, 2, 2, 2, 2] and m[3, 2] and not m[3, 1] and ref.window_mask(4, 0).sum() == 10
    t = ref.query_temperature(range(9), 0.5, 4)
    assert torch.allclose(t, torch.tensor([1.0] * 3 + [1 + 0.5 * math.log(2)] * 4 + [1 + 0.5 * math.log(3)] * 2, dtype=torch.float64))


def test_oracle_router_and_clamped_expert():
    """The correction chooses but does not weigh; identity experts hand the input on."""
    z, correction = torch.tensor([2.0, 1.0, 0.0, -1.0]), torch.tensor([-1.0, 0.0, 0.0, 0.9])
    ids, w = ref.route(z, correction, 2)
    assert ids == [3, 1] and torch.allclose(w, torch.softmax(z, -1)[[3, 1]])
    one = {"gate": torch.tensor([[5.0]]), "up": torch.tensor([[-5.0]]), "down": torch.tensor([[1.0]])}
    got = ref.clamped_expert(torch.tensor([1.0]), one, "", 0.5)
    assert torch.allclose(got, torch.tensor([0.5 / (1 + math.exp(-1.702 * 0.5)) * 0.5]))
    low = ref.clamped_expert(torch.tensor([-1.0]), one, "", 0.5)                    # a gate has no lower bound
    assert torch.allclose(low, torch.tensor([-5.0 / (1 + math.exp(1.702 * 5.0)) * 1.5]))
    w = {"router": torch.tensor([[0.0], [9.0]]), "correction": torch.zeros(2), "e0.gate": torch.ones(1, 1), "e0.up": torch.ones(1, 1), "e0.down": torch.ones(1, 1)}
    cfg = {"router": {"experts": 1, "identity": 1, "top": 1}, "expert": {"ff": 1, "limit": 1.0}}
    assert torch.allclose(ref.experts(torch.tensor([[2.0]]), w, "", cfg), torch.tensor([[2.0]]) * torch.softmax(torch.tensor([0.0, 18.0]), -1)[1])


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_oracle_runs_every_configuration(name):
    cfg = CONFIGS[name]()
    layers = []
    out = ref.forward(tokens(0, 60, cfg["vocab"]), ref.random_weights(cfg), cfg, layer_outputs=layers)
    assert out.shape == (60, cfg["vocab"]) and bool(out.isfinite().all()) and len(layers) == len(cfg["layers"])
