"""Host side of the Lenuzen design: registry, configuration, what a checkpoint must hold, windows and chunks side by side in the
cache manager and in a step's metadata; and the oracle against itself."""
import math

import pytest
import torch
import torch.nn.functional as F

from minivllm_amd.engine.ragged import ragged_arrays, ragged_step
from minivllm_amd.engine.sequence import Sequence
from minivllm_amd.engine.windows import SlidingWindow
from minivllm_amd.layers.talk import talk_head_size
from minivllm_amd.models import registry
from minivllm_amd.models.lenuzen import LenuzenForCausalLM, engine_config
from lenuzen_cases import CONFIGS, YARN, config, dense, mixed_config, talk_layer, unit_layer
from oracle import lenuzen_oracle as ref
from sokevik_cases import manager, tokens

CPU = torch.device("cpu")


# ---- registry and configuration ----
def test_registry_has_the_design():
    assert registry.design_of({"architecture": "Lenuzen"}) is registry.DESIGNS["Lenuzen"]
    full = registry.DESIGNS["Lenuzen"].normalize(mixed_config())
    assert (full["vocab_size"], full["hidden_size"], full["num_layers"]) == (150, 80, 5)


def test_kernel_sources_follow_the_configuration():
    sources = registry.DESIGNS["Lenuzen"].kernel_sources
    one, other = set(sources(config([unit_layer()]))), set(sources(config([talk_layer()])))
    assert {"window_prefill_heads.hip", "window_decode_split.hip"} <= one - other and {"talk.hip", "talk_prefill.hip"} <= other - one
    assert set(sources(mixed_config())) == one | other


def build(cfg):
    return LenuzenForCausalLM(engine_config(cfg), 16, torch.float32, CPU)


def test_configurations_that_make_no_sense_are_refused():
    with pytest.raises(ValueError, match="mixer type"):
        build(config([{**unit_layer(), "type": "nothing"}]))
    with pytest.raises(ValueError, match="feed-forward"):
        build(config([unit_layer(mlp={"kind": "nothing"})]))
    with pytest.raises(ValueError, match="rotated dimensions"):
        build(config([talk_layer(dim=8, rot=10)]))
    with pytest.raises(ValueError, match="at most 64"):
        build(config([talk_layer(heads=66)]))
    with pytest.raises(ValueError, match="16384 columns"):
        build(config([talk_layer(heads=64, dim=264)]))


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
    assert seen == set(weights) and model.lm_head_weight is model.embedding
    drawn = {}
    model.load_weights = drawn.update
    model.reset_parameters()
    assert {k: tuple(t.shape) for k, t in drawn.items()} == {k: tuple(t.shape) for k, t in weights.items()}
    for lost in ("norm1", "mix.o"):
        with pytest.raises(KeyError):
            build(cfg).load_weights({k: t for k, t in weights.items() if not k.endswith(lost)})


def test_projections_are_filled_up():
    """Columns past the width, rows past the gates and a head's dims past its values are zeros."""
    cfg = mixed_config()
    model, w = build(cfg), ref.random_weights(cfg)
    model.load_weights(w)
    m = model.layer_stack[1].mixer                                         # 6 / 2 heads of 40 and 24
    rows = 6 * 40 + 2 * 40 + 2 * 24
    assert tuple(m.proj.weight.shape) == (384, 128) and m.gate_col == rows
    assert torch.equal(m.proj.weight[rows:rows + 6, :80], w["l1.mix.g"].float()) and not m.proj.weight[rows + 6:].any() and not m.proj.weight[:, 80:].any()
    assert torch.equal(m.proj.bias[240:320], w["l1.mix.k.b"].float()) and not m.proj.bias[rows:].any()
    out = m.out.weight.view(80, 6, 64)
    assert torch.equal(out[:, :, :24].flatten(1), w["l1.mix.o"].float()) and not out[:, :, 24:].any()
    assert torch.allclose(model.final_gain, w["final.norm"].float() * 0.7)


def test_caches_are_allocated_per_layer():
    model = build(mixed_config())
    model.allocate_state(12, 3)
    a, b = model.layer_stack[0].mixer, model.layer_stack[1].mixer
    assert tuple(a.k_cache.shape) == tuple(a.v_cache.shape) == (12, 16, 2, 64) and tuple(b.cache.shape) == (12, 16, 2, 128)
    assert model.windows == [20, 33, SlidingWindow(20), SlidingWindow(33), SlidingWindow(47)]     # a chunk and a window of one size are two
    assert [model.windows[l.mixer.window] for l in model.layer_stack] == [33, SlidingWindow(20), SlidingWindow(47), 20, SlidingWindow(33)]
    large = build(CONFIGS["large"]())
    assert [large.windows[l.mixer.window] for l in large.layer_stack] == [0, SlidingWindow(0), 80]


def test_sizes_that_kernels_step_in():
    assert [talk_head_size(n) for n in (1, 32, 33, 96, 97, 128, 130)] == [32, 32, 64, 96, 128, 128, 136] and talk_head_size(20, 70) == 96


# ---- cache manager and metadata ----
def test_windows_and_chunks_of_one_model():
    """A request holds a ring per window and a chunk per chunk size, and gives both back."""
    model = build(mixed_config())
    m = manager(model.windows, 30)
    s = Sequence([1] * 100, block_size=16)
    m.allocate(s)
    assert [len(t) for t in s.group_tables] == [2, 3, 4, 4, 5]
    m.deallocate(s)
    assert all(len(p.free_block_ids) == 30 for p in m.pools)


def test_rows_find_their_way_back():
    """Pieces are sorted by how they read their keys; the two maps between packed and sorted rows undo each other."""
    m = manager([20, SlidingWindow(20)], 30, slots=5)
    seqs = []
    for before, n in ((30, 50), (0, 1), (10, 5), (0, 45), (39, 3)):
        s = Sequence([1] * (before + n), block_size=16)
        m.allocate(s)
        s.num_computed_tokens, s.num_scheduled_tokens = before, n
        seqs.append(s)
    arrays, views, counts, facts = ragged_arrays(seqs, m.windows, 16)
    total, (dst, src) = facts["num_tokens"], (views[0][k] for k in ("dst_row", "src_row"))
    assert [int(dst[src[i]]) for i in range(total)] == list(range(total)) and not (dst == src).all()
    at = arrays["positions"][src]                                          # sorted: single rows, pieces behind a cached part, the others
    a, b = counts[0]["num_decode"], counts[0]["num_prefixed"]
    pieces = views[0]["prefixed_cu_q"]
    assert a == 1 and pieces.tolist() == [0, 5, 6, 16] and at[a:a + b].tolist() == [*range(10, 15), 39, *range(30, 40)]
    assert views[0]["fresh_cu"].tolist() == [0, 2, 22, 42, 62, 82, 87]
    step = ragged_step(seqs, m.windows, 16, CPU)
    assert step.windows[0].src_row.tolist() == src.tolist() and step.windows[1].num_long == 95


# ---- oracle against itself ----
def test_oracle_norms_and_gelu():
    g = torch.Generator().manual_seed(1)
    x, w = torch.randn(5, 40, generator=g, dtype=torch.float64) * 3 + 100, torch.randn(40, generator=g, dtype=torch.float64)
    assert torch.allclose(ref.centred_norm(x, w, 1e-3), F.layer_norm(x, (40,), w, None, 1e-3))
    assert torch.allclose(ref.unit(x, 0.0).pow(2).mean(-1), torch.ones(5, dtype=torch.float64))
    z = torch.linspace(-9, 9, 200, dtype=torch.float64)
    assert torch.allclose(ref.gelu_tanh(z), F.gelu(z, approximate="tanh"))


def test_oracle_masks():
    s, c = ref.sliding_mask(7, 3), ref.chunk_mask(7, 3)
    assert s.sum(1).tolist() == [1, 2, 3, 3, 3, 3, 3] and c.sum(1).tolist() == [1, 2, 3, 1, 2, 3, 1]
    assert s[4, 2] and not s[4, 1] and c[5, 3] and not c[5, 2] and not c[3, 4]
    assert torch.equal(ref.sliding_mask(6, 0), ref.chunk_mask(6, 0)) and ref.chunk_mask(6, 0).sum() == 21


def test_oracle_rotation():
    """A rotated product depends on the distance only; dims past the pairs stay; the ends of the YaRN blend."""
    g = torch.Generator().manual_seed(1)
    x, y = torch.randn(10, generator=g, dtype=torch.float64), torch.randn(10, generator=g, dtype=torch.float64)
    rot = {"base": 50.0, "dims": 8, "scaling": YARN}
    q, k = (ref.rotate(v.expand(40, 1, 10), rot)[:, 0] for v in (x, y))
    assert torch.allclose(q[7] @ k[3], q[29] @ k[25]) and not torch.allclose(q[7] @ k[3], q[8] @ k[3]) and torch.equal(q[11, 8:], x[8:])
    amplitude = 0.1 * math.log(YARN["factor"]) + 1
    assert torch.allclose(q[0, :8], x[:8] * amplitude)
    turned = ref.rotate(torch.tensor([1.0, 0.0, 0.0, 0.0], dtype=torch.float64).expand(2, 1, 4), {"base": 9.0, "dims": 4})[1, 0]
    assert torch.allclose(turned, torch.tensor([math.cos(1), math.sin(1), 0.0, 0.0], dtype=torch.float64))
    freq, _ = ref.pair_frequencies({"base": 1e6, "dims": 32, "scaling": {"factor": 8.0, "fast": 4.0, "slow": 1.0, "original": 1000}})
    assert math.isclose(freq[0], 1.0) and math.isclose(freq[-1], 1e6 ** (-15 / 16) / 8)


def test_oracle_sink_and_mixed_heads():
    """The sink takes weight and gives nothing; an identity mixes nothing, a permutation swaps heads."""
    s = torch.tensor([[[0.0, 0.0], [1.0, 2.0]]], dtype=torch.float64)
    p = ref.weights_of(s, ref.chunk_mask(2, 0), 0.0)
    assert torch.allclose(p[0, 0], torch.tensor([0.5, 0.0], dtype=torch.float64))
    assert torch.allclose(p[0, 1], torch.tensor([math.e, math.e ** 2], dtype=torch.float64) / (1 + math.e + math.e ** 2))
    two = torch.randn(2, 3, 3, dtype=torch.float64, generator=torch.Generator().manual_seed(2))
    assert torch.equal(ref.mix_heads(two, torch.eye(2, dtype=torch.float64)), two)
    assert torch.equal(ref.mix_heads(two, torch.tensor([[0.0, 1.0], [1.0, 0.0]], dtype=torch.float64)), two.flip(0))
    assert torch.equal(ref.mix_heads(two, torch.tensor([[0.0, 0.0], [3.0, 0.0]], dtype=torch.float64))[1], 3 * two[0])


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_oracle_runs_every_configuration(name):
    cfg = CONFIGS[name]()
    layers = []
    out = ref.forward(tokens(0, 60, cfg["vocab"]), ref.random_weights(cfg), cfg, layer_outputs=layers)
    assert out.shape == (60, cfg["vocab"]) and bool(out.isfinite().all()) and len(layers) == len(cfg["layers"])


def test_oracle_is_causal_and_local():
    """A token changes nothing before it, nothing a window behind it, and nothing in later chunks."""
    for layer, last in ((unit_layer(window=9), 38), (talk_layer(chunk=10), 39)):
        cfg = config([{**layer, "mlp": dense()}])
        w, toks = ref.random_weights(cfg), tokens(4, 60, cfg["vocab"])
        other = [*toks[:30], (toks[30] + 1) % cfg["vocab"], *toks[31:]]
        moved = (ref.forward(toks, w, cfg) - ref.forward(other, w, cfg)).abs().amax(-1) > 1e-9
        assert moved.nonzero()[:, 0].tolist() == list(range(30, last + 1))
