"""Host side of the ragged-step engine and the Sokevik design: configuration, checkpoint reader, rotary tables, cache
manager, step metadata, scheduler; and the oracle against itself."""
import json
import random

import numpy as np
import pytest
import torch

from minivllm_amd.engine.ragged import LONG_ROWS, ragged_arrays, ragged_step
from minivllm_amd.engine.scheduler import Scheduler
from minivllm_amd.engine.sequence import Sequence
from minivllm_amd.layers.basic import rotary_pair_table
from minivllm_amd.layers.mixers import attention_head_dim
from minivllm_amd.models import registry
from minivllm_amd.sampling_parameters import SamplingParams
from minivllm_amd.utils.safetensors_io import read_safetensors
from oracle import sokevik_oracle as ref
from sokevik_cases import CONFIGS, attention_layer, config, manager, mlstm_layer, shared, tokens


# ---- configuration, registry, checkpoint ----
def test_registry_chooses_by_architecture():
    assert registry.design_of({}) is registry.DESIGNS["Qwen3"]
    assert registry.design_of({"architecture": "Sokevik"}) is registry.DESIGNS["Sokevik"]
    with pytest.raises(ValueError, match="unknown architecture"):
        registry.design_of({"architecture": "Nobody"})


def test_kernel_sources_follow_the_configuration():
    sources = registry.DESIGNS["Sokevik"].kernel_sources
    only_memory = sources(config([mlstm_layer()]))
    assert "mlstm.hip" in only_memory and "paged_decode.hip" not in only_memory
    only_attention = sources(config([attention_layer(dim=64, vdim=64, rot=64)]))
    assert "mlstm.hip" not in only_attention and "prefill_other_dims.hip" not in only_attention
    assert "prefill_other_dims.hip" in sources(config([attention_layer(dim=96, vdim=64)]))
    assert not any("pingpong" in s for s in only_attention + only_memory)


def test_weights_of_is_followed_and_circles_are_refused():
    from minivllm_amd.models.sokevik import _owner
    a = attention_layer()
    layers = [a, mlstm_layer(), shared(a, 0), shared(a, 2)]
    assert [_owner(layers, i) for i in range(4)] == [0, 1, 0, 0]
    with pytest.raises(ValueError, match="circle"):
        _owner([shared(a, 1), shared(a, 0)], 0)


def test_attention_head_dim_covers_both_sizes():
    for dim, vdim in [(48, 64), (64, 48), (8, 8), (100, 20), (130, 20), (300, 20), (17, 3)]:
        for dtype in (torch.bfloat16, torch.float32):
            d = attention_head_dim(dim, vdim, dtype)
            assert d >= max(dim, vdim) and d % 8 == 0
    assert attention_head_dim(64, 64, torch.bfloat16) == 64 and attention_head_dim(48, 16, torch.float32) == 64


def test_safetensors_reader(tmp_path):
    want = {"a": torch.randn(3, 5).bfloat16(), "b": torch.randn(7), "c": torch.arange(6, dtype=torch.int32).view(2, 3),
            "scalar": torch.tensor(2.5).bfloat16(), "none": torch.empty(0, 4)}
    names = {torch.bfloat16: "BF16", torch.float32: "F32", torch.int32: "I32"}
    header, blobs, at = {"__metadata__": {"x": "y"}}, [], 0
    for name, t in want.items():
        raw = t.contiguous().view(torch.uint8 if t.numel() and t.dim() else t.dtype).numpy().tobytes() if t.dtype != torch.bfloat16 \
            else t.view(torch.int16).numpy().tobytes()
        header[name] = {"dtype": names[t.dtype], "shape": list(t.shape), "data_offsets": [at, at + len(raw)]}
        blobs.append(raw)
        at += len(raw)
    text = json.dumps(header).encode()
    path = tmp_path / "x.safetensors"
    path.write_bytes(len(text).to_bytes(8, "little") + text + b"".join(blobs))
    got = read_safetensors(str(path))
    assert set(got) == set(want)
    for name, t in want.items():
        assert got[name].dtype == t.dtype and got[name].shape == t.shape and torch.equal(got[name], t), name
    header["b"]["shape"] = [8]
    text = json.dumps(header).encode()
    path.write_bytes(len(text).to_bytes(8, "little") + text + b"".join(blobs))
    with pytest.raises(ValueError):
        read_safetensors(str(path))


def test_greedy_sampling_parameters():
    assert SamplingParams(greedy=True).temperature < 1e-6
    assert SamplingParams().temperature == 1.0


# ---- rotary tables ----
@pytest.mark.parametrize("scaling", [None, {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 100},
                                     {"factor": 2.0, "low": 0.5, "high": 3.0, "original": 30}])
def test_rotary_pair_table(scaling):
    table = rotary_pair_table(300.0, 24, 50, scaling)
    f = ref.pair_frequencies(24, 300.0, scaling)
    ang = torch.arange(50, dtype=torch.float64)[:, None] * f
    assert torch.allclose(table[..., 0].double(), ang.cos(), atol=1e-7) and torch.allclose(table[..., 1].double(), ang.sin(), atol=1e-7)
    if scaling:                       # all three branches are met: kept, divided, blended
        plain = ref.pair_frequencies(24, 300.0)
        ratio = plain / f
        assert (ratio == 1).any() and (abs(ratio - scaling["factor"]) < 1e-9).any()
        assert ((ratio > 1.001) & (ratio < scaling["factor"] - 0.001)).any()


# ---- oracle against itself ----
def test_oracle_values_turned_back_depend_on_distance_only():
    """Rotating values by their positions and the result back by the query's: a shift of all positions changes nothing."""
    v = torch.randn(9, 2, 12, dtype=torch.float64)
    f = ref.pair_frequencies(12, 100.0)
    pos = torch.arange(9)
    w = torch.rand(9, 9, dtype=torch.float64).tril()

    def run(p):
        return ref.rotate_pairs(torch.einsum("ij,jhd->ihd", w, ref.rotate_pairs(v, p, f)), p, f, -1.0)
    assert torch.allclose(run(pos), run(pos + 31), atol=1e-9)


def test_oracle_recurrence_has_the_closed_form():
    """Against explicit weights: o_t = sum_s exp(i_s + sum f_(s+1..t)) (k_s . q_t) v_s over the normaliser."""
    g = torch.Generator().manual_seed(3)
    n, h, d, v = 7, 2, 4, 5
    q, k, vals = (torch.randn(n, h, x, generator=g, dtype=torch.float64) for x in (d, d, v))
    li = torch.randn(n, h, generator=g, dtype=torch.float64)
    lf = -torch.rand(n, h, generator=g, dtype=torch.float64)
    got = ref.mlstm_recurrence(q, k, vals, li, lf)
    for head in range(h):
        for t in range(n):
            w = torch.stack([torch.exp(li[s, head] + lf[s + 1:t + 1, head].sum()) for s in range(t + 1)])
            dots = k[:t + 1, head] @ q[t, head]
            num = (w * dots) @ vals[:t + 1, head]
            # in these units the floor exp(-m) of the stabilised form is 1
            m = torch.zeros((), dtype=torch.float64)
            for s in range(t + 1):
                m = torch.maximum(lf[s, head] + m, li[s, head])
            den = torch.maximum((w * dots).sum().abs(), torch.ones(())) + 1e-6 * torch.exp(m)
            assert torch.allclose(got[t, head], num / den, atol=1e-9)


def test_oracle_runs_every_configuration():
    for make in CONFIGS.values():
        cfg = make()
        out = ref.forward(tokens(0, 30, cfg["vocab"]), ref.random_weights(cfg), cfg)
        assert out.shape == (30, cfg["vocab"]) and bool(out.isfinite().all())


# ---- cache manager ----
def test_cache_manager_holds_one_chunk_per_window():
    m = manager(windows=(20, 0), num_blocks=8, block_size=16, slots=2)
    seq = Sequence(list(range(50)), block_size=16)
    assert m.can_allocate(seq)
    m.allocate(seq)
    assert [len(t) for t in seq.group_tables] == [2, 4]            # 20 tokens; all 50
    for _ in range(30):
        seq.append_token(1)
        m.append(seq)
    assert [len(t) for t in seq.group_tables] == [2, 5]
    other = Sequence([1] * 33, block_size=16)
    m.allocate(other)
    assert {*seq.group_tables[1]} & {*other.group_tables[1]} == set() and seq.state_slot != other.state_slot
    assert not m.can_allocate(Sequence([1], block_size=16))        # no slot left
    held = seq.group_tables[1]
    m.deallocate(seq)
    assert seq.state_slot < 0 and seq.group_tables == [] and seq.num_computed_tokens == 0
    third = Sequence([1] * 80, block_size=16)
    m.allocate(third)
    assert {*third.group_tables[1]} == {*held}                     # blocks and slot come round again
    assert m.holds(8 * 16) and not m.holds(8 * 16 + 1)


# ---- step metadata ----
def _brute_force(seqs, window, bs, index):
    """Per row: which (kind, position in chunk) it has and where its key goes, computed row by row."""
    rows = []
    for s in seqs:
        p0, n = s.num_computed_tokens, s.num_scheduled_tokens
        size = window or p0 + n
        last_chunk = (p0 + n - 1) // size
        for p in range(p0, p0 + n):
            kind = "decode" if n == 1 else "prefixed" if p // size == p0 // size and p0 % size else "fresh"
            stored = p // size == last_chunk or kind == "prefixed"
            slot = s.group_tables[index][(p % size) // bs] * bs + (p % size) % bs
            rows.append((kind, p % size, slot if stored else -1))
    return rows


@pytest.mark.parametrize("seed", range(12))
def test_ragged_arrays_against_row_by_row(seed):
    rng = random.Random(seed)
    windows, bs = [rng.choice([7, 16, 20, 48]), 0], 16
    m = manager(windows, 400, bs, 8)
    seqs = []
    for _ in range(rng.randint(1, 6)):
        total = rng.randint(1, 150)
        s = Sequence(tokens(seed, total, 99), block_size=bs)
        m.allocate(s)
        s.num_scheduled_tokens = rng.choice([1, 1, 2, 3, min(40, total), total])
        s.num_scheduled_tokens = min(s.num_scheduled_tokens, total)
        s.num_computed_tokens = total - s.num_scheduled_tokens
        seqs.append(s)
    arrays, per_window, counts, facts = ragged_arrays(seqs, windows, bs, memory_units=3)
    packed = [seqs[i] for i in facts["order"]]
    assert [s.num_scheduled_tokens > 1 for s in packed] == sorted(s.num_scheduled_tokens > 1 for s in packed)
    cu = arrays["cu_seqlens"]
    for e, s in enumerate(packed):
        lo, hi = cu[e], cu[e + 1]
        assert arrays["input_ids"][lo:hi].tolist() == s.token_ids[s.num_computed_tokens:]
        assert arrays["positions"][lo:hi].tolist() == list(range(s.num_computed_tokens, len(s)))
        assert (arrays["row_entry"][lo:hi] == e).all() and facts["starts"][facts["order"][e]] == lo
        assert (arrays["bank_in"][e] == arrays["bank_out"][e]) == (s.num_scheduled_tokens == 1)
        assert arrays["bank_out"][e] == 2 * s.state_slot + s.state_bank
    for g, window in enumerate(windows):
        rows, w, c = _brute_force(packed, window, bs, g), per_window[g], counts[g]
        dst = w.get("dst_row", np.arange(len(rows)))
        assert sorted(dst.tolist()) == list(range(len(rows)))
        bounds = {"decode": (0, c["num_decode"]), "prefixed": (c["num_decode"], c["num_decode"] + c["num_prefixed"]),
                  "fresh": (c["num_decode"] + c["num_prefixed"], len(rows))}
        for r, (kind, place, slot) in enumerate(rows):
            lo, hi = bounds[kind]
            assert lo <= dst[r] < hi
            early, late = w["slots"][r], w["late_slots"][dst[r]] if "late_slots" in w else -1
            assert max(early, late) == slot and min(early, late) == -1 if slot >= 0 else (early, late) == (-1, -1)
            if kind == "prefixed":
                i = int(np.searchsorted(w["prefixed_cu_q"], dst[r] - lo, side="right")) - 1
                q0, k0, k1 = w["prefixed_cu_q"][i], w["prefixed_cu_k"][i], w["prefixed_cu_k"][i + 1]
                q1 = w["prefixed_cu_q"][i + 1]
                assert (k1 - k0) - (q1 - q0) + (dst[r] - lo - q0) == place
                assert early == slot                              # its own piece reads it from the cache
            elif kind == "fresh":
                i = int(np.searchsorted(w["fresh_cu"], dst[r] - lo, side="right")) - 1
                assert dst[r] - lo - w["fresh_cu"][i] == place
            else:
                assert w["chunk_lens"][dst[r]] == place + 1
        # a slot that is read by a piece of the step is not overwritten before attention
    segments = arrays.get("segments", np.zeros((0, 4), np.int32))
    long_entries = [e for e, s in enumerate(packed) if s.num_scheduled_tokens >= LONG_ROWS]
    assert sorted(set(segments[:, 0].tolist())) == long_entries
    for e in long_entries:
        mine = segments[segments[:, 0] == e]
        assert mine[0, 1] == cu[e] and mine[-1, 1] + mine[-1, 2] == cu[e + 1] and (mine[:-1, 2] % 64 == 0).all()
        assert (mine[1:, 1] == mine[:-1, 1] + mine[:-1, 2]).all()
        assert [int(f) for f in mine[:, 3]] == [(i == 0) | 2 * (i == len(mine) - 1) | 4 * (len(mine) == 1) for i in range(len(mine))]


def test_ragged_step_tensors_are_the_arrays():
    m = manager((20, 0))
    s = Sequence(list(range(50)), block_size=16)
    m.allocate(s)
    s.num_computed_tokens, s.num_scheduled_tokens = 13, 37
    step = ragged_step([s], [20, 0], 16, torch.device("cpu"))
    assert step.positions.tolist() == list(range(13, 50)) and step.num_tokens == 37
    w = step.windows[0]
    assert (w.num_decode, w.num_prefixed, w.num_fresh) == (0, 7, 30) and w.fresh_cu.tolist() == [0, 20, 30]
    assert w.prefixed_cu_k.tolist() == [0, 20] and w.late_slots is not None
    assert all(t.data_ptr() % 16 == 0 for t in (step.positions, w.slots, w.late_slots))
    assert step.windows[1].late_slots is None


# ---- scheduler ----
class _Recorder:
    """A runner that samples token 7 for every finished portion and checks the steps it is given."""

    def __init__(self, m, budget):
        self.cache_manager, self.budget, self.steps, self.seen = m, budget, [], {}

    def run(self, seqs, is_prefill):
        assert len({s.seq_id for s in seqs}) == len(seqs)
        assert sum(s.num_scheduled_tokens for s in seqs) <= self.budget
        out = []
        for s in seqs:
            assert s.num_scheduled_tokens >= 1 and s.num_computed_tokens + s.num_scheduled_tokens <= len(s)
            for w, table in zip(self.cache_manager.windows, s.group_tables):
                assert len(table) == self.cache_manager.blocks_for(w, len(s))
            out.append(7 if s.num_computed_tokens + s.num_scheduled_tokens == len(s) else None)
        slots = [s.state_slot for s in seqs]
        assert len(set(slots)) == len(slots) and min(slots) >= 0
        self.steps.append((is_prefill, [s.num_scheduled_tokens for s in seqs]))
        return out


def _engine(m, budget, slots, **extra):
    from minivllm_amd.engine.llm_engine import LLMEngine
    runner = _Recorder(m, budget)
    return LLMEngine(dict(block_size=16, max_num_sequences=slots, max_num_batched_tokens=budget, max_position=4096, **extra),
                     model_runner=runner), runner


def test_engine_mixes_portions_and_decoding():
    eng, runner = _engine(manager((20, 0), 64), 40, 4)
    eng.add_prompt([1] * 10, SamplingParams(max_tokens=6, ignore_eos=True))
    eng.step()
    eng.add_prompt([1] * 100, SamplingParams(max_tokens=3, ignore_eos=True))
    done = {}
    for _ in range(50):
        finished, _, _ = eng.step()
        done.update(finished)
        if eng.scheduler.is_finished():
            break
    assert [v for _, v in sorted(done.items())] == [[7] * 6, [7] * 3]
    assert (True, [1, 39]) in runner.steps                        # a decoded token beside a portion of the prompt
    assert (False, [1, 1]) in runner.steps


@pytest.mark.parametrize("seed", range(8))
def test_engine_finishes_random_loads(seed):
    """Tight pools, few slots, small budgets: every request ends with its count, and everything is given back."""
    rng = random.Random(100 + seed)
    m = manager((rng.choice([16, 40]), 0), num_blocks=14, block_size=16, slots=3)
    budget = rng.choice([5, 33, 200])
    eng, runner = _engine(m, budget, 3)
    want = {}
    for i in range(12):
        n, new = rng.randint(1, 120), rng.randint(1, 40)
        eng.add_prompt([1] * n, SamplingParams(max_tokens=new, ignore_eos=True))
        want[eng.scheduler.waiting[-1].seq_id] = new
    got = {}
    for _ in range(5000):
        finished, _, _ = eng.step()
        got.update({k: len(v) for k, v in finished})
        if eng.scheduler.is_finished():
            break
    assert got == want
    assert all(len(p.free_block_ids) == 14 and not p.used_block_ids for p in m.pools) and len(m.free_slots) == 3


def test_engine_refuses_what_no_pool_holds():
    eng, _ = _engine(manager((20, 0), num_blocks=4), 8, 2)
    eng.add_prompt([1] * 60, SamplingParams(max_tokens=4))        # longer than a step's budget: it comes in portions
    with pytest.raises(ValueError, match="blocks"):
        eng.add_prompt([1] * 60, SamplingParams(max_tokens=6))


def test_preemption_starts_over():
    sch = Scheduler(4, 64, 0, 16, -1, cache_manager=manager((0,), num_blocks=4, block_size=16, slots=4))
    a, b = Sequence([1] * 32, SamplingParams(ignore_eos=True), 16), Sequence([1] * 32, SamplingParams(ignore_eos=True), 16)
    sch.add_sequence(a), sch.add_sequence(b)
    seqs, prefill = sch.schedule()
    assert prefill and seqs == [a, b]
    sch.postprocess(seqs, [5, 5])
    seqs, prefill = sch.schedule()                                # both need a third block: the later one goes back
    assert not prefill and seqs == [a] and b.state_slot < 0 and b.num_computed_tokens == 0 and list(sch.waiting) == [b]
    assert len(b) == 33
