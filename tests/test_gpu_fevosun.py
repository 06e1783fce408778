"""Fevosun on the GPU: every mechanism against the plain oracle, and the model through its cache, batches and engine."""
import json
import math
import random

import numpy as np
import pytest
import torch

from minivllm_amd.engine.hybrid_runner import HybridModelRunner
from minivllm_amd.engine.ragged import ragged_step
from minivllm_amd.engine.sequence import Sequence
from minivllm_amd.engine.windows import SlidingWindow
from minivllm_amd.layers.basic import rotary_pair_table
from minivllm_amd.layers.experts import ExpertOutput, SparseExperts, interleave_gate_up, moe_linear, moe_plan, moe_route_softmax
from minivllm_amd.layers.fused import gated_unit, stream_norm
from minivllm_amd.layers.mixers import RotaryLatentAttention, SharedKeyAttention, distance_slopes
from minivllm_amd.layers.window import copy_rows, head_rope, latent_rope_store, window_decode, window_prefill
from minivllm_amd.models.fevosun import FevosunForCausalLM, engine_config
from minivllm_amd.sampling_parameters import SamplingParams
from fevosun_cases import CONFIGS, YARN, attention_layer, config, latent_layer, moe
from oracle import fevosun_oracle as ref
from sokevik_cases import Driver, manager, tokens

pytestmark = pytest.mark.gpu
DEV = torch.device("cuda:0")
DTYPES = [torch.float32, torch.bfloat16]


def rel(got, want):
    """Root mean square error over the root mean square of the expected values."""
    got, want = got.detach().double().cpu(), want.double()
    assert got.shape == want.shape and bool(got.isfinite().all())
    return ((got - want).pow(2).mean().sqrt() / want.pow(2).mean().sqrt().clamp_min(1e-30)).item()


def row_rel(got, want):
    """The same of the worst row."""
    got, want = got.detach().double().cpu().flatten(1), want.double().flatten(1)
    assert got.shape == want.shape and bool(got.isfinite().all())
    return ((got - want).pow(2).mean(-1).sqrt() / want.pow(2).mean(-1).sqrt().clamp_min(1e-30)).max().item()


def tol(dtype, f32=2e-6, bf16=8e-3):
    return f32 if dtype == torch.float32 else bf16


def gen(seed):
    return torch.Generator().manual_seed(seed)


def rand(g, *shape, dtype=torch.float32, scale=1.0):
    return (torch.randn(*shape, generator=g) * scale).to(dtype)


def inside(t, left=8, right=16):
    """The same values as a view of wider rows, as a slice of a projection is; NaN around them."""
    wide = torch.full((t.shape[0], left + t[0].numel() + right), float("nan"), dtype=t.dtype, device=DEV)
    view = wide[:, left:left + t[0].numel()]
    view.copy_(t.flatten(1))
    return view.unflatten(-1, t.shape[1:])


# ---- rows ----
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width", [(1, 8), (37, 40), (500, 1024)])
def test_copy_rows(dtype, rows, width):
    g = gen(width)
    src, at, from_ = rand(g, rows, width, dtype=dtype), torch.randperm(rows + 9, generator=g)[:rows], torch.randint(0, rows, (rows,), generator=g)
    at[::5] = -1
    a, b = torch.zeros(rows + 9, width, dtype=dtype, device=DEV), torch.zeros(rows, width + 8, dtype=dtype, device=DEV)
    copy_rows(inside(src), a, at.to(DEV), from_.to(DEV), b[:, :width], None)
    want = torch.zeros(rows + 9, width, dtype=dtype)
    want[at[at >= 0]] = src[from_[at >= 0]]
    assert torch.equal(a.cpu(), want) and torch.equal(b[:, :width].cpu(), src[from_]) and not b[:, width:].any()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("interleaved", [True, False])
@pytest.mark.parametrize("heads,dim,rot,dims,scaling", [(5, 16, 20, 20, YARN), (3, 32, 32, 32, None), (2, 8, 6, 4, None), (1, 64, 64, 64, YARN), (7, 32, 48, 16, None)])
def test_head_rope(dtype, interleaved, heads, dim, rot, dims, scaling):
    """In place for the later rows, into another tensor with zeros behind for the first ones; nothing else changes."""
    g, rows, first = gen(rot), 29, 11
    cos, sin = ref.rotation({"base": 300.0, "dims": dims, "scaling": scaling}, 500)
    table = rotary_pair_table(300.0, dims, 500, scaling).to(DEV)
    x, pos = rand(g, rows, heads, dim + rot, dtype=dtype), torch.randint(0, 500, (rows,), generator=g)
    want = x.double().clone()
    want[..., dim:] = ref.rotate(x.double()[..., dim:], cos[pos], sin[pos], interleaved)
    for n in (0, first, rows):
        mine = inside(x, 8 * 4, 8)
        out = torch.full((max(n, 1), heads, 24 + rot + 40), 7.0, dtype=dtype, device=DEV)
        head_rope(mine, dim, rot, table, pos.to(DEV), interleaved, out if n else None, 24, n)
        assert torch.equal(mine[:n].cpu(), x[:n]) and torch.equal(mine[..., :dim].cpu(), x[..., :dim])
        if n < rows:
            assert rel(mine[n:, :, dim:], want[n:, :, dim:]) < tol(dtype, 1e-6, 4e-3)
        if n:
            assert rel(out[..., 24:24 + rot], want[:n, :, dim:]) < tol(dtype, 1e-6, 4e-3)
            assert not out[..., 24 + rot:].any() and bool((out[..., :24] == 7).all())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rank,rot,dims,width,rank2,interleaved", [(72, 20, 20, 128, 0, False), (40, 6, 6, 96, 50, True), (512, 64, 64, 576, 700, False),
                                                                    (1, 32, 16, 64, 1, True), (1500, 70, 70, 1632, 1999, True)])
def test_latent_rope_store(dtype, rank, rot, dims, width, rank2, interleaved):
    g, rows, eps = gen(rank), 21, 1e-2
    at, width2 = -(-rank // 16) * 16, -(-rank2 // 64) * 64
    latent, part, second = rand(g, rows, rank, dtype=dtype), rand(g, rows, rot, dtype=dtype), rand(g, rows, rank2, dtype=dtype)
    w, w2, pos = rand(g, rank), rand(g, rank2), torch.randint(0, 90, (rows,), generator=g)
    cos, sin = ref.rotation({"base": 30.0, "dims": dims, "scaling": YARN}, 90)
    want = torch.zeros(rows, width, dtype=torch.float64)
    want[:, :rank] = ref.rms(latent.double(), eps) * w.double()
    want[:, at:at + rot] = ref.rotate(part.double(), cos[pos], sin[pos], interleaved)
    src = torch.full((rows, width), 5.0, dtype=dtype)                      # what lies between the parts is not read
    src[:, :rank], src[:, at:at + rot] = latent, part
    slots, keys = torch.randperm(48, generator=g)[:rows], torch.randperm(30, generator=g)[:rows]
    slots[3] = keys[4] = -1
    cache, out = torch.full((3, 16, width), 9.0, dtype=dtype, device=DEV), torch.full((30, width), 9.0, dtype=dtype, device=DEV)
    on = lambda t: t.to(DEV)
    got2 = latent_rope_store(inside(src), on(w), eps, at, rot, rotary_pair_table(30.0, dims, 90, YARN).to(DEV), on(pos), interleaved, cache, on(slots),
                             out, on(keys), inside(torch.nn.functional.pad(second, (0, width2 - rank2), value=5.0)) if rank2 else None, on(w2) if rank2 else None)
    live, kept = slots >= 0, keys >= 0
    assert rel(cache.view(48, width)[on(slots[live])], want[live]) < tol(dtype, 2e-6, 4e-3)
    assert rel(out[on(keys[kept])], want[kept]) < tol(dtype, 2e-6, 4e-3)
    assert int((cache == 9).all(-1).sum()) == 48 - int(live.sum()) and int((out == 9).all(-1).sum()) == 30 - int(kept.sum())
    if rank2:
        assert rel(got2[:, :rank2], ref.rms(second.double(), eps) * w2.double()) < tol(dtype, 2e-6, 4e-3) and not got2[:, rank2:].any()


# ---- attention ----
def attend_reference(q, k, v, scale, window, slopes=None, temps=None, gate=None):
    """One entry: q (n, H, d), k (m, G, d), v (m, G, e), query i at key m - n + i; float64."""
    n, heads, m, groups = q.shape[0], q.shape[1], k.shape[0], k.shape[1]
    q, k, v = q.double(), k.double(), v.double()
    away = (torch.arange(m - n, m)[:, None] - torch.arange(m)[None, :])
    see = (away >= 0) & ((away < window) if window else torch.ones_like(away, dtype=torch.bool))
    out = torch.empty(n, heads, v.shape[2], dtype=torch.float64)
    for h in range(heads):
        s = q[:, h] @ k[:, h * groups // heads].T * scale
        if temps is not None:
            s = s * temps[:, None]
        if slopes is not None:
            s = s - slopes[h].double() * away
        out[:, h] = torch.softmax(s.masked_fill(~see, -math.inf), -1) @ v[:, h * groups // heads]
    return out if gate is None else out * torch.sigmoid(gate.double())


def prefix_sums(lens):
    return torch.tensor([0, *np.cumsum(lens)], dtype=torch.int32)


SHARED = [(4, 2, 32), (6, 2, 64), (5, 1, 96), (8, 2, 128), (2, 2, 192), (4, 1, 256), (3, 3, 320)]
PARTS = [(4, 32, 32), (3, 64, 64), (2, 96, 32), (2, 128, 64), (2, 192, 32), (1, 256, 64), (2, 64, 96), (1, 128, 32), (2, 32, 64)]
WINDOWS = [0, 1, 31, 64, 130, 1000]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", WINDOWS)
@pytest.mark.parametrize("heads,groups,dim", SHARED)
def test_window_prefill_of_shared_keys(dtype, window, heads, groups, dim):
    """Entries of any length behind pasts of any length; bias, temperature and gate, and none of them."""
    g, lens, pasts = gen(dim + window), [70, 1, 200, 33], [0, 40, 17, 129]
    rows, keys = sum(lens), sum(lens) + sum(pasts)
    q, k, gate = rand(g, rows, heads, dim, dtype=dtype, scale=2.0), rand(g, keys, groups, dim, dtype=dtype), rand(g, rows, heads, dim, dtype=dtype)
    pos = torch.randint(0, 3000, (rows,), generator=g)
    slopes, scale = distance_slopes(heads), dim ** -0.5
    cu_q, cu_k = prefix_sums(lens), prefix_sums([a + b for a, b in zip(lens, pasts)])
    for full in (True, False):
        temps = ref.query_temperature(pos.tolist(), 0.3, 100) if full else None
        out = torch.full((rows, heads, dim), float("nan"), dtype=dtype, device=DEV)
        extra = dict(slopes=slopes.to(DEV), temperature=(0.3, 100), gate=inside(gate), positions=pos.to(DEV)) if full else {}
        window_prefill(out, inside(q), inside(k), cu_q.to(DEV), cu_k.to(DEV), scale, window, **extra)
        for e in range(len(lens)):
            a, b = slice(int(cu_q[e]), int(cu_q[e + 1])), slice(int(cu_k[e]), int(cu_k[e + 1]))
            want = attend_reference(q[a], k[b], k[b], scale, window, slopes if full else None, None if temps is None else temps[a], gate[a] if full else None)
            assert rel(out[a], want) < tol(dtype, 3e-6, 1.5e-2), e


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", WINDOWS)
@pytest.mark.parametrize("heads,dim,rot", PARTS)
def test_window_prefill_of_keys_in_two_parts(dtype, window, heads, dim, rot):
    g, lens, pasts = gen(dim + rot + window), [65, 150, 32], [0, 64, 7]
    rows, keys = sum(lens), sum(lens) + sum(pasts)
    q, k, k2, v = rand(g, rows, heads, dim + rot, dtype=dtype, scale=2.0), rand(g, keys, heads, dim, dtype=dtype), rand(g, keys, rot, dtype=dtype), rand(g, keys, heads, dim, dtype=dtype)
    scale, both = (dim + rot) ** -0.5, torch.cat([k, k2[:, None].expand(-1, heads, -1)], -1)
    cu_q, cu_k = prefix_sums(lens), prefix_sums([a + b for a, b in zip(lens, pasts)])
    out = torch.full((rows, heads, dim), float("nan"), dtype=dtype, device=DEV)
    window_prefill(out, inside(q), inside(k), cu_q.to(DEV), cu_k.to(DEV), scale, window, k2=inside(k2), v=inside(v))
    for e in range(len(lens)):
        a, b = slice(int(cu_q[e]), int(cu_q[e + 1])), slice(int(cu_k[e]), int(cu_k[e + 1]))
        assert rel(out[a], attend_reference(q[a], both[b], v[b], scale, window)) < tol(dtype, 3e-6, 1.5e-2), e


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("parts", [False, True])
@pytest.mark.parametrize("window", [5, 64, 97])
def test_window_edges_in_prompts(dtype, parts, window):
    """One key far above all others: seen by the queries up to window - 1 behind it, not by the next one; keys at the start of the
    entry, at tile borders and in the part that the past brings."""
    g, n, past, heads, dim, rot = gen(window), 260, window + 20, 2, 64, 32
    for at in (0, 1, 19, past - 1, past, past + 63, past + 64, past + 127):
        k, v = rand(g, past + n, heads, dim, dtype=dtype, scale=0.1), rand(g, past + n, heads, dim, dtype=dtype, scale=0.1)
        q = torch.ones(n, heads, dim, dtype=dtype)
        k[at], v[at] = 1.0, 5.0
        cu_q, cu_k = prefix_sums([n]).to(DEV), prefix_sums([past + n]).to(DEV)
        out = torch.empty(n, heads, dim, dtype=dtype, device=DEV)
        if parts:
            zeros = torch.zeros(n, heads, rot, dtype=dtype), torch.zeros(past + n, rot, dtype=dtype)
            window_prefill(out, torch.cat([q, zeros[0]], -1).to(DEV), k.to(DEV), cu_q, cu_k, 0.5, window, k2=zeros[1].to(DEV), v=v.to(DEV))
            want = attend_reference(q, k, v, 0.5, window)
        else:
            window_prefill(out, q.to(DEV), k.to(DEV), cu_q, cu_k, 0.5, window)
            want = attend_reference(q, k, k, 0.5, window)
        level = 5.0 if parts else 1.0
        seen = [0 <= past + i - at < window for i in range(n)]
        assert (((out.float().cpu().mean((1, 2)) - level).abs() < 0.1 * level) == torch.tensor(seen)).all(), at
        assert (out.double().cpu() - want).abs().max() < tol(dtype, 1e-5, 3e-2) * level


def ring_case(seed, lens, rows_of, heads, groups, width, dtype, window, bs=16, scale=1.0):
    """Rings of entries that hold ``lens[e]`` tokens, of which the last ``rows_of[e]`` ask; block tables shuffled, NaN elsewhere."""
    g, w = gen(seed), SlidingWindow(window)
    places = [min(n, w.places) if w.places else n for n in lens]
    need = [-(-p // bs) for p in places]
    perm, blocks = torch.randperm(sum(need) + 3, generator=g).tolist(), []
    for n in need:
        blocks.append([perm.pop() for _ in range(n)])
    tables = torch.full((len(lens), max(need) + 2), -1, dtype=torch.int32)
    cache = torch.full((sum(need) + 3, bs, groups, width), float("nan"), dtype=dtype)
    keys = [rand(g, n, groups, width, dtype=dtype) for n in lens]
    for e, n in enumerate(lens):
        tables[e, :need[e]] = torch.tensor(blocks[e], dtype=torch.int32)
        for b in blocks[e]:
            cache[b] = 0.0                                               # blocks are handed out with whatever finite numbers they hold
        for p in range(max(0, n - (w.places or n)), n):
            place = p % w.places if w.places else p
            cache[blocks[e][place // bs], place % bs] = keys[e][p]
    asked = [(e, lens[e] - r + i) for e, r in enumerate(rows_of) for i in range(r)]
    q = rand(g, len(asked), heads, width, dtype=dtype, scale=scale)
    entry = torch.tensor([e for e, _ in asked], dtype=torch.int32)
    return w, q, keys, cache, tables, entry, asked


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", [0, 1, 20, 64, 300])
@pytest.mark.parametrize("heads,groups,width", [(4, 2, 32), (6, 2, 64), (18, 1, 96), (8, 2, 128), (2, 2, 192), (35, 1, 256), (3, 3, 320), (70, 1, 512), (5, 1, 576)])
def test_window_decode(dtype, window, heads, groups, width):
    """Single rows and rows of short entries, whose later rows are in the ring already; rings that have come round."""
    lens, rows_of = [1, 20, 21, 47, 50, 333, 700], [1, 1, 2, 31, 1, 17, 1]
    w, q, keys, cache, tables, entry, asked = ring_case(width + window, lens, rows_of, heads, groups, width, dtype, window, scale=2.0)
    values, g = 512 if width == 576 else width, gen(3)
    slopes, gate, scale = distance_slopes(heads), rand(g, len(asked), heads, values, dtype=dtype), width ** -0.5
    lengths = torch.tensor([p + 1 for _, p in asked])
    on = lambda t: t.to(DEV)
    for full in (True, False):
        out = torch.full((len(asked), heads, values), float("nan"), dtype=dtype, device=DEV)
        extra = dict(slopes=on(slopes), temperature=(0.3, 100), gate=inside(gate)) if full else {}
        window_decode(out, inside(q), on(cache), on(tables), on(entry), on(lengths), scale, window, w.places, **extra)
        want = torch.cat([attend_reference(q[i:i + 1], keys[e][:p + 1], keys[e][:p + 1, :, :values], scale, window, slopes if full else None,
                                           ref.query_temperature([p], 0.3, 100) if full else None, gate[i:i + 1] if full else None)
                          for i, (e, p) in enumerate(asked)])
        assert rel(out, want) < tol(dtype, 3e-6, 1.5e-2) and row_rel(out, want) < tol(dtype, 2e-5, 6e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", [5, 33, 64])
def test_window_edges_while_decoding(dtype, window):
    """One key far above all others, decoded past until the ring has come round: seen for window - 1 tokens after its own."""
    heads, width, n, bs = 2, 64, 3 * window + 60, 16
    w = SlidingWindow(window)
    m = manager([w], 20, bs, 1)
    for at in (0, 1, window - 1, window, w.places - 1, w.places):
        s = Sequence([1] * n, block_size=bs)
        m.allocate(s)
        table = s.group_tables[0]
        cache, keys = torch.zeros(20, bs, 1, width, dtype=dtype), rand(gen(at), n, 1, width, dtype=dtype, scale=0.1)
        keys[at] = 1.0
        caches = []
        for p in range(n):
            place = p % w.places
            cache[table[place // bs], place % bs] = keys[p]
            caches.append(cache.clone())
        for p in range(max(at - 1, 0), min(at + window + 3, n)):
            out = torch.empty(1, heads, width, dtype=dtype, device=DEV)
            window_decode(out, torch.ones(1, heads, width, dtype=dtype, device=DEV), caches[p].to(DEV), torch.tensor([table], dtype=torch.int32, device=DEV),
                          torch.zeros(1, dtype=torch.int32, device=DEV), torch.tensor([p + 1], device=DEV), 0.5, window, w.places)
            assert (abs(float(out.float().mean()) - 1.0) < 0.1) == (0 <= p - at < window), (at, p)
        m.deallocate(s)


def test_window_decode_in_shares():
    """Long rows are cut into shares that a second launch joins (gate included); a caller's workspace serves as well."""
    from minivllm_amd.layers.window import window_decode_workspace_bytes
    for dtype in DTYPES:
        w, q, keys, cache, tables, entry, asked = ring_case(1, [5000, 3, 2049], [1, 1, 1], 4, 2, 64, dtype, 4000)
        need = window_decode_workspace_bytes(3, 4, 2, 64, 64, tables.shape[1] * 16, dtype)
        assert need > 0
        gate, on = rand(gen(0), 3, 4, 64, dtype=dtype), lambda t: t.to(DEV)
        want = torch.cat([attend_reference(q[i:i + 1], keys[e], keys[e], 0.2, 4000, gate=gate[i:i + 1]) for i, (e, _) in enumerate(asked)])
        for ws in (None, torch.empty(need, dtype=torch.uint8, device=DEV)):
            out = torch.empty(3, 4, 64, dtype=dtype, device=DEV)
            window_decode(out, on(q), on(cache), on(tables), on(entry), torch.tensor([5000, 3, 2049], device=DEV), 0.2, 4000, w.places, gate=on(gate), workspace=ws)
            assert row_rel(out, want) < tol(dtype, 1e-5, 2e-2)


# ---- mixers as layers ----
def weights_of(entry, width, seed=0, peak=1.0):
    w = {k[len("l0.mix."):]: t for k, t in ref.random_weights(config([entry], width=width), seed).items() if k.startswith("l0.mix.")}
    for n in ("q", "uq"):
        if n in w:
            w[n] = w[n] * peak
    return w


def mixer_case(entry, width, dtype, seed=0, peak=1.0, eps=1e-3):
    """The mixer between its two projections as a function of (h, step), and the oracle's."""
    w, m, view = weights_of(entry, width, seed, peak), entry["mixer"], SlidingWindow(entry["mixer"]["mask"]["size"])
    inputs = -(-width // 64) * 64
    if entry["type"] == "attention":
        t = m.get("q_temp")
        mixer = SharedKeyAttention(m["heads"], m["kv_heads"], m["dim"], m["scale"], 0, view, 16, dtype, (t["coef"], t["every"]) if t else (0.0, 0),
                                   distance_slopes(m["heads"]))
    else:
        mixer = RotaryLatentAttention(m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], m["scale"], 0, view, 16, dtype, eps,
                                      "q_rank" in m, m.get("q_rank", 0), 64)
        mixer.table = rotary_pair_table(m["rot"]["base"], m["rot"]["dims"], 2048, m["rot"].get("scaling")).to(DEV)
    front, behind = mixer.load(lambda n: w[n], lambda t: t.to(DEV, dtype).contiguous(), inputs)
    mixer.allocate(24, DEV)

    def run(h, step):
        h = torch.nn.functional.pad(h, (0, inputs - width)).to(DEV)
        proj = h @ front.T
        z = torch.full((h.shape[0], mixer.sizes[1] + 16), float("nan"), dtype=dtype, device=DEV)
        mixer(h, proj, z[:, :mixer.sizes[1]], step)
        return (z[:, :mixer.sizes[1]] @ behind.T).cpu()

    wd = {k: t.double() for k, t in w.items()}
    plain = (lambda h: ref.attention(h, wd, "", m)) if entry["type"] == "attention" else (lambda h: ref.latent_attention(h, wd, "", m, eps, "q_rank" in m))
    return run, plain, mixer


MIXERS = {
    "groups": attention_layer(heads=6, kv_heads=2, dim=40, window=20), "one": attention_layer(heads=5, kv_heads=1, dim=128, window=150, q_temp=(0.3, 50)),
    "wide": attention_layer(heads=2, kv_heads=2, dim=300, window=64), "short": attention_layer(heads=4, kv_heads=4, dim=16, window=3, q_temp=None),
    "yarn": latent_layer(heads=5, window=33), "queries": latent_layer(heads=3, dim=64, rot_dim=64, vdim=64, rank=64, q_rank=30, scaling=None, window=64),
    "many": latent_layer(heads=18, dim=16, rot_dim=2, vdim=48, rank=150, window=100), "large": latent_layer(heads=2, dim=128, rot_dim=64, vdim=128, rank=512, q_rank=200, window=7),
    "odd": latent_layer(heads=3, dim=200, rot_dim=70, vdim=100, rank=300, window=40, q_rank=9, scaling=None)}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(MIXERS))
@pytest.mark.parametrize("cuts", [[230], [1] * 40 + [2] * 95, [31, 32, 33, 1, 2, 70, 31, 30], [150, 80], [17, 183, 30]], ids=str)
def test_mixers_in_portions(dtype, name, cuts):
    """Peaked scores: decoded rows, short portions, long ones with and without a past give the whole sequence's rows."""
    width, rows = 96, sum(cuts)
    run, plain, mixer = mixer_case(MIXERS[name], width, dtype, peak=2.0)
    h = rand(gen(8), rows, width, dtype=dtype)
    m = manager([mixer.view], 24, 16, 2)
    s = Sequence([1] * rows, block_size=16)
    m.allocate(s)
    got, at = [], 0
    for n in cuts:
        s.num_computed_tokens, s.num_scheduled_tokens = at, n
        got.append(run(h[at:at + n], ragged_step([s], [mixer.view], 16, DEV)))
        at += n
    got, want = torch.cat(got), plain(h.double())
    assert rel(got, want) < tol(dtype, 5e-6, 2.5e-2) and row_rel(got, want) < tol(dtype, 1e-4, 0.15)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["groups", "yarn", "queries"])
def test_mixers_in_batches(dtype, name):
    """Unequal entries in one step, in every form at once, rings and blocks shuffled and used again."""
    width, eps = 80, 1e-3
    run, plain, mixer = mixer_case(MIXERS[name], width, dtype, peak=2.0)
    m, rng = manager([mixer.view], 24, 16, 4), random.Random(1)
    for round_ in range(2):
        total = {"a": 150, "b": 61, "c": 9, "d": 120}
        rows = {k: rand(gen(100 * round_ + i), n, width, dtype=dtype) for i, (k, n) in enumerate(total.items())}
        seqs, at, got = {k: Sequence([1] * n, block_size=16) for k, n in total.items()}, dict.fromkeys(total, 0), {k: [] for k in total}
        for s in seqs.values():
            m.allocate(s)
        while any(at[k] < total[k] for k in total):
            live = [k for k in total if at[k] < total[k] and rng.random() < 0.8]
            if not live:
                continue
            for k in live:
                seqs[k].num_computed_tokens = at[k]
                seqs[k].num_scheduled_tokens = min(rng.choice([1, 1, 2, 5, 31, 32, 50]), total[k] - at[k])
            step = ragged_step([seqs[k] for k in live], [mixer.view], 16, DEV)
            h = torch.cat([rows[live[i]][at[live[i]]:at[live[i]] + seqs[live[i]].num_scheduled_tokens] for i in step.order])
            out = run(h, step)
            for i, k in enumerate(live):
                n = seqs[k].num_scheduled_tokens
                got[k].append(out[step.starts[i]:step.starts[i] + n])
                at[k] += n
        for k in total:
            want = plain(rows[k].double())
            assert rel(torch.cat(got[k]), want) < tol(dtype, 5e-6, 2.5e-2) and row_rel(torch.cat(got[k]), want) < tol(dtype, 1e-4, 0.15), k
            m.deallocate(seqs[k])


# ---- mixture of experts ----
@pytest.mark.parametrize("experts,identity,top", [(9, 3, 4), (5, 0, 1), (18, 5, 3), (1, 1, 2), (64, 7, 6), (120, 100, 9), (1000, 24, 12), (3, 5, 8)])
@pytest.mark.parametrize("shift", [0.0, -3.0])
def test_softmax_router(experts, identity, top, shift):
    """Choices and weights token by token, far logits included; identity experts are told by their sign."""
    g, rows, n = gen(experts + top), 50, experts + identity
    z, correction = rand(g, rows, n + 3, scale=4.0), rand(g, n, scale=0.1) + shift
    z[0] += 300.0
    ids, weights = moe_route_softmax(z.to(DEV), correction.to(DEV), experts, identity, top)
    for t in range(rows):
        want, w = ref.route(z[t, :n].double(), correction.double(), top)
        assert ids[t].tolist() == [e if e < experts else -1 for e in want], t
        assert torch.allclose(weights[t].cpu().double(), w, atol=1e-6)
    _, normed = moe_route_softmax(z.to(DEV), correction.to(DEV), experts, identity, top, renormalize=True)
    assert torch.allclose(normed.sum(1).cpu(), torch.ones(rows), atol=1e-5)


@pytest.mark.parametrize("rows,top,experts", [(1, 2, 1), (7, 3, 10), (2500, 3, 300)])
def test_plan_leaves_out_what_is_no_experts(rows, top, experts):
    ids = torch.randint(-1, experts, (rows, top), generator=gen(rows)).int()
    place = moe_plan(ids.to(DEV), experts).place.cpu().long()
    live = ids.view(-1) >= 0
    assert bool((place[~live] == -1).all()) and sorted(place[live].tolist()) == list(range(int(live.sum())))
    by_place = torch.empty(int(live.sum()), dtype=torch.int32)
    by_place[place[live]] = ids.view(-1)[live]
    assert bool((by_place[1:] >= by_place[:-1]).all())


@pytest.mark.parametrize("limit,alpha,shift", [(0.7, 1.702, 1.0), (math.inf, 1.0, 0.0), (3.0, 0.5, -0.25)])
@pytest.mark.parametrize("rows,top,experts,n,k", [(5, 3, 10, 80, 128), (64, 8, 16, 272, 1088), (700, 3, 7, 336, 192), (1500, 2, 3, 64, 576), (1300, 2, 2, 336, 192)])
@pytest.mark.parametrize("path", ["few", "many", "any"])
def test_clamped_experts_products(rows, top, experts, n, k, path, limit, alpha, shift):
    if path == "few" and rows * top > 512:
        pytest.skip("more pairs than the unsorted form takes")
    dtype, g, f = torch.float32 if path == "any" else torch.bfloat16, gen(n + k), -(-n // 64) * 64
    x, ids = rand(g, rows, k, dtype=dtype), torch.randint(-1, experts, (rows, top), generator=g).int()
    gate, up = (rand(g, experts, f, k, dtype=dtype, scale=2 * k ** -0.5) for _ in range(2))
    both, on = torch.stack([interleave_gate_up(a, b) for a, b in zip(gate, up)]), lambda t: t.to(DEV)
    plan = None if path == "few" else moe_plan(on(ids), experts)
    act = moe_linear(on(x), on(both), on(ids), plan, top, glu=(alpha, limit, shift))
    place = torch.arange(rows * top) if plan is None else plan.place.cpu().long()
    e, xr = ids.view(-1).long(), x.double().repeat_interleave(top, 0)
    for i in range(experts):
        r = (e == i).nonzero()[:, 0]
        if len(r):
            z = (xr[r] @ gate[i].double().T).clamp(max=limit)
            want = z * torch.sigmoid(alpha * z) * ((xr[r] @ up[i].double().T).clamp(-limit, limit) + shift)
            assert row_rel(act.cpu()[place[r]], want) < tol(dtype, 1e-5, 1.5e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width", [(1, 16), (37, 40), (600, 1024)])
def test_gated_unit(dtype, rows, width):
    x = rand(gen(width), rows, 2 * width, dtype=dtype, scale=3.0)
    a, b = x.double().chunk(2, 1)
    z = a.clamp(max=0.9)
    want = z * torch.sigmoid(1.702 * z) * (b.clamp(-0.9, 0.9) + 1)
    out = torch.zeros(rows, width + 24, dtype=dtype, device=DEV)
    gated_unit(inside(x), out[:, 8:8 + width], 1.702, 0.9, 1.0)
    assert rel(out[:, 8:8 + width], want) < tol(dtype, 1e-6, 4e-3) and not out[:, :8].any() and not out[:, 8 + width:].any()
    assert rel(gated_unit(x.to(DEV)), ref.silu(a) * b) < tol(dtype, 1e-6, 4e-3)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [80, 97, 1028])
@pytest.mark.parametrize("sorted_rows", [True, False])
def test_residual_of_choices_that_are_no_experts(dtype, width, sorted_rows):
    """Their rows of the products are never read (NaN there); the input counts in their place."""
    g, rows, top = gen(width), 37, 3
    x, y, own = rand(g, rows, 1, width), rand(g, rows, width, dtype=dtype), rand(g, rows, width + 8, dtype=dtype)
    parts, weights, ids = rand(g, rows * top, width, dtype=dtype), rand(g, rows, top), torch.randint(-1, 2, (rows, top), generator=g).int()
    live = ids.view(-1) >= 0
    place = torch.full((rows * top,), -1)
    place[live] = torch.randperm(int(live.sum()), generator=g)
    at = place if sorted_rows else torch.arange(rows * top)
    shown = torch.full_like(parts, float("nan"))
    shown[at[live]] = parts[live]
    each = torch.where(live[:, None], parts.double(), own.double()[:, :width].repeat_interleave(top, 0)).view(rows, top, width)
    total = x.double()[:, 0] + y.double() + (weights.double()[..., None] * each).sum(1)
    on, one = lambda t: t.to(DEV), torch.ones(1, device=DEV)
    out = ExpertOutput(on(shown), on(weights), on(place.int()) if sorted_rows else None, on(y), None, on(ids), on(own))
    h, new = stream_norm(on(x), out, one, one[None], torch.ones(width, device=DEV), 1e-3)
    assert rel(new[:, 0], total) < 2e-6 and rel(h, ref.rms(total, 1e-3)) < tol(dtype, 4e-6, 4e-3)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cfg", [moe(shared=None), moe(experts=12, top=5, identity=1, ff=72, shared=None), moe(experts=5, top=1, identity=0, shared=None),
                                 moe(experts=2, top=5, identity=6, shared=None), moe(experts=40, top=8, identity=20, ff=64, shared=None)], ids="abcde")
def test_experts(dtype, cfg):
    width, inputs, r = 80, 128, cfg["router"]
    w = {k[len("l0.mlp."):]: t for k, t in ref.random_weights(config([attention_layer(mlp=cfg)]), 3).items() if k.startswith("l0.mlp.")}
    m = SparseExperts(width, inputs, r["experts"], r["top"], cfg["expert"]["ff"], softmax=True, identity=r["identity"], glu=(1.702, cfg["expert"]["limit"], 1.0))
    m.load(lambda n: w[n], lambda t: t.to(DEV, dtype).contiguous())
    h = rand(gen(4), 600, width, dtype=dtype)
    want, one = ref.experts(h.double(), {k: t.double() for k, t in w.items()}, "", cfg), torch.ones(1, device=DEV)
    for lo, n in ((0, 600), (0, 1), (1, 5), (40, 64)):
        padded = torch.nn.functional.pad(h[lo:lo + n], (0, inputs - width)).to(DEV)
        _, x = stream_norm(torch.zeros(n, 1, width, device=DEV), m(padded), one, one[None], torch.ones(width, device=DEV), 1.0)
        err = (x[:, 0].cpu().double() - want[lo:lo + n]).pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt()
        assert err.max() < tol(dtype, 1e-5, 3e-2), (lo, n, int(err.argmax()))


# ---- the model ----
_runners: dict = {}


def make_runner(name, dtype, **extra):
    key = (name, dtype, tuple(sorted(extra.items())))
    if key not in _runners:
        cfg = CONFIGS[name]()
        full = engine_config({**cfg, "dtype": "fp32" if dtype == torch.float32 else "bf16", "block_size": 16, "max_cached_blocks": 40,
                              "max_num_sequences": 4, "max_position": 1024, **extra, "enforce_eager": True})
        runner = HybridModelRunner(full, FevosunForCausalLM)
        weights = ref.random_weights(cfg, seed=11)
        runner.model.load_weights(weights)
        if not extra.get("enforce_eager", True):
            runner.capture_decode_graphs()           # after the weights: a captured step holds their addresses
        _runners[key] = runner, cfg, weights
    return _runners[key]


_wanted: dict = {}


def oracle_logits(seed, n, cfg, weights):
    key = (json.dumps(cfg), seed, n)
    if key not in _wanted:
        _wanted[key] = ref.forward(tokens(seed, n, cfg["vocab"]), weights, cfg)
    return _wanted[key]


# a row's logits error over the logits' spread: all rows, the median.  bf16: a router's close call goes the other way in some
# rows of a random model, and from there into later ones
MODEL_TOL = {torch.float32: (2e-4, 2e-5), torch.bfloat16: (1.0, 5e-2)}


def row_errors(got, want):
    d = got.double() - want
    return (d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt() / want.std()


def check_rows(got, want, dtype, *what):
    err = row_errors(got, want)
    assert err.max() < MODEL_TOL[dtype][0] and err.median() < MODEL_TOL[dtype][1], (*what, int(err.argmax()), float(err.max()), float(err.median()))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
@pytest.mark.parametrize("sizes", [[170], [1], [2], [3, 5, 64, 1, 1, 33], [64], [150, 1]], ids=str)
def test_model_in_portions(dtype, name, sizes):
    runner, cfg, weights = make_runner(name, dtype)
    n = 170 if sizes != [1] or dtype == torch.float32 else 90
    want = oracle_logits(7, 170, cfg, weights)[:n]
    got = Driver(runner).run_alone("a", tokens(7, 170, cfg["vocab"])[:n], sizes)
    check_rows(got, want, dtype)


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_residual_layer_by_layer(name):
    runner, cfg, weights = make_runner(name, torch.float32)
    toks, want, got = tokens(7, 60, cfg["vocab"]), [], []
    ref.forward(toks, weights, cfg, layer_outputs=want)
    s = Sequence(toks, block_size=16)
    runner.cache_manager.allocate(s)
    s.num_scheduled_tokens = 60
    runner.forward_step([s], got)
    runner.cache_manager.deallocate(s)
    assert len(got) == len(want) == len(cfg["layers"])
    for i, (a, b) in enumerate(zip(got, want)):
        assert rel(a, b) < 2e-5, i


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_mixed_batches_and_reuse(dtype, name):
    """Portions beside decoded tokens, requests left out of steps, pages given back and used again in a small pool: every request's
    logits are its own."""
    runner, cfg, weights = make_runner(name, dtype)
    lens = {"a": 170, "b": 61, "c": 7, "d": 130, "e": 96, "f": 33}
    toks = {k: tokens(20 + i, n, cfg["vocab"]) for i, (k, n) in enumerate(lens.items())}
    rng, drv, at, waiting, live = random.Random(4), Driver(runner), dict.fromkeys(lens, 0), list(lens), []
    while waiting or live:
        while waiting and len(live) < 4:
            live.append(waiting.pop(0))
        chosen = [k for k in live if rng.random() < 0.8] or live[:1]
        portions = {k: toks[k][at[k]:at[k] + rng.choice([1, 1, 1, 2, 3, 17, 40, 64])] for k in chosen}
        for k in chosen:
            at[k] += len(portions[k])
        ended = [k for k in chosen if at[k] == lens[k]]
        drv.step(portions, ended)
        live = [k for k in live if k not in ended]
    for i, k in enumerate(lens):
        check_rows(torch.cat(drv.logits[k]), oracle_logits(20 + i, lens[k], cfg, weights), dtype, k)
    assert len(runner.cache_manager.free_slots) == 4
    assert all(len(p.free_block_ids) == 40 for p in runner.cache_manager.pools)


def test_logits_do_not_depend_on_cuts_and_company():
    """bf16: the same tokens whole, in portions, token by token and beside others differ by rounding only (away from a
    router's close calls: in most rows)."""
    runner, cfg, _ = make_runner("mixed", torch.bfloat16)
    toks = tokens(3, 120, cfg["vocab"])
    base = Driver(runner).run_alone("a", toks, [120]).double()
    others = [Driver(runner).run_alone("a", toks, sizes) for sizes in ([1], [2], [33], [7, 60])]
    drv = Driver(runner)
    for at in range(0, 120, 40):
        drv.step({"x": tokens(50, 35, cfg["vocab"])[:35 - at // 4], "a": toks[at:at + 40], "y": tokens(51, 3, cfg["vocab"])[:1]}, ["x"])
    drv.step({"y": [1]}, ["y", "a"])
    for got in [*others, torch.cat(drv.logits["a"])]:
        assert row_errors(got, base).median() < 4e-2


def test_first_tokens_and_one_token_prompts():
    runner, cfg, weights = make_runner("mixed", torch.float32)
    want = oracle_logits(7, 170, cfg, weights)
    for n in (1, 2, 3, 4):
        check_rows(Driver(runner).run_alone("x", tokens(7, 170, cfg["vocab"])[:n], [n]), want[:n], torch.float32, n)


def test_long_decoding():
    """A few hundred decoded tokens: every ring comes round several times."""
    runner, cfg, weights = make_runner("mixed", torch.float32)
    got = Driver(runner).run_alone("x", tokens(31, 330, cfg["vocab"]), [5, 1])
    assert row_errors(got, oracle_logits(31, 330, cfg, weights)).max() < 2e-4


def greedy_reference(prompt, new, weights, cfg):
    """Greedy continuation by the oracle and the smallest lead of a chosen token over the next one."""
    toks, lead = list(prompt), math.inf
    for _ in range(new):
        logits = ref.forward(toks, weights, cfg)[-1]
        top = logits.topk(2)
        lead = min(lead, float(top.values[0] - top.values[1]) / float(logits.std()))
        toks.append(int(top.indices[0]))
    return toks[len(prompt):], lead


def generate(runner, prompts, new, budget=64, slots=4, **kw):
    from minivllm_amd.engine.llm_engine import LLMEngine
    runner.sample_calls = 0
    eng = LLMEngine(dict(runner.config, max_num_batched_tokens=budget, max_num_sequences=slots, **kw), model_runner=runner)
    return eng.generate(prompts, SamplingParams(greedy=True, max_tokens=new, ignore_eos=True))["token_ids"]


@pytest.mark.parametrize("name", ["mixed", "other"])
def test_greedy_generation_through_the_engine(name):
    """fp32: the engine's greedy ids are the oracle's; captured decode steps and small step budgets give the same ones."""
    runner, cfg, weights = make_runner(name, torch.float32)
    prompts = [tokens(60 + i, n, cfg["vocab"]) for i, n in enumerate([5, 40, 1, 23, 71, 2])]
    got = generate(runner, prompts, 12)
    for p, ids in zip(prompts, got):
        want, lead = greedy_reference(p, 12, weights, cfg)
        assert lead > 1e-3, "the case has a tie: choose other prompts"
        assert ids == want
    assert generate(runner, prompts, 12, budget=7) == got
    graphed, _, _ = make_runner(name, torch.float32, enforce_eager=False, max_model_length=256)
    for async_decode in (True, False):
        assert generate(graphed, prompts, 12, async_decode=async_decode) == got
    assert generate(graphed, prompts, 12, budget=9) == got


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_captured_decode(name):
    """Decoding until the rings have come round: replays of the captured step give the eager step's ids (fp32)."""
    eager, cfg, _ = make_runner(name, torch.float32)
    graphed, _, _ = make_runner(name, torch.float32, enforce_eager=False, max_model_length=256)
    prompts = [tokens(80 + i, n, cfg["vocab"]) for i, n in enumerate([3, 18, 31, 64, 19])]
    want, got = generate(eager, prompts, 100), generate(graphed, prompts, 100)
    same = sum(a == b for w, g in zip(want, got) for a, b in zip(w, g))
    assert same / 500 > 0.95 and all(w[:4] == g[:4] for w, g in zip(want, got))


def test_captured_decode_in_bf16():
    eager, cfg, _ = make_runner("mixed", torch.bfloat16)
    graphed, _, _ = make_runner("mixed", torch.bfloat16, enforce_eager=False, max_model_length=256)
    prompts = [tokens(80 + i, n, cfg["vocab"]) for i, n in enumerate([3, 18, 31, 64, 19])]
    want, got = generate(eager, prompts, 60), generate(graphed, prompts, 60)
    # greedy ids of a model with random weights part after a near-tie: the partings have to be rare
    same = sum(a == b for w, g in zip(want, got) for a, b in zip(w, g))
    assert same / 300 > 0.6 and all(w[:4] == g[:4] for w, g in zip(want, got))


def test_preempted_requests_start_over():
    """A pool too small for all of them: preempted requests are computed again and end with the same ids."""
    runner, cfg, _ = make_runner("other", torch.float32)
    prompts = [tokens(40 + i, n, cfg["vocab"]) for i, n in enumerate([30, 28, 45])]
    want = generate(runner, prompts, 40)
    small, _, _ = make_runner("other", torch.float32, max_cached_blocks=8)
    assert generate(small, prompts, 40) == want
    assert len(small.cache_manager.free_slots) == 4


def write_checkpoint(folder, cfg, weights):
    header, blobs, at = {}, [], 0
    for k, t in weights.items():
        raw = t.contiguous().view(torch.int16).numpy().tobytes()
        header[k] = {"dtype": "BF16", "shape": list(t.shape), "data_offsets": [at, at + len(raw)]}
        blobs.append(raw)
        at += len(raw)
    text = json.dumps(header).encode()
    (folder / "config.json").write_text(json.dumps(cfg))
    (folder / "model.safetensors").write_bytes(len(text).to_bytes(8, "little") + text + b"".join(blobs))


def test_trace_replay_and_command_line(tmp_path, capsys):
    """A checkpoint folder through the trace replay (files in the order of entries and places) and the generate command."""
    from minivllm_amd.__main__ import main
    from minivllm_amd.engine.replay import replay
    cfg = CONFIGS["mixed"]()
    weights = ref.random_weights(cfg, seed=3)
    write_checkpoint(tmp_path, cfg, weights)
    a, b = tokens(1, 50, cfg["vocab"]), tokens(2, 30, cfg["vocab"])
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:41], "want": [40, 3]}, {"id": "b", "tokens": b[:1], "want": [0]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[1:30], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[41:42], "want": [0]}], "end": ["b"]},
             {"step": 3, "entries": [{"id": "c", "tokens": b, "want": [29]}, {"id": "a", "tokens": a[42:], "want": [7]}], "end": ["a", "c"]}]
    said, out = [], tmp_path / "out"
    out.mkdir()
    replay(str(tmp_path), "float32", str(out), 128, [json.dumps(s) + "\n" for s in steps] + ["\n"], said.append)
    assert said == [f"done {i}" for i in range(4)] and sorted(p.name for p in out.iterdir()) == ["0.f32", "2.f32", "3.f32"]
    wa, wb = ref.forward(a, weights, cfg), ref.forward(b, weights, cfg)
    for n, rows in ((0, [wa[40], wa[3], wb[0]]), (2, [wa[41]]), (3, [wb[29], wa[49]])):
        got = torch.from_numpy(np.fromfile(out / f"{n}.f32", dtype="<f4")).view(len(rows), -1)
        check_rows(got, torch.stack(rows), torch.float32, n)
    capsys.readouterr()
    main(["generate", "--model", str(tmp_path), "--dtype", "float32", "--prompt", " ".join(map(str, b[:9])), "--max-tokens", "6", "--greedy"])
    ids = json.loads(capsys.readouterr().out.strip().splitlines()[-1])["token_ids"]
    want, lead = greedy_reference(b[:9], 6, weights, cfg)
    assert lead > 1e-3 and ids == [want]
