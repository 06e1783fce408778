"""Lenuzen on the GPU: every mechanism against the plain oracle, and the model through its cache, batches and engine."""
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
from minivllm_amd.layers.basic import Linear, rotary_pair_table
from minivllm_amd.layers.fused import embed_rows, gelu_tanh, head_rope_store, linear_small_m, post_norm
from minivllm_amd.layers.mixers import TalkingAttention, UnitHeadAttention
from minivllm_amd.layers.talk import talk_decode, talk_decode_workspace_bytes, talk_prefill
from minivllm_amd.layers.window import window_decode, window_decode_workspace_bytes, window_prefill
from minivllm_amd.models.lenuzen import LenuzenForCausalLM, engine_config
from minivllm_amd.sampling_parameters import SamplingParams
from lenuzen_cases import CONFIGS, STEEP, YARN, config, talk_layer, unit_layer
from oracle import lenuzen_oracle as ref
from sokevik_cases import Driver, manager, tokens

pytestmark = pytest.mark.gpu
DEV = torch.device("cuda:0")
DTYPES = [torch.float32, torch.bfloat16]
LOG2E = math.log2(math.e)


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


def on(t):
    return t.to(DEV)


def inside(t, left=8, right=16):
    """The same values as a view of wider rows, as a slice of a projection is; NaN around them."""
    wide = torch.full((t.shape[0], left + t[0].numel() + right), float("nan"), dtype=t.dtype, device=DEV)
    view = wide[:, left:left + t[0].numel()]
    view.copy_(t.flatten(1))
    return view.unflatten(-1, t.shape[1:])


def prefix_sums(lens):
    return torch.tensor([0, *np.cumsum(lens)], dtype=torch.int32)


# ---- rows: norms, rotation, gelu, the residual ----
def turn(x, pos, rot, interleaved):
    """The oracle's rotation of rows at any positions; the halves layout as the same pairs in another order."""
    dims, most = rot["dims"], int(pos.max()) + 1
    if not interleaved:
        order = torch.cat([torch.stack([torch.arange(dims // 2), torch.arange(dims // 2) + dims // 2], 1).view(-1), torch.arange(dims, x.shape[-1])])
        back = torch.empty_like(order)
        back[order] = torch.arange(len(order))
        return turn(x[..., order], pos, rot, True)[..., back]
    out = x.clone()
    for t in range(x.shape[0]):
        whole = torch.zeros(most, *x.shape[1:], dtype=x.dtype)
        whole[pos[t]] = x[t]
        out[t] = ref.rotate(whole, rot)[pos[t]]
    return out


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [3, 530])
@pytest.mark.parametrize("heads,groups,dim,vdim,size,dims,scaling", [(6, 2, 40, 24, 64, 28, YARN), (4, 1, 96, 128, 128, 96, STEEP), (5, 5, 16, 20, 32, 0, None),
                                                                      (2, 1, 150, 200, 256, 8, YARN), (33, 11, 8, 8, 32, 6, None)])
@pytest.mark.parametrize("form", ["unit", "rows", "halves"])
def test_norms_rotation_and_store(dtype, rows, heads, groups, dim, vdim, size, dims, scaling, form):
    """Unit heads behind the rotation into rows of key and value; norms over whole rows into separate caches; the other layout."""
    if form == "rows" and size > 128 and heads + 2 * groups > 64:
        pytest.skip("more heads than a workgroup takes")
    g, eps, interleaved = gen(rows + dim), 1e-2, form != "halves"
    x = rand(g, rows, heads * dim + groups * (dim + vdim), dtype=dtype)
    x[0, :dim] *= 1e-3                                                     # eps counts
    pos, factor = torch.randint(0, 60, (rows,), generator=g), rand(g, heads) + 1
    q, k, v = (t.double() for t in x.split([heads * dim, groups * dim, groups * vdim], 1))
    gains = {"gain_q": rand(g, heads * dim) + 1, "gain_k": rand(g, groups * dim) + 1}
    if form == "rows":
        q, k = ref.unit(q, eps) * gains["gain_q"].double(), ref.unit(k, eps) * gains["gain_k"].double()
    q, k, v = q.view(rows, heads, dim), k.view(rows, groups, dim), v.view(rows, groups, vdim)
    rot = {"base": 40.0, "dims": dims, "scaling": scaling}
    if dims:
        seen = torch.cat([turn(t[:40], pos[:40], rot, interleaved) for t in (q, k)], 1)      # the plain rotation is slow: the first rows
        rows_checked = len(seen)
    else:
        seen, rows_checked = torch.cat([q, k], 1), rows
    q, k, v = seen[:, :heads], seen[:, heads:], v[:rows_checked]
    if form != "rows":
        q, k, v = ref.unit(q, eps), ref.unit(k, eps), ref.unit(v, eps)
    q = q * 0.3 * (factor.double()[:, None] if form != "rows" else 1)
    table = rotary_pair_table(40.0, dims, 64, scaling).to(DEV) if dims else None
    slots, keys = torch.randperm(rows + 30, generator=g)[:rows], torch.randperm(rows + 9, generator=g)[:rows]
    slots[1] = keys[2] = -1
    blocks, bound = -(-(rows + 30) // 16), tol(dtype, 2e-6, 4e-3)
    full = torch.zeros(rows_checked, groups, 2 * size, dtype=torch.float64)
    full[..., :dim], full[..., size:size + vdim] = k, v
    common = dict(eps=eps, q_scale=0.3, rot_table=table, interleaved=interleaved, slots=on(slots))
    if form == "rows":
        dst = torch.randperm(rows, generator=g).int()
        kc, vc = (torch.full((blocks, 16, groups, size), 7.0, dtype=dtype, device=DEV) for _ in range(2))
        got, gk, gv = head_rope_store(inside(x), on(pos), heads, groups, dim, vdim, size, row_norm=True, k_cache=kc, v_cache=vc, dst_row=on(dst),
                                      **{n: on(t) for n, t in gains.items()}, **common)
        got, gk, gv = (t[on(dst.long())][:rows_checked] for t in (got, gk, gv))
        assert rel(torch.cat([gk, gv], -1), full) < bound
        cached = torch.cat([kc.view(-1, groups, size), vc.view(-1, groups, size)], -1)
    else:
        cache = torch.full((blocks, 16, groups, 2 * size), 7.0, dtype=dtype, device=DEV)
        packed = torch.full((rows + 9, groups, 2 * size), 7.0, dtype=dtype, device=DEV)
        got = head_rope_store(inside(x), on(pos), heads, groups, dim, vdim, size, unit_qk=True, unit_v=True, head_scale=on(factor), kv_cache=cache, kv_out=packed,
                              kv_rows=on(keys), **common)[:rows_checked]
        kept = (keys[:rows_checked] >= 0).nonzero()[:, 0]
        assert rel(packed[on(keys[kept])], full[kept]) < bound and int((packed == 7).all(-1).all(-1).sum()) == 10
        cached = cache.view(-1, groups, 2 * size)
    assert rel(got[..., :dim], q) < bound and row_rel(got[..., :dim], q) < 4 * bound and not got[..., dim:].any()
    live = (slots[:rows_checked] >= 0).nonzero()[:, 0]
    assert rel(cached[on(slots[live])], full[live]) < bound
    assert int((cached == 7).all(-1).all(-1).sum()) == blocks * 16 - rows + 1


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [1, 37, 600])
@pytest.mark.parametrize("width", [80, 97, 1028, 3000])
@pytest.mark.parametrize("centred", [True, False])
def test_post_norm(dtype, rows, width, centred):
    """Rows far from zero on average, eps that counts, the residual kept or not, padding, the final norm."""
    g, eps, padded = gen(rows + width), 3e-2, -(-width // 64) * 64
    x, y = rand(g, rows, width, scale=2.0), (rand(g, rows, width) * rand(g, rows, 1).abs() * 0.3 + 5.0 * rand(g, rows, 1)).to(dtype)
    w, final = rand(g, width), rand(g, width)
    norm = ref.centred_norm if centred else (lambda v, w, eps: ref.unit(v, eps) * w)
    want = x.double() + norm(y.double(), w.double(), eps)
    mine = on(x)
    h, new = post_norm(mine, inside(y), on(w), eps, centred, padded=padded)
    assert new is mine and rel(new, want) < 2e-6 and rel(h[:, :width], want) < tol(dtype, 2e-6, 3e-3) and not h[:, width:].any()
    mine = on(x)
    h, _ = post_norm(mine, on(y), on(w), eps, centred, final_gain=on(final), want_x=False)
    assert torch.equal(mine.cpu(), x) and h.shape == (rows, width) and rel(h, norm(want, final.double(), eps)) < tol(dtype, 3e-6, 3e-3)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [80, 63, 1028])
def test_embedding_rows(dtype, width):
    embed, toks = rand(gen(1), 50, width, dtype=dtype), torch.randint(0, 50, (33,), generator=gen(2))
    h, x = embed_rows(on(toks), on(embed), 1.7, padded=1088)
    want = embed.double()[toks] * 1.7
    assert rel(x, want) < 1e-6 and rel(h[:, :width], want) < tol(dtype, 1e-6, 3e-3) and not h[:, width:].any() and h.shape[1] == 1088


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width", [(1, 16), (37, 40), (600, 1024)])
def test_gelu(dtype, rows, width):
    x = rand(gen(width), rows, width, dtype=dtype, scale=3.0)
    x[0, :4] = torch.tensor([0.0, -30.0, 30.0, -1e4])
    want = ref.gelu_tanh(x.double())
    out = torch.zeros(rows, width + 24, dtype=dtype, device=DEV)
    gelu_tanh(inside(x), out[:, 8:8 + width])
    assert rel(out[:, 8:8 + width], want) < tol(dtype, 1e-6, 4e-3) and not out[:, :8].any() and not out[:, 8 + width:].any()
    mine = on(x)
    assert gelu_tanh(mine, out=mine) is mine and torch.equal(mine, out[:, 8:8 + width])


@pytest.mark.parametrize("rows", [1, 17, 64, 200])
def test_linear_with_gelu(rows):
    """The small-batch product's epilogue and the separate launch behind the library's product."""
    g = gen(rows)
    layer = Linear(512, 272, bias=True, small_rows=64)
    layer.weight.data, layer.bias.data = rand(g, 272, 512, dtype=torch.bfloat16, scale=512 ** -0.5).to(DEV), rand(g, 272, dtype=torch.bfloat16).to(DEV)
    x = rand(g, rows, 512, dtype=torch.bfloat16)
    z = x.double() @ layer.weight.detach().double().cpu().T + layer.bias.detach().double().cpu()
    with torch.inference_mode():
        assert rel(layer(on(x), gelu=True), ref.gelu_tanh(z)) < 8e-3 and rel(layer(on(x)), z) < 4e-3
        if rows <= 64:
            assert torch.equal(layer(on(x), gelu=True), linear_small_m(on(x), layer.weight, layer.bias, gelu=True))


# ---- windows over keys and values of their own ----
def window_reference(q, k, v, scale, window, gate=None):
    """Queries at the end of their keys; float64."""
    n, m = q.shape[0], k.shape[0]
    padded = torch.cat([torch.zeros(m - n, *q.shape[1:], dtype=torch.float64), q.double()])
    out = ref.values_out(ref.weights_of(ref.head_scores(padded, k.double(), scale), ref.sliding_mask(m, window)), v.double())[m - n:]
    return out if gate is None else out * torch.sigmoid(gate.double())[..., None]


WINDOWS = [0, 1, 31, 64, 130, 1000]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", WINDOWS)
@pytest.mark.parametrize("heads,groups,dim", [(4, 2, 32), (6, 2, 64), (5, 1, 96), (8, 2, 128), (2, 2, 192), (4, 1, 256), (3, 3, 320)])
def test_window_prefill_of_keys_and_values(dtype, window, heads, groups, dim):
    """Entries of any length behind pasts of any length, keys and values side by side, a gate per head and none."""
    g, lens, pasts = gen(dim + window), [70, 1, 200, 33], [0, 40, 17, 129]
    rows, keys = sum(lens), sum(lens) + sum(pasts)
    q, kv, gate = rand(g, rows, heads, dim, dtype=dtype, scale=2.0), rand(g, keys, groups, 2 * dim, dtype=dtype), rand(g, rows, heads, dtype=dtype)
    cu_q, cu_k, both = prefix_sums(lens), prefix_sums([a + b for a, b in zip(lens, pasts)]), on(kv)
    for gated in (True, False):
        out = torch.full((rows, heads, dim), float("nan"), dtype=dtype, device=DEV)
        window_prefill(out, inside(q), both[..., :dim], on(cu_q), on(cu_k), dim ** -0.5, window, v=both[..., dim:], gate=inside(gate, 3, 5) if gated else None)
        for e in range(len(lens)):
            a, b = slice(int(cu_q[e]), int(cu_q[e + 1])), slice(int(cu_k[e]), int(cu_k[e + 1]))
            want = window_reference(q[a], kv[b, :, :dim], kv[b, :, dim:], dim ** -0.5, window, gate[a] if gated else None)
            assert rel(out[a], want) < tol(dtype, 3e-6, 1.5e-2), e


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", [5, 64, 97])
def test_window_edges_in_prompts(dtype, window):
    """One key far above all others: seen by the queries up to window - 1 behind it, not by the next one; keys at the start of the
    entry, at tile borders and in the part that the past brings."""
    g, n, past, heads, dim = gen(window), 260, window + 20, 2, 64
    for at in (0, 1, 19, past - 1, past, past + 63, past + 64, past + 127):
        k, v = rand(g, past + n, heads, dim, dtype=dtype, scale=0.1), rand(g, past + n, heads, dim, dtype=dtype, scale=0.1)
        q = torch.ones(n, heads, dim, dtype=dtype)
        k[at], v[at] = 1.0, 5.0
        out = torch.empty(n, heads, dim, dtype=dtype, device=DEV)
        window_prefill(out, on(q), on(k), on(prefix_sums([n])), on(prefix_sums([past + n])), 0.5, window, v=on(v))
        seen = [0 <= past + i - at < window for i in range(n)]
        assert (((out.float().cpu().mean((1, 2)) - 5.0).abs() < 0.5) == torch.tensor(seen)).all(), at
        assert (out.double().cpu() - window_reference(q, k, v, 0.5, window)).abs().max() < tol(dtype, 1e-4, 0.15)


def ring_case(seed, lens, rows_of, heads, groups, dim, dtype, window, bs=16, scale=1.0):
    """Rings of entries that hold ``lens[e]`` tokens, of which the last ``rows_of[e]`` ask; rows of a key and its value, block
    tables shuffled, NaN elsewhere."""
    g, w = gen(seed), SlidingWindow(window)
    places = [min(n, w.places) if w.places else n for n in lens]
    need = [-(-p // bs) for p in places]
    perm, blocks = torch.randperm(sum(need) + 3, generator=g).tolist(), []
    for n in need:
        blocks.append([perm.pop() for _ in range(n)])
    tables = torch.full((len(lens), max(need) + 2), -1, dtype=torch.int32)
    cache = torch.full((sum(need) + 3, bs, groups, 2 * dim), float("nan"), dtype=dtype)
    rows = [rand(g, n, groups, 2 * dim, dtype=dtype) for n in lens]
    for e, n in enumerate(lens):
        tables[e, :need[e]] = torch.tensor(blocks[e], dtype=torch.int32)
        for b in blocks[e]:
            cache[b] = 0.0                                               # blocks are handed out with whatever finite numbers they hold
        for p in range(max(0, n - (w.places or n)), n):
            place = p % w.places if w.places else p
            cache[blocks[e][place // bs], place % bs] = rows[e][p]
    asked = [(e, lens[e] - r + i) for e, r in enumerate(rows_of) for i in range(r)]
    q = rand(g, len(asked), heads, dim, dtype=dtype, scale=scale)
    return w, q, rows, cache, tables, torch.tensor([e for e, _ in asked], dtype=torch.int32), asked


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", [0, 1, 20, 64, 300])
@pytest.mark.parametrize("heads,groups,dim", [(4, 2, 32), (6, 2, 64), (18, 1, 96), (8, 2, 128), (2, 2, 192), (35, 1, 256), (3, 3, 320), (70, 1, 128)])
def test_window_decode_of_keys_and_values(dtype, window, heads, groups, dim):
    """Single rows and rows of short entries, whose later rows are in the ring already; rings that have come round."""
    lens, rows_of = [1, 20, 21, 47, 50, 333, 700], [1, 1, 2, 31, 1, 17, 1]
    w, q, rows, cache, tables, entry, asked = ring_case(dim + window, lens, rows_of, heads, groups, dim, dtype, window, scale=2.0)
    gate, scale = rand(gen(3), len(asked), heads, dtype=dtype), dim ** -0.5
    for gated in (True, False):
        out = torch.full((len(asked), heads, dim), float("nan"), dtype=dtype, device=DEV)
        window_decode(out, inside(q), on(cache), on(tables), on(entry), on(torch.tensor([p + 1 for _, p in asked])), scale, window, w.places,
                      gate=inside(gate, 3, 5) if gated else None)
        want = torch.cat([window_reference(q[i:i + 1], rows[e][:p + 1, :, :dim], rows[e][:p + 1, :, dim:], scale, window, gate[i:i + 1] if gated else None)
                          for i, (e, p) in enumerate(asked)])
        assert rel(out, want) < tol(dtype, 3e-6, 1.5e-2) and row_rel(out, want) < tol(dtype, 2e-5, 6e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", [5, 33, 64])
def test_window_edges_while_decoding(dtype, window):
    """One key far above all others, decoded past until the ring has come round: seen for window - 1 tokens after its own."""
    heads, dim, n, bs, w = 2, 64, 3 * window + 60, 16, SlidingWindow(window)
    m = manager([w], 20, bs, 1)
    for at in (0, 1, window - 1, window, w.places - 1, w.places):
        s = Sequence([1] * n, block_size=bs)
        m.allocate(s)
        table = s.group_tables[0]
        cache, rows = torch.zeros(20, bs, 1, 2 * dim, dtype=dtype), rand(gen(at), n, 1, 2 * dim, dtype=dtype, scale=0.1)
        rows[at, :, :dim], rows[at, :, dim:] = 1.0, 5.0
        caches = []
        for p in range(n):
            place = p % w.places
            cache[table[place // bs], place % bs] = rows[p]
            caches.append(cache.clone())
        for p in range(max(at - 1, 0), min(at + window + 3, n)):
            out = torch.empty(1, heads, dim, dtype=dtype, device=DEV)
            window_decode(out, torch.ones(1, heads, dim, dtype=dtype, device=DEV), on(caches[p]), torch.tensor([table], dtype=torch.int32, device=DEV),
                          torch.zeros(1, dtype=torch.int32, device=DEV), torch.tensor([p + 1], device=DEV), 0.5, window, w.places)
            assert (abs(float(out.float().mean()) - 5.0) < 0.5) == (0 <= p - at < window), (at, p)
        m.deallocate(s)


def test_window_decode_in_shares():
    """Long rows are cut into shares that a second launch joins (gate included); a caller's workspace serves as well."""
    for dtype in DTYPES:
        w, q, rows, cache, tables, entry, asked = ring_case(1, [5000, 3, 2049], [1, 1, 1], 4, 2, 64, dtype, 4000)
        need = window_decode_workspace_bytes(3, 4, 2, 128, 64, tables.shape[1] * 16, dtype)
        assert need > 0
        gate = rand(gen(0), 3, 4, dtype=dtype)
        want = torch.cat([window_reference(q[i:i + 1], rows[e][..., :64], rows[e][..., 64:], 0.2, 4000, gate[i:i + 1]) for i, (e, _) in enumerate(asked)])
        for ws in (None, torch.empty(need, dtype=torch.uint8, device=DEV)):
            out = torch.empty(3, 4, 64, dtype=dtype, device=DEV)
            window_decode(out, on(q), on(cache), on(tables), on(entry), torch.tensor([5000, 3, 2049], device=DEV), 0.2, 4000, w.places, gate=on(gate), workspace=ws)
            assert row_rel(out, want) < tol(dtype, 1e-5, 2e-2)


# ---- mixed heads ----
def talk_reference(q, k, v, talk, sinks=None):
    """Queries at the end of their keys, all of them seen up to the own one; scores in natural units; float64."""
    n, m = q.shape[0], k.shape[0]
    padded = torch.cat([torch.zeros(m - n, *q.shape[1:], dtype=torch.float64), q.double()])
    s = ref.mix_heads(ref.head_scores(padded, k.double(), 1.0), talk.double())[:, m - n:].masked_fill(~ref.chunk_mask(m, 0)[m - n:], -math.inf)
    p = torch.exp(s) / ((0 if sinks is None else torch.exp(sinks.double())[:, None, None]) + torch.exp(s).sum(-1, keepdim=True))
    return ref.values_out(p, v.double())


def talk_matrix(g, heads):
    """Not symmetric, not triangular, numbers that bf16 holds; some heads count little in their own."""
    return (torch.eye(heads) * 0.6 + rand(g, heads, heads, scale=0.8 * heads ** -0.5)).bfloat16().float()


def scaled(q, dtype):
    """Queries as the kernels take them (log2 e inside), and what they stand for."""
    mine = (q * LOG2E).to(dtype)
    return mine, mine.double() / LOG2E


# (heads, kv heads, dim): pieces of four heads and fewer, one tile of heads and more, the sizes without a tiled kernel behind
TALK = [(8, 2, 32), (6, 2, 64), (32, 8, 128), (5, 5, 96), (16, 4, 128), (20, 1, 64), (12, 4, 32), (1, 1, 32), (24, 3, 96), (33, 3, 32), (28, 7, 64), (2, 1, 128),
        (40, 4, 64), (64, 2, 32), (7, 1, 160), (36, 12, 16), (3, 3, 200)]
TALK_IDS = ["x".join(map(str, t)) for t in TALK]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,groups,dim", TALK, ids=TALK_IDS)
def test_talk_prefill(dtype, heads, groups, dim):
    """Packed pieces of any length, with and without a sink, rows of the result in another order."""
    g, lens = gen(heads + dim), [70, 1, 129, 33, 16, 2]
    rows = sum(lens)
    q, want_q = scaled(rand(g, rows, heads, dim, scale=2.0 * dim ** -0.5), dtype)
    k, v, talk, sinks = rand(g, rows, groups, dim, dtype=dtype), rand(g, rows, groups, dim, dtype=dtype), talk_matrix(g, heads), rand(g, heads)
    cu, order = prefix_sums(lens), torch.randperm(rows, generator=g).int()
    for s, o in ((sinks, order), (torch.zeros(heads), None), (None, None)):
        out = torch.full((rows, heads, dim), float("nan"), dtype=dtype, device=DEV)
        talk_prefill(out, on(q), on(k), on(v), on(talk), on(cu), sinks=None if s is None else on(s), out_rows=None if o is None else on(o))
        got = out.cpu() if o is None else out.cpu()[o.long()]
        for e in range(len(lens)):
            a = slice(int(cu[e]), int(cu[e + 1]))
            assert rel(got[a], talk_reference(want_q[a], k[a], v[a], talk, s)) < tol(dtype, 3e-6, 1.5e-2), (e, s is None)


def paged(g, keys, bs, spare=2):
    """Keys of entries in shuffled blocks (finite numbers elsewhere): cache and tables."""
    need = [-(-t.shape[0] // bs) for t in keys]
    perm = torch.randperm(sum(need) + spare, generator=g).tolist()
    cache = rand(g, sum(need) + spare, bs, *keys[0].shape[1:], dtype=keys[0].dtype, scale=3.0)
    tables = torch.full((len(keys), max(need) + 1), -1, dtype=torch.int32)
    for e, t in enumerate(keys):
        for b in range(need[e]):
            tables[e, b] = perm.pop()
            part = t[b * bs:(b + 1) * bs]
            cache[tables[e, b], :len(part)] = part
    return cache, tables


def paged_pair(seed, k, v, bs):
    return (*paged(gen(seed), k, bs), paged(gen(seed), v, bs)[0])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("bs", [16, 48])
@pytest.mark.parametrize("heads,groups,dim", TALK, ids=TALK_IDS)
def test_talk_prefill_behind_a_past(dtype, bs, heads, groups, dim):
    """Pieces behind cached keys in a paged cache, and the same keys packed."""
    g, lens, pasts = gen(heads * dim), [40, 2, 17, 1, 65], [100, 31, 15, 64, 1]
    rows = sum(lens)
    q, want_q = scaled(rand(g, rows, heads, dim, scale=2.0 * dim ** -0.5), dtype)
    k, v = ([rand(g, a + b, groups, dim, dtype=dtype) for a, b in zip(lens, pasts)] for _ in range(2))
    talk, sinks, cu_q, cu_k = talk_matrix(g, heads), rand(g, heads), prefix_sums(lens), prefix_sums([a + b for a, b in zip(lens, pasts)])
    kc, tables, vc = paged_pair(5, k, v, bs)
    outs = [torch.full((rows, heads, dim), float("nan"), dtype=dtype, device=DEV) for _ in range(2)]
    talk_prefill(outs[0], on(q), on(kc), on(vc), on(talk), on(cu_q), on(cu_k), on(tables), on(sinks))
    talk_prefill(outs[1], on(q), on(torch.cat(k)), on(torch.cat(v)), on(talk), on(cu_q), on(cu_k), None, on(sinks))
    assert torch.equal(outs[0], outs[1])
    for e in range(len(lens)):
        a = slice(int(cu_q[e]), int(cu_q[e + 1]))
        assert rel(outs[0][a], talk_reference(want_q[a], k[e], v[e], talk, sinks)) < tol(dtype, 3e-6, 1.5e-2), e


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("bs", [16, 80])
@pytest.mark.parametrize("heads,groups,dim", TALK, ids=TALK_IDS)
def test_talk_decode(dtype, bs, heads, groups, dim):
    """Rows with one key and with many, a row without any; every kind of head; results beside others' columns."""
    g, lens = gen(heads * dim + bs), [1, 2, 31, 32, 33, 64, 65, 200, 517]
    n = len(lens)
    q, want_q = scaled(rand(g, n + 1, heads, dim, scale=2.0 * dim ** -0.5), dtype)
    k, v = ([rand(g, a, groups, dim, dtype=dtype) for a in lens] for _ in range(2))
    talk, sinks = talk_matrix(g, heads), rand(g, heads)
    kc, tables, vc = paged_pair(6, k, v, bs)
    tables, lengths = torch.cat([tables, torch.full_like(tables[:1], -1)]), torch.tensor([*lens, 0])
    for s in (sinks, torch.zeros(heads), None):
        wide = torch.full((n + 1, heads * dim + 24), 3.0, dtype=dtype, device=DEV)
        out = wide[:, 8:8 + heads * dim].unflatten(-1, (heads, dim))
        talk_decode(out, on(q), on(kc), on(vc), on(tables), on(lengths), on(talk), None if s is None else on(s))
        want = torch.cat([talk_reference(want_q[i:i + 1], k[i], v[i], talk, s) for i in range(n)])
        assert rel(out[:n], want) < tol(dtype, 3e-6, 1.5e-2) and row_rel(out[:n], want) < tol(dtype, 2e-5, 6e-2)
        assert not out[n:].any() and bool((wide[:, :8] == 3).all() and (wide[:, 8 + heads * dim:] == 3).all())


def test_talk_decode_in_shares():
    """Long rows are cut into shares that a second launch joins (sinks included); a caller's workspace serves as well."""
    g, heads, groups, dim, lens = gen(1), 12, 4, 64, [3000, 3, 1025]
    q, want_q = scaled(rand(g, 3, heads, dim, scale=0.2), torch.bfloat16)
    k, v = ([rand(g, a, groups, dim, dtype=torch.bfloat16) for a in lens] for _ in range(2))
    talk, sinks = talk_matrix(g, heads), rand(g, heads) + 2
    kc, tables, vc = paged_pair(7, k, v, 16)
    need = talk_decode_workspace_bytes(3, heads, groups, dim, tables.shape[1] * 16, torch.bfloat16)
    assert need > 0 and talk_decode_workspace_bytes(3, heads, groups, dim, tables.shape[1] * 16, torch.float32) == 0
    want = torch.cat([talk_reference(want_q[i:i + 1], k[i], v[i], talk, sinks) for i in range(3)])
    for ws in (None, torch.empty(need, dtype=torch.uint8, device=DEV)):
        out = torch.empty(3, heads, dim, dtype=torch.bfloat16, device=DEV)
        talk_decode(out, on(q), on(kc), on(vc), on(tables), on(torch.tensor(lens)), on(talk), on(sinks), ws)
        assert row_rel(out, want) < 2e-2


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,groups,dim", [(8, 2, 64), (32, 8, 128), (6, 3, 32), (9, 1, 40)])
def test_one_key_that_one_head_asks_for(dtype, heads, groups, dim):
    """Only head ``g`` finds the key, only head ``h`` listens to it: h's result is that key's value, the others' a mean of all; in a
    prompt and decoded, with the key first, at tile borders and last.  Running maxima that move late are part of it."""
    n = 150
    for at, asks, hears in ((0, 0, heads - 1), (31, heads - 1, 0), (32, 1, 1), (97, heads // 2, heads // 2 - 1), (149, 2, 4)):
        k, v = torch.zeros(n, groups, dim, dtype=dtype), torch.zeros(n, groups, dim, dtype=dtype)
        q, talk = torch.zeros(1, heads, dim, dtype=dtype).expand(n, -1, -1).clone(), torch.zeros(heads, heads)
        q[:, asks, 3], k[at, asks * groups // heads, 3] = 8.0, 8.0
        v[at], talk[hears, asks] = 1.0, 0.5
        mine, _ = scaled(q, dtype)
        out = torch.empty(n, heads, dim, dtype=dtype, device=DEV)
        talk_prefill(out, on(mine), on(k), on(v), on(talk), on(prefix_sums([n])), sinks=torch.zeros(heads, device=DEV))
        kc, tables, vc = paged_pair(9, [k], [v], 16)
        last = torch.empty(n, heads, dim, dtype=dtype, device=DEV)
        talk_decode(last, on(mine), on(kc), on(vc), on(tables.expand(n, -1).contiguous()), torch.arange(1, n + 1, device=DEV), on(talk), torch.zeros(heads, device=DEV))
        for got in (out, last):
            got = got.float().cpu().mean(-1)
            assert not got[:at].any()
            for p in range(at, n):
                plain = torch.full((heads,), 1 / (p + 2))                  # the sink is one more
                plain[hears] = 1.0
                assert (got[p] - plain).abs().max() < 8e-3, (at, p)


def test_scores_that_grow_along_the_keys():
    """Every tile's scores pass the ones before by far more than a running maximum may lag behind, then fall again."""
    for dtype in DTYPES:
        g, heads, groups, dim, n = gen(1), 8, 2, 64, 260
        rise = torch.cat([torch.linspace(-40, 60, 170), torch.linspace(60, -80, 90)])
        q = rand(g, n, heads, dim, scale=0.05)
        k, v, talk = rand(g, n, groups, dim), rand(g, n, groups, dim, dtype=dtype), talk_matrix(g, heads).abs()
        q[..., 0], k[..., 0] = 1.0, rise[:, None]
        (q, want_q), k = scaled(q, dtype), k.to(dtype)
        out = torch.empty(n, heads, dim, dtype=dtype, device=DEV)
        talk_prefill(out, on(q), on(k), on(v), on(talk), on(prefix_sums([n])))
        assert rel(out, talk_reference(want_q, k, v, talk)) < tol(dtype, 1e-4, 2e-2)


def test_many_pieces_in_one_call():
    """More pieces than a wave has lanes: the other order of work items."""
    g, heads, groups, dim = gen(1), 8, 2, 32
    lens = [1 + i % 41 for i in range(70)]
    rows, cu = sum(lens), prefix_sums(lens)
    q, want_q = scaled(rand(g, rows, heads, dim, scale=0.4), torch.bfloat16)
    k, v, talk = rand(g, rows, groups, dim, dtype=torch.bfloat16), rand(g, rows, groups, dim, dtype=torch.bfloat16), talk_matrix(g, heads)
    out = torch.full((rows, heads, dim), float("nan"), dtype=torch.bfloat16, device=DEV)
    talk_prefill(out, on(q), on(k), on(v), on(talk), on(cu))
    want = torch.cat([talk_reference(*(t[int(a):int(b)] for t in (want_q, k, v)), talk) for a, b in zip(cu, cu[1:])])
    assert rel(out, want) < 1.5e-2 and row_rel(out, want) < 6e-2


# ---- mixers as layers ----
def mixer_case(entry, width, dtype, seed=0, peak=1.0, eps=1e-3):
    """The mixer as a function of (h, step), and the oracle's; ``peak`` sharpens the scores."""
    w = {k[len("l0.mix."):]: t for k, t in ref.random_weights(config([entry], width=width), seed).items() if k.startswith("l0.mix.")}
    for n in ("temp", "q.norm"):
        if n in w:
            w[n] = w[n] * peak
    m, inputs = entry["mixer"], -(-width // 64) * 64
    sizes = (m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"], 0)
    if entry["type"] == "attention":
        view = SlidingWindow(m["mask"]["size"])
        mixer = UnitHeadAttention(inputs, *sizes, view, 16, dtype, eps, small_rows=64)
    else:
        view = m["mask"]["size"]
        mixer = TalkingAttention(inputs, *sizes, 16, dtype, eps, sink=0.0, small_rows=64)
    if m["rot"]["dims"]:
        mixer.table = rotary_pair_table(m["rot"]["base"], m["rot"]["dims"], 2048, m["rot"].get("scaling")).to(DEV)
    mixer.load(lambda n: w[n], lambda t: t.to(DEV, dtype).contiguous(), inputs)
    mixer.allocate(24, DEV)
    wd = {k: t.double() for k, t in w.items()}

    @torch.inference_mode()
    def run(h, step):
        return mixer(torch.nn.functional.pad(h, (0, inputs - width)).to(DEV), step).cpu()

    plain = ref.attention if entry["type"] == "attention" else ref.talking_attention
    return run, lambda h: plain(h, wd, "", m, eps), view


MIXERS = {
    "unit": unit_layer(), "one": unit_layer(heads=5, kv_heads=1, dim=128, vdim=100, window=150, rot=128), "wide": unit_layer(heads=2, kv_heads=2, dim=200, vdim=300, window=64),
    "short": unit_layer(heads=4, kv_heads=4, dim=16, vdim=16, window=3, rot=4, scaling=None, scale=-0.8), "all": unit_layer(heads=8, kv_heads=2, dim=48, vdim=64, window=0),
    "talk": talk_layer(), "heads": talk_layer(heads=20, kv_heads=5, dim=64, vdim=64, chunk=100, rot=64), "none": talk_layer(heads=4, kv_heads=1, dim=96, vdim=70, chunk=0, rot=40, scaling=None),
    "chunk": talk_layer(heads=8, kv_heads=2, dim=128, vdim=128, chunk=64, rot=20), "pairs": talk_layer(heads=2, kv_heads=1, dim=30, vdim=20, chunk=2, rot=0),
    "large": talk_layer(heads=3, kv_heads=3, dim=150, vdim=130, chunk=70, rot=100, scale=0.1), "many": talk_layer(heads=40, kv_heads=10, dim=24, vdim=24, chunk=33)}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(MIXERS))
@pytest.mark.parametrize("cuts", [[230], [1] * 40 + [2] * 95, [31, 32, 33, 1, 2, 70, 31, 30], [150, 80], [17, 183, 30]], ids=["whole", "twos", "odd", "halves", "middle"])
def test_mixers_in_portions(dtype, name, cuts):
    """Peaked scores: decoded rows, short portions, long ones with and without a past give the whole sequence's rows."""
    width, rows = 96, sum(cuts)
    run, plain, view = mixer_case(MIXERS[name], width, dtype, peak=2.0)
    h = rand(gen(8), rows, width, dtype=dtype)
    m = manager([view], 24, 16, 2)
    s = Sequence([1] * rows, block_size=16)
    m.allocate(s)
    got, at = [], 0
    for n in cuts:
        s.num_computed_tokens, s.num_scheduled_tokens = at, n
        got.append(run(h[at:at + n], ragged_step([s], [view], 16, DEV)))
        at += n
    got, want = torch.cat(got), plain(h.double())
    assert rel(got, want) < tol(dtype, 5e-6, 2.5e-2) and row_rel(got, want) < tol(dtype, 1e-4, 0.15)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["unit", "one", "talk", "heads", "large"])
def test_mixers_in_batches(dtype, name):
    """Unequal entries in one step, in every form at once, rings, chunks and blocks shuffled and used again."""
    width = 80
    run, plain, view = mixer_case(MIXERS[name], width, dtype, peak=2.0)
    m, rng = manager([view], 24, 16, 4), random.Random(1)
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
            step = ragged_step([seqs[k] for k in live], [view], 16, DEV)
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


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,groups,dim", [(4, 2, 64), (3, 1, 40)])
@pytest.mark.parametrize("chunk", [24, 32])
def test_chunk_edges(dtype, heads, groups, dim, chunk):
    """One token's key far above all others: its value reaches the later tokens of its own chunk and no other, whatever portions
    the sequence comes in; tokens at both ends of chunks, of pages and in the middle."""
    n, width = 3 * chunk + 9, 64
    entry = talk_layer(heads=heads, kv_heads=groups, dim=dim, vdim=dim, chunk=chunk, rot=0, scale=1.0)
    m = entry["mixer"]
    mixer = TalkingAttention(width, heads, groups, dim, dim, 1.0, 0, 16, dtype, 1e-6, sink=0.0, small_rows=64)
    w = {"q": torch.zeros(heads * dim, width), "k": torch.zeros(groups * dim, width), "v": torch.zeros(groups * dim, width), "o": torch.zeros(width, heads * dim),
         "q.norm": torch.ones(heads * dim), "k.norm": torch.ones(groups * dim), "talk": torch.eye(heads)}
    w["q"][::dim, 0] = 1.0                                                 # every query: its head's first channel
    w["k"][::dim, 1] = 1.0                                                 # the marked key: the same; the others' second channel
    w["k"][1::dim, 0] = 1e-3
    w["v"][:, 1], w["o"][0] = 1.0, 1.0
    mixer.load(lambda name: w[name], lambda t: t.to(DEV, dtype).contiguous(), width)
    mixer.allocate(24, DEV)
    cache = manager([chunk], 24, 16, 2)
    for at in (0, 1, 15, chunk - 1, chunk, chunk + 1, 2 * chunk - 1, 2 * chunk):
        h = torch.zeros(n, width, dtype=dtype)
        h[:, 0], h[at, 1] = 1.0, 1.0
        reach = torch.tensor([at <= p and p // chunk == at // chunk for p in range(n)])
        assert torch.equal(ref.talking_attention(h.double(), {k: t.double() for k, t in w.items()}, "", m, 1e-6)[:, 0] > 1.0, reach)
        for cuts in ([n], [2], [1], [chunk - 1, chunk + 2], [5, 40, 1, 33]):
            s = Sequence([1] * n, block_size=16)
            cache.allocate(s)
            got, p, i = [], 0, 0
            while p < n:
                size = min(cuts[min(i, len(cuts) - 1)], n - p)
                s.num_computed_tokens, s.num_scheduled_tokens = p, size
                with torch.inference_mode():
                    got.append(mixer(on(h[p:p + size]), ragged_step([s], [chunk], 16, DEV)).cpu())
                p, i = p + size, i + 1
            cache.deallocate(s)
            assert torch.equal(torch.cat(got)[:, 0].float() > 1.0, reach), (at, cuts)


# ---- the model ----
_runners: dict = {}


def make_runner(name, dtype, **extra):
    key = (name, dtype, tuple(sorted(extra.items())))
    if key not in _runners:
        cfg = CONFIGS[name]()
        full = engine_config({**cfg, "dtype": "fp32" if dtype == torch.float32 else "bf16", "block_size": 16, "max_cached_blocks": 40,
                              "max_num_sequences": 4, "max_position": 1024, **extra, "enforce_eager": True})
        runner = HybridModelRunner(full, LenuzenForCausalLM)
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


MODEL_TOL = {torch.float32: 2e-4, torch.bfloat16: 0.15}      # a row's logits error over the logits' spread


def row_errors(got, want):
    d = got.double() - want
    return (d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt() / want.std()


def check_rows(got, want, dtype, *what):
    err = row_errors(got, want)
    assert err.max() < MODEL_TOL[dtype] and err.median() < MODEL_TOL[dtype] / 4, (*what, int(err.argmax()), float(err.max()), float(err.median()))


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
    """bf16: the same tokens whole, in portions, token by token and beside others differ by rounding only."""
    runner, cfg, _ = make_runner("mixed", torch.bfloat16)
    toks = tokens(3, 120, cfg["vocab"])
    base = Driver(runner).run_alone("a", toks, [120]).double()
    others = [Driver(runner).run_alone("a", toks, sizes) for sizes in ([1], [2], [33], [7, 60])]
    drv = Driver(runner)
    for at in range(0, 120, 40):
        drv.step({"x": tokens(50, 35, cfg["vocab"])[:35 - at // 4], "a": toks[at:at + 40], "y": tokens(51, 3, cfg["vocab"])[:1]}, ["x"])
    drv.step({"y": [1]}, ["y", "a"])
    for got in [*others, torch.cat(drv.logits["a"])]:
        assert row_errors(got, base).median() < 4e-2 and row_errors(got, base).max() < 0.15


def test_first_tokens_and_one_token_prompts():
    runner, cfg, weights = make_runner("mixed", torch.float32)
    want = oracle_logits(7, 170, cfg, weights)
    for n in (1, 2, 3, 4):
        check_rows(Driver(runner).run_alone("x", tokens(7, 170, cfg["vocab"])[:n], [n]), want[:n], torch.float32, n)


def test_long_decoding():
    """A few hundred decoded tokens: every ring comes round several times, every chunk is started anew."""
    runner, cfg, weights = make_runner("mixed", torch.float32)
    got = Driver(runner).run_alone("x", tokens(31, 330, cfg["vocab"]), [5, 1])
    check_rows(got, oracle_logits(31, 330, cfg, weights), torch.float32)


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
