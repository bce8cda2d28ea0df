"""Kokuvik on the GPU against the plain CPU restatement (oracle/kokuvik.py): each mechanism's kernels alone, then whole models built
from small random checkpoints through the loader, the ragged runner, the paged state cache, the generation engine, the command
line and the trace replay.  float32 runs are held to rounding error; bfloat16 runs to the rounding of their activations.  Where
random weights would hide a fault (a kept first key far back, a window's edge, a sink, a write long ago), one key is made to
dominate."""

import json
import os
import subprocess
import sys

import pytest
import torch

from tests import _kokuvik as T
from tests import _layered as L
from tests.test_layered_gpu import _close, _feed, _step

pytestmark = pytest.mark.gpu
DEV = "cuda"
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
F64 = torch.float64
TOL = {torch.float32: 2e-5, torch.bfloat16: 2e-2}
DTYPES = [torch.float32, torch.bfloat16]


def d(t):
    return t.detach().cpu().to(F64)


# ------------------------------------------------------------------------------------------------------------------- #
# retention alone
# ------------------------------------------------------------------------------------------------------------------- #
class _Retention:
    """A case of the retention kernels: random rows per sequence, the slots' states full of what an earlier owner left."""

    def __init__(self, dtype, heads, dk, dv, dims, decay, lens, base=50.0, pad=0, seed=0):
        from oracle import kokuvik as O

        torch.manual_seed(seed + dk * 7 + dv)
        self.dtype, self.heads, self.dk, self.dv, self.pairs, self.eps = dtype, heads, dk, dv, dims // 2, 1e-5
        self.qk, self.v, self.pad = heads * dk, heads * dv, pad
        self.decay = torch.tensor(decay, dtype=torch.float32)
        self.rows = {s: torch.randn(n, 2 * (self.qk + self.v) + pad).to(dtype) for s, n in lens.items()}
        self.freq = torch.tensor([base ** (-2.0 * i / dims) for i in range(self.pairs)], dtype=F64).float().to(DEV) if dims else None
        self.rot = {"dims": dims, "base": base}
        self.state = torch.full((4, heads, dk, dv), 3.0, device=DEV)
        self.O = O

    def want(self, s):
        n, O = self.rows[s].shape[0], self.O
        r = d(self.rows[s])
        q, k = r[:, :self.qk].view(n, self.heads, self.dk), r[:, self.qk:2 * self.qk].view(n, self.heads, self.dk)
        if self.pairs:
            pos = torch.arange(n)
            q, k = O.rotate_halves(q, pos, self.rot, torch.float32), O.rotate_halves(k, pos, self.rot, torch.float32)
        v = r[:, 2 * self.qk:2 * self.qk + self.v].view(n, self.heads, self.dv)
        o, S = O.retention_scan(q, k * self.dk ** -0.5, v, d(self.decay))
        g = r[:, 2 * self.qk + self.v:2 * (self.qk + self.v)]
        return O.rms_norm(o, None, self.eps).reshape(n, -1) * (g * torch.sigmoid(g)), S

    def run(self, plan):
        """``plan``: steps of ``(slot, first, count)``.  Returns the outputs per sequence; their place among wider rows is checked."""
        from lite_llama_amd.kernels.attention import rotation_table
        from lite_llama_amd.kernels.recurrent import retention

        got = {s: [] for s in self.rows}
        for entries in plan:
            step = _step([(s, f, c, 0) for s, f, c in entries])
            rows = torch.cat([self.rows[s][f:f + c] for s, f, c in entries]).to(DEV)
            cols = lambda at, n: rows[:, at:at + n]   # noqa: E731
            wide = torch.full((rows.shape[0], self.v + 24), 2.0, dtype=self.dtype, device=DEV)
            table = rotation_table(step, self.freq, self.pairs) if self.pairs else None
            retention(cols(0, self.qk), cols(self.qk, self.qk), cols(2 * self.qk, self.v), self.heads, self.dk, self.dv, step, self.state,
                      decay=self.decay.to(DEV), gate=cols(2 * self.qk + self.v, self.v), eps=self.eps, k_scale=self.dk ** -0.5,
                      half=self.pairs, rot_table=table, out=wide[:, 8:8 + self.v])
            assert torch.all(wide[:, :8] == 2.0) and torch.all(wide[:, 8 + self.v:] == 2.0)
            at = 0
            for s, _, c in entries:
                got[s].append(wide[at:at + c, 8:8 + self.v].clone())
                at += c
        return {s: torch.cat(g) for s, g in got.items() if g}


HEADS = [(2, 64, 32, 64), (3, 16, 24, 8), (1, 128, 128, 128), (2, 8, 8, 0), (5, 10, 6, 4), (1, 1, 1, 0), (2, 9, 33, 8), (1, 256, 72, 128),
         (2, 200, 40, 16), (1, 24, 1100, 24)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,dk,dv,dims", HEADS)
def test_retention_over_starts_portions_and_decoded_tokens(dtype, heads, dk, dv, dims):
    """Portions of one and two tokens, of a chunk less one, a chunk, a chunk and one, several chunks; a start beside a portion and
    decoded tokens; stale states in every slot."""
    lens = {1: 140, 3: 47, 0: 5}
    case = _Retention(dtype, heads, dk, dv, dims, [1.0 - 0.3 / (1 + 3 * i) for i in range(heads)], lens)
    plan = [[(1, 0, 1)], [(1, 1, 2), (3, 0, 1)], [(1, 3, 31), (3, 1, 1)], [(1, 34, 1), (3, 2, 1)], [(1, 35, 32), (3, 3, 33), (0, 0, 5)],
            [(1, 67, 70), (3, 36, 10)], [(1, 137, 1), (3, 46, 1)], [(1, 138, 2)]]
    got = case.run(plan)
    for s in lens:
        want, state = case.want(s)
        _close(got[s], want, TOL[dtype])
        _close(case.state[s], state, 5e-6)
    assert torch.all(case.state[2] == 3.0)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("pad", [0, 3])     # (3: rows off every 16-byte border)
def test_retention_result_does_not_depend_on_the_cut_or_the_company(dtype, pad):
    lens = {0: 130, 1: 130, 2: 64}
    mk = lambda: _Retention(dtype, 2, 32, 48, 32, [0.9, 0.999], lens, pad=pad, seed=5)   # noqa: E731
    base = mk()
    whole = base.run([[(0, 0, 130)]])[0]
    for plan in ([[(0, i, 1)] for i in range(130)], [[(0, 2 * i, 2)] for i in range(65)], [[(0, 0, 33), (1, 0, 130)], [(2, 0, 64), (0, 33, 97)]],
                 [[(1, 0, 1), (0, 0, 5)]] + [[(0, 5 + 25 * i, 25), (1, 1 + i, 1)] for i in range(5)]):
        case = mk()
        got = case.run(plan)[0]
        _close(got, d(whole), 3e-6 if dtype == torch.float32 else 1.2e-2)
        _close(case.state[0], d(base.state[0]), 3e-6)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("at", [0, 1, 31, 32, 63, 64, 255, 256])
@pytest.mark.parametrize("decoded", [False, True])
def test_retention_reads_a_write_made_long_before_and_forgets_by_the_heads_decay(dtype, at, decoded):
    """One strong key at ``at`` (the first tokens, chunk and page edges); 400 tokens later its query brings the value back times
    decay^distance -- in a head that keeps everything, one that has lost half, one that has lost all."""
    decay = [1.0, 0.5 ** (1 / 400), 0.5]
    total = at + 420
    case = _Retention(dtype, 3, 16, 8, 16, decay, {1: total}, base=1e6)
    r = case.rows[1]
    u = torch.nn.functional.normalize(torch.randn(16) * torch.tensor([0.0] * 5 + [1.0] * 3).repeat(2), dim=0)   # (pairs that hardly turn)
    for h in range(3):
        r[:, 16 * h:16 * h + 16] *= 0.01
        r[:, 48 + 16 * h:64 + 16 * h] *= 0.01
        r[at, 48 + 16 * h:64 + 16 * h] = 40.0 * u.to(dtype)
        r[at + 400:, 16 * h:16 * h + 16] += 2.0 * u.to(dtype)
    cut = at + 395 if decoded else at + 407
    plan = [[(1, 0, cut)]] + ([[(1, cut + i, 1)] for i in range(total - cut)] if decoded else [[(1, cut, total - cut)]])
    got = case.run(plan)[1]
    want, _ = case.want(1)
    _close(got, want, 1e-4 if dtype == torch.float32 else 2e-2)
    q, k, v = (d(r[:, a:a + n]) for a, n in ((0, 48), (48, 48), (96, 24)))
    z = d(r[:, 120:])
    same = lambda h: torch.nn.functional.cosine_similarity(d(got)[at + 401:, 8 * h:8 * h + 8] / (z * torch.sigmoid(z))[at + 401:, 8 * h:8 * h + 8],   # noqa: E731
                                                           v[at, 8 * h:8 * h + 8].expand(total - at - 401, 8)).min()
    assert same(0) > 0.9 and same(1) > 0.8 and same(2) < 0.8


def test_retention_decays_of_one_and_near_zero_and_a_long_run():
    case = _Retention(torch.float32, 4, 16, 16, 16, [1.0, 1.0 - 2.0 ** -20, 1e-6, 0.0], {2: 1500})
    got = case.run([[(2, 0, 1)], [(2, 1, 700)], [(2, 701, 799)]])[2]
    want, state = case.want(2)
    _close(got, want, 5e-5)
    _close(case.state[2], state, 1e-5)


def test_retention_wrapper_refuses_what_the_kernels_would_misread():
    from lite_llama_amd.kernels.recurrent import retention

    step = _step([(0, 0, 3, 0)])
    rows = torch.randn(3, 16, device=DEV)
    st, dec = torch.zeros(1, 2, 8, 8, device=DEV), torch.ones(2, device=DEV)
    ok = dict(decay=dec, gate=rows, eps=1e-5)
    retention(rows, rows, rows, 2, 8, 8, step, st, **ok)
    for kw in (dict(decay=dec.half()), dict(decay=dec[:1]), dict(gate=rows[:2]), dict(half=4), dict(half=5, rot_table=torch.zeros(3, 16, device=DEV)),
               dict(half=4, rot_table=torch.zeros(2, 8, device=DEV)), dict(out=torch.zeros(3, 12, device=DEV))):
        with pytest.raises(ValueError):
            retention(rows, rows, rows, 2, 8, 8, step, st, **dict(ok, **kw))
    with pytest.raises(ValueError):
        retention(rows, rows, rows, 2, 8, 8, step, st.half(), **ok)
    with pytest.raises(ValueError):
        retention(torch.randn(3, 600, device=DEV), torch.randn(3, 600, device=DEV), rows, 2, 300, 8, step, torch.zeros(1, 2, 300, 8, device=DEV), **ok)


# ------------------------------------------------------------------------------------------------------------------- #
# rotation of an attention layer's projected rows
# ------------------------------------------------------------------------------------------------------------------- #
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,kv_heads,dk,dv,dims", [(4, 2, 16, 8, 8), (3, 1, 12, 10, 6), (2, 1, 64, 40, 64), (1, 1, 2, 1, 2)])
def test_rotation_of_pairs_over_all_bands_with_and_without_keys(dtype, heads, kv_heads, dk, dv, dims):
    """Positions from 0 to beyond 4000; a layer that borrows its keys rotates its queries alone and writes no cache."""
    from lite_llama_amd.kernels.attention import conv_rope_cache
    from lite_llama_amd.model_layers import RotarySpec
    from oracle import kokuvik as O

    torch.manual_seed(dk)
    rot = T.rot(dims, base=1000.0, original=300, factor=8.0, low=1.0, high=4.0)
    f = torch.tensor(RotarySpec.from_config(rot).table()[0], dtype=F64).float().to(DEV)
    table = torch.zeros(2, 5000, dtype=torch.int32)
    table[0, :3], table[1, 4093:4098] = torch.arange(3, dtype=torch.int32), torch.arange(3, 8, dtype=torch.int32)
    step = _step([(0, 0, 3, 0), (1, 4093, 5, 0)], table)
    pos = torch.tensor([0, 1, 2, 4093, 4094, 4095, 4096, 4097])
    rows = torch.randn(8, (heads + kv_heads) * dk + kv_heads * dv + 9, device=DEV).to(dtype)
    kc, vc = torch.zeros(9, kv_heads, dk, device=DEV, dtype=dtype), torch.zeros(9, kv_heads, dv, device=DEV, dtype=dtype)
    q = conv_rope_cache(rows, heads, kv_heads, dk, dv, step, kc, vc, freq=f, pairs=dims // 2)
    qn, kn = heads * dk, kv_heads * dk
    tol = 2e-6 if dtype == torch.float32 else 1e-2
    want = O.rotate_interleaved(d(rows[:, :qn]).view(8, heads, dk), pos, rot, torch.float32)
    _close(q, want, tol)
    _close(kc[:8], O.rotate_interleaved(d(rows[:, qn:qn + kn]).view(8, kv_heads, dk), pos, rot, torch.float32), tol)
    _close(vc[:8], d(rows[:, qn + kn:qn + kn + kv_heads * dv]).view(8, kv_heads, dv), tol)
    assert torch.count_nonzero(kc[8]) == 0 and torch.count_nonzero(vc[8]) == 0
    alone = conv_rope_cache(rows, heads, 0, dk, dv, step, None, None, freq=f, pairs=dims // 2)
    assert torch.equal(alone, q)


# ------------------------------------------------------------------------------------------------------------------- #
# attention alone: window + kept keys, a learned sink, a gate per head
# ------------------------------------------------------------------------------------------------------------------- #
def _attention_case(dtype, heads, kv_heads, dk, dv, total, plan, window, keep, hot=None, scale=0.3, sink=0.0, gate=True):
    """Queries against a paged cache through the attention kernels, fed by ``plan`` (steps of ``(slot, first, count)``); returns (got,
    want) of the slot-1 sequence.  ``hot``: one key whose score towers over the rest for every query that may see it; ``sink``: a
    number around which the heads' sinks lie."""
    from lite_llama_amd.kernels.attention import ragged_attention
    from oracle import kokuvik as O

    torch.manual_seed(total + heads + keep)
    q, k, v = torch.randn(total, heads, dk), torch.randn(total, kv_heads, dk), torch.randn(total, kv_heads, dv)
    if hot is not None:
        u = torch.nn.functional.normalize(torch.randn(dk), dim=0)
        k[hot] = 9.0 * u
        q = q + 9.0 * u
    q, k, v = q.to(dtype), k.to(dtype), v.to(dtype)
    sinks = (sink + 0.5 * torch.randn(heads)).to(dtype)
    z = (1.5 * torch.randn(total, heads + 5)).to(dtype)      # gate logits: a column range of wider rows
    rows_total = 2 * total + 64
    table = torch.randperm(rows_total)[:2 * total].view(2, total).to(torch.int32).to(DEV)
    kc, vc = torch.randn(rows_total, kv_heads, dk).to(dtype).to(DEV), torch.randn(rows_total, kv_heads, dv).to(dtype).to(DEV)
    kc[table[1].long()], vc[table[1].long()] = k.to(DEV), v.to(DEV)
    q0 = torch.randn(total, heads, dk).to(dtype)
    got = []
    for seqs in plan:
        step = _step([(s, f, c, 0) for s, f, c in seqs], table.cpu())
        qs = torch.cat([(q if s == 1 else q0)[f:f + c] for s, f, c in seqs]).to(DEV).contiguous()
        zs = torch.cat([z[f:f + c] for _, f, c in seqs]).to(DEV)
        wide = torch.full((qs.shape[0], heads * dv + 24), 3.0, dtype=dtype, device=DEV)
        ragged_attention(qs, kc, vc, scale, step, table, sink=sinks.to(DEV), window=window, keep_first=keep, out=wide[:, 8:8 + heads * dv],
                         head_gate=zs[:, 3:3 + heads] if gate else None)
        assert torch.all(wide[:, :8] == 3.0) and torch.all(wide[:, 8 + heads * dv:] == 3.0)
        at = 0
        for s, f, c in seqs:
            if s == 1:
                got.append(wide[at:at + c, 8:8 + heads * dv])
            at += c
    mask = O.visible(total, window if window else total + 1, keep)
    outs = []
    for a in range(heads):
        g = a // (heads // kv_heads)
        w = O.sink_softmax(d(q)[:, a] @ d(k)[:, g].T * scale, mask, d(sinks)[a])
        outs.append(w @ d(v)[:, g] * (torch.sigmoid(d(z)[:, 3 + a:4 + a]) if gate else 1.0))
    return torch.cat(got), torch.cat(outs, -1)


SHAPES = [(4, 2, 16, 8), (3, 3, 12, 10), (20, 1, 8, 8), (2, 1, 136, 40), (6, 3, 80, 72)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", SHAPES)
@pytest.mark.parametrize("window,keep", [(0, 0), (40, 0), (40, 5), (9, 33)])
def test_gate_per_head_in_portions_in_mixed_steps_and_decoded_over_partitions(dtype, shape, window, keep):
    total = 560
    plan = [[(1, 0, 270), (0, 0, 5)], [(1, 270, 2)], [(1, 272, 268), (0, 5, 1)]] + [[(0, 6 + i, 1), (1, 540 + i, 1)] for i in range(20)]
    got, want = _attention_case(dtype, *shape, total, plan, window, keep)
    _close(got, want, 5e-5 if dtype == torch.float32 else 3e-2)
    plain, base = _attention_case(dtype, *shape, total, plan, window, keep, gate=False)
    _close(plain, base, 5e-5 if dtype == torch.float32 else 3e-2)
    assert (base - want).abs().max() > 0.2 * base.abs().max()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", SHAPES[:2])
@pytest.mark.parametrize("keep,hot", [(1, 0), (4, 3), (4, 4), (40, 39), (40, 40), (300, 255), (300, 256), (300, 299), (300, 300)])
def test_kept_first_keys_reach_tokens_far_behind_them_and_the_next_key_does_not(dtype, shape, keep, hot):
    total, window = 700, 50
    plan = [[(1, 0, 300), (0, 0, 5)], [(1, 300, 2)], [(1, 302, 388)]] + [[(0, 5 + i, 1), (1, 690 + i, 1)] for i in range(10)]
    got, want = _attention_case(dtype, *shape, total, plan, window, keep, hot=hot)
    _close(got, want, 5e-5 if dtype == torch.float32 else 3e-2)
    far = hot + window + 5
    assert (got[far:].float().cpu() - want[far:]).abs().max() < 0.1 * want.abs().max()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", SHAPES[:4])
@pytest.mark.parametrize("window,keep,hot", [(1, 0, 5), (1, 2, 5), (9, 3, 40), (64, 1, 191), (100, 33, 256), (300, 4, 70), (6, 11, 20)])
def test_window_edge_with_kept_keys_in_prompts_and_in_decoding(dtype, shape, window, keep, hot):
    """The dominating key sits behind the kept ones: position hot + window - 1 still sees it, hot + window does not; the edge is
    crossed inside a portion and by decoded tokens."""
    total, edge = hot + window + 40, hot + window
    for plan in ([[(1, 0, 7), (0, 0, 3)], [(1, 7, total - 7)]],
                 [[(1, 0, edge - 3)]] + [[(1, i, 1), (0, i - edge + 3, 1)] for i in range(edge - 3, total)]):
        got, want = _attention_case(dtype, *shape, total, plan, window, keep, hot=hot, gate=False)
        _close(got, want, 5e-5 if dtype == torch.float32 else 3e-2)
        gap = (want[edge - 1] - want[edge]).abs().max()
        assert gap > 0.5 and (got[edge - 1:edge + 1].float().cpu() - want[edge - 1:edge + 1]).abs().max() < 0.05 * gap


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", SHAPES[:3])
@pytest.mark.parametrize("sink", [-40.0, 2.0, 12.0])
def test_learned_sink_enters_the_denominator_once(dtype, shape, sink):
    """Contexts that span several partitions of the decoded form: a sink counted per partition would show at once; a dominant sink
    leaves nearly nothing, a faint one everything."""
    total = 620
    plan = [[(1, 0, 600)]] + [[(1, 600 + i, 1)] for i in range(20)]
    got, want = _attention_case(dtype, *shape, total, plan, 0, 0, scale=0.1, sink=sink)
    _close(got, want, 5e-5 if dtype == torch.float32 else 3e-2)
    none, base = _attention_case(dtype, *shape, total, plan, 0, 0, scale=0.1, sink=-60.0)
    near = (want[50:] - base[50:]).abs().max() / base[50:].abs().max()
    assert near < 1e-6 if sink < 0 else near > 0.02


@pytest.mark.parametrize("dtype", DTYPES)
def test_first_tokens_of_a_sequence_see_exactly_themselves(dtype):
    for plan in ([[(1, 0, 6)]], [[(1, i, 1)] for i in range(6)], [[(1, 0, 2)], [(1, 2, 4)]]):
        got, want = _attention_case(dtype, 4, 2, 16, 8, 6, plan, 2, 3, sink=1.0)
        _close(got, want, 5e-5 if dtype == torch.float32 else 3e-2)


# ------------------------------------------------------------------------------------------------------------------- #
# feed-forwards alone
# ------------------------------------------------------------------------------------------------------------------- #
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("experts,top,width,count,keep", [(8, 4, 96, 2, 1), (9, 1, 60, 9, 4), (12, 5, 33, 3, 2), (64, 8, 128, 8, 4), (1, 1, 16, 1, 1),
                                                          (6, 6, 40, 2, 2), (10, 3, 64, 1, 1)])
def test_router_scores_groups_by_their_best_member_and_renormalises(dtype, experts, top, width, count, keep):
    from lite_llama_amd.kernels.fused_moe import group_router
    from oracle import kokuvik as O

    torch.manual_seed(experts * 7 + top)
    n = 61
    h = torch.randn(n, width, device=DEV).to(dtype)
    wr = (torch.randn(experts, width, device=DEV) * 3.0 * width ** -0.5).to(dtype)
    ids, weights, extra = group_router(h, wr, top, count, keep, scoring="softmax_groups")
    want_ids, want_w = O.route(d(h), d(wr), top, {"count": count, "keep": keep})
    assert extra is None
    z = (d(h) @ d(wr).T).sort(-1).values
    clear = z.diff(dim=-1).min(-1).values > 1e-4 if experts > 1 else torch.ones(n, dtype=torch.bool)   # (no close calls)
    assert clear.sum() > n // 3
    assert torch.equal(ids.cpu().long()[clear], want_ids[clear])
    _close(weights[clear.to(DEV)], want_w[clear], 1e-5)
    assert torch.allclose(weights.sum(-1).cpu(), torch.ones(n), atol=1e-5)


def test_router_prefers_the_group_with_the_largest_member_over_the_one_with_the_largest_sum():
    from lite_llama_amd.kernels.fused_moe import group_router

    wr = torch.zeros(6, 4, device=DEV)
    wr[:, 0] = torch.tensor([3.0, -9.0, 2.9, 2.8, 0.0, 0.5])
    h = torch.ones(3, 4, device=DEV)
    h[1] *= 1e3                                   # logits in the thousands: the softmax must not overflow
    h[2] = 0                                      # all equal: lower indices first
    ids, w, _ = group_router(h, wr, 2, 3, 1, scoring="softmax_groups")
    assert ids.tolist() == [[0, 1]] * 3
    assert w[0, 1].item() == pytest.approx(torch.softmax(torch.tensor([3.0, -9.0]), 0)[1].item(), rel=1e-4)
    assert w[1].tolist() == [1.0, 0.0] and w[2].tolist() == [0.5, 0.5]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("ff,off", [(40, 16), (37, 5), (1, 1)])
def test_squared_relu_writes_a_column_range(dtype, ff, off):
    from lite_llama_amd.kernels.norm_act import relu_square

    torch.manual_seed(ff)
    rows = (torch.randn(9, ff + 11, device=DEV) * 3).to(dtype)
    out = torch.full((9, off + ff + 8), 7.0, device=DEV).to(dtype)
    got = relu_square(rows[:, 8:], ff, out=out[:, off:off + ff])
    assert got.data_ptr() == out[:, off:].data_ptr()
    _close(got, torch.relu(d(rows[:, 8:8 + ff])) ** 2, 1e-6 if dtype == torch.float32 else 5e-3)
    assert torch.all(out[:, :off] == 7.0) and torch.all(out[:, off + ff:] == 7.0)
    assert torch.equal(relu_square(rows[:, 8:], ff), got)


# ------------------------------------------------------------------------------------------------------------------- #
# whole models: loader -> runner -> cache
# ------------------------------------------------------------------------------------------------------------------- #
_MODELS = {}


def _model(tmp_path_factory, name, dtype):
    from lite_llama_amd.weights import load_pretrained

    key = (name, dtype)
    if key not in _MODELS:
        cfg = T.CONFIGS[name]
        tens = T.tensors(cfg, seed=len(name))
        folder = L.write(tmp_path_factory.mktemp(name), cfg, tens)
        _MODELS[key] = (load_pretrained(folder, device=DEV, dtype=dtype), cfg, tens, folder)
    return _MODELS[key]


@pytest.mark.parametrize("name", sorted(T.CONFIGS))
def test_whole_prompt_layers_and_logits(tmp_path_factory, name):
    from lite_llama_amd.executor.ragged import RaggedRunner
    from oracle import kokuvik as O

    model, cfg, tens, _ = _model(tmp_path_factory, name, torch.float32)
    toks = L.prompt(cfg, 45)
    layers = []
    want = O.forward(toks, tens, cfg, layers_out=layers)
    runner = RaggedRunner(model, 64, 2, block_size=16, device=DEV)
    got_layers = []
    got = runner.step([(runner.admit(), toks)], list(range(len(toks))), collect_layers=got_layers)
    runner.check_errors()
    assert len(got_layers) == len(layers)
    for g, w in zip(got_layers, layers):
        _close(g, w, 2e-5)
    _close(got, want, 2e-5)


@pytest.mark.parametrize("name", sorted(T.CONFIGS))
@pytest.mark.parametrize("sizes", [[1], [2], [3, 2, 7, 1, 16, 5], [40, 1]])
def test_portions_and_token_by_token_decoding_equal_the_whole_prompt(tmp_path_factory, name, sizes):
    """Portions down to two tokens, pure token-by-token decoding from the first token on, and a long portion followed by decoding;
    pages of 8 tokens, so portions, windows, chunks and pages start and end inside one another."""
    from lite_llama_amd.executor.ragged import RaggedRunner
    from oracle import kokuvik as O

    model, cfg, tens, _ = _model(tmp_path_factory, name, torch.float32)
    toks = L.prompt(cfg, 58, seed=1)
    want = O.forward(toks, tens, cfg)
    runner = RaggedRunner(model, 64, 2, block_size=8, device=DEV)
    _close(_feed(runner, runner.admit(), toks, sizes), want, 3e-5)
    runner.check_errors()


@pytest.mark.parametrize("name", ["mix", "odd"])
def test_unequal_requests_in_one_batch_equal_each_alone_and_freed_pages_and_slots_are_used_again(tmp_path_factory, name):
    """Four requests of different lengths ride together in changing portions, three slots and a pool that only holds them because
    finished requests give their pages back; a late request takes over a used slot (with the states its last owner left) and used
    pages."""
    from lite_llama_amd.executor.ragged import RaggedRunner
    from oracle import kokuvik as O

    model, cfg, tens, _ = _model(tmp_path_factory, name, torch.float32)
    lens = {"a": 41, "b": 9, "c": 26, "d": 33}
    toks = {k: L.prompt(cfg, n, seed=ord(k)) for k, n in lens.items()}
    want = {k: O.forward(v, tens, cfg) for k, v in toks.items()}
    runner = RaggedRunner(model, 96, 3, block_size=8, device=DEV)      # 12 pages: a + b + c need 11, d needs 5
    sizes = {"a": [5, 1, 1, 9, 2, 30], "b": [2, 1, 3, 1, 1, 1], "c": [1, 13, 2, 2, 8], "d": [16, 1, 1, 15]}
    at, slot, got, k = {x: 0 for x in lens}, {}, {x: [] for x in lens}, 0
    waiting, live = ["a", "b", "c", "d"], []
    while waiting or live:
        while waiting and runner.free_slots and runner.blocks_held() + runner.blocks_for(lens[waiting[0]]) <= runner.total_blocks:
            who = waiting.pop(0)
            slot[who] = runner.admit()
            live.append(who)
        entries, rows, owners, base = [], [], [], 0
        for who in live:
            if (k + ord(who)) % 4 == 0 and len(live) > 1:
                continue                                              # left out of this step, goes on later
            c = min(sizes[who][min(k, len(sizes[who]) - 1)], lens[who] - at[who])
            entries.append((slot[who], toks[who][at[who]:at[who] + c]))
            rows += range(base, base + c)
            owners += [who] * c
            base, at[who] = base + c, at[who] + c
        k += 1
        if not entries:
            continue
        out = runner.step(entries, rows)
        for j, who in enumerate(owners):
            got[who].append(out[j:j + 1])
        ended = [n for n in live if at[n] == lens[n]]
        runner.release([slot[n] for n in ended])
        live = [n for n in live if n not in ended]
    runner.check_errors()
    assert slot["d"] in (slot["a"], slot["b"], slot["c"])
    assert runner.cache.free_blocks == runner.total_blocks
    for who in lens:
        _close(torch.cat(got[who]), want[who], 2e-5)


@pytest.mark.parametrize("name", ["odd", "wide"])
def test_long_decoding_past_windows_and_over_many_pages(tmp_path_factory, name):
    from lite_llama_amd.executor.ragged import RaggedRunner
    from oracle import kokuvik as O

    model, cfg, tens, _ = _model(tmp_path_factory, name, torch.float32)
    toks = L.prompt(cfg, 150, seed=5)
    want = O.forward(toks, tens, cfg)
    runner = RaggedRunner(model, 160, 1, block_size=16, device=DEV)
    _close(_feed(runner, runner.admit(), toks, [6, 1]), want, 3e-5)


@pytest.mark.parametrize("name", ["mix", "odd", "wide"])
def test_long_prompts_through_many_chunks_and_partitions(tmp_path_factory, name):
    from lite_llama_amd.executor.ragged import RaggedRunner
    from oracle import kokuvik as O

    model, cfg, tens, _ = _model(tmp_path_factory, name, torch.float32)
    toks = L.prompt(cfg, 420, seed=6)
    want = O.forward(toks, tens, cfg)
    runner = RaggedRunner(model, 900, 2, device=DEV)
    _close(_feed(runner, runner.admit(), toks, [420]), want, 3e-5)
    _close(_feed(runner, runner.admit(), toks, [129, 1, 255, 1]), want, 3e-5)


@pytest.mark.parametrize("name", sorted(T.CONFIGS))
def test_bfloat16_model_tracks_the_oracle_and_its_own_portions(tmp_path_factory, name):
    from lite_llama_amd.executor.ragged import RaggedRunner
    from oracle import kokuvik as O

    model, cfg, tens, _ = _model(tmp_path_factory, name, torch.bfloat16)
    toks = L.prompt(cfg, 70, seed=2)
    want = O.forward(toks, tens, cfg)
    runner = RaggedRunner(model, 160, 2, block_size=16, device=DEV)
    whole = _feed(runner, runner.admit(), toks, [70]).float().cpu()
    parts = _feed(runner, runner.admit(), toks, [2, 9, 1, 1, 30, 1]).float().cpu()
    spread = want.std().item()
    # medians over the tokens: a token whose router sees two experts within a rounding step of each other may choose the other
    err = lambda a, b: (a.to(F64) - b.to(F64)).pow(2).mean(-1).sqrt().median().item()   # noqa: E731
    assert err(whole, want) < 0.06 * spread
    assert err(parts, whole) < 0.04 * spread


@pytest.mark.parametrize("dtype", DTYPES)
def test_captured_decode_steps_replay_like_eager_ones(tmp_path_factory, dtype):
    from lite_llama_amd.executor.ragged import RaggedRunner

    model, cfg, _, _ = _model(tmp_path_factory, "mix", dtype)
    a, b = L.prompt(cfg, 290, seed=21), L.prompt(cfg, 40, seed=22)
    eager = RaggedRunner(model, 512, 2, block_size=16, device=DEV)
    graph = RaggedRunner(model, 512, 2, block_size=16, device=DEV, capture_decode=True)
    out = {"eager": [], "graph": []}
    for name, r in (("eager", eager), ("graph", graph)):
        sa, sb = r.admit(), r.admit()
        r.step([(sa, a[:240])], [])
        for i in range(240, 262):                                   # one sequence decoding across a partition edge
            out[name].append(r.step([(sa, a[i:i + 1])]).float().cpu().clone())
        r.step([(sa, a[262:263]), (sb, b[:30])], [])
        for i in range(10):                                         # two sequences decoding together
            out[name].append(r.step([(sa, a[263 + i:264 + i]), (sb, b[30 + i:31 + i])]).float().cpu().clone())
        r.release([sb])
        for i in range(273, 290):
            out[name].append(r.step([(sa, a[i:i + 1])]).float().cpu().clone())
        r.check_errors()
    assert graph.replays >= 40 and eager.replays == 0
    for e, g2 in zip(out["eager"], out["graph"]):
        assert torch.allclose(e, g2, rtol=0, atol=1e-6 if dtype == torch.float32 else 2e-2), (e - g2).abs().max()


# ------------------------------------------------------------------------------------------------------------------- #
# entry points: engine, command line, trace replay
# ------------------------------------------------------------------------------------------------------------------- #
def test_engine_generates_greedily_like_the_oracle(tmp_path_factory):
    from lite_llama_amd.engine import GenerationEngine, SamplingParams
    from oracle import kokuvik as O

    model, cfg, tens, _ = _model(tmp_path_factory, "odd", torch.float32)
    prompts = [L.prompt(cfg, n, seed=n) for n in (3, 19, 1, 11, 7)]
    engine = GenerationEngine(model, max_tokens=96, max_requests=3, block_size=8, max_step_tokens=10, device=DEV)
    outs = engine.generate(prompts, SamplingParams(max_new_tokens=6))
    for p, o in zip(prompts, outs):
        assert o == O.greedy(p, tens, cfg, 6)
    captured = GenerationEngine(model, max_tokens=96, max_requests=3, block_size=8, max_step_tokens=10, device=DEV, capture_decode=True)
    assert captured.generate(prompts, SamplingParams(max_new_tokens=6)) == outs and captured.runner.replays > 0
    assert engine.runner.cache.free_blocks == engine.runner.total_blocks and engine.runner.free_slots == 3
    sampled = engine.generate(prompts[:2], SamplingParams(max_new_tokens=5, temperature=0.8, top_p=0.9, repetition_penalty=1.2))
    assert [len(s) for s in sampled] == [5, 5] and all(0 <= t < cfg["vocab"] for s in sampled for t in s)


def test_command_line_generate_and_trace_replay(tmp_path_factory, tmp_path):
    from oracle import kokuvik as O

    _, cfg, tens, folder = _model(tmp_path_factory, "wide", torch.float32)
    prompt = L.prompt(cfg, 9, seed=4)
    env = dict(os.environ, PYTHONPATH=ROOT)
    done = subprocess.run([sys.executable, "-m", "lite_llama_amd", "generate", "--model", folder, "--dtype", "float32",
                           "--prompt-ids", ",".join(map(str, prompt)), "--max-new-tokens", "4"],
                          capture_output=True, text=True, env=env, cwd=ROOT, timeout=300)
    assert done.returncode == 0, done.stderr[-2000:]
    line = json.loads(done.stdout.strip().splitlines()[-1])
    assert line["prompt"] == prompt and line["generated"] == O.greedy(prompt, tens, cfg, 4)

    a, b = L.prompt(cfg, 31, seed=8), L.prompt(cfg, 6, seed=9)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:13], "want": [0, 12]}, {"id": "b", "tokens": b[:2], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[2:], "want": [3]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[13:30], "want": []}], "end": []},
             {"step": 3, "entries": [{"id": "a", "tokens": a[30:], "want": [0]}, {"id": "c", "tokens": b, "want": [5]}], "end": ["a", "c"]}]
    out = tmp_path / "out"
    done = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", "float32", "--out", str(out),
                           "--max-tokens", "128"], input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True,
                          text=True, env=env, cwd=ROOT, timeout=300)
    assert done.returncode == 0, done.stderr[-2000:]
    assert [ln for ln in done.stdout.splitlines() if ln.startswith("done")] == [f"done {i}" for i in range(4)]
    import numpy as np

    la, lb = O.forward(a, tens, cfg), O.forward(b, tens, cfg)
    read = lambda i: torch.from_numpy(np.fromfile(out / f"{i}.f32", dtype="<f4")).view(-1, cfg["vocab"])   # noqa: E731
    _close(read(0), la[[0, 12]], 2e-5)
    _close(read(1), lb[[5]], 2e-5)
    assert not (out / "2.f32").exists()
    _close(read(3), torch.stack([la[30], lb[5]]), 2e-5)


def _random_config(seed):
    """A configuration drawn from the whole range the reader takes: both mixers in any order, borrowing layers, head counts and widths
    with and without the matrix-core forms' multiples, windows from 1 key to longer than the prompt, kept keys from none to more than
    the window, rotations of a part or all of a head with and without bands, every feed-forward kind."""
    import random

    r = random.Random(seed)
    layers, owners = [], []
    for i in range(r.randint(2, 5)):
        experts, groups = r.choice([(1, None), (5, None), (6, (3, 2)), (8, (2, 1)), (9, (9, 3)), (12, (4, 4))])
        room = experts if groups is None else experts // groups[0] * groups[1]
        mlp = {"dense": T.dense(r.choice([16, 40, 44, 3])), None: None,
               "moe": T.moe(experts, r.randint(1, room), r.choice([8, 12, 24]), shared=r.choice([0, 8, 20, 7]), groups=groups)}[
                   r.choice(["dense", "moe", "moe", None])]
        if r.random() < 0.5:
            dim = r.choice([8, 16, 32, 64, 12, 6, 130])
            layers.append(T.retention(r.randint(1, 5), dim, r.choice([8, 16, 40, 10, 1]), r.choice([dim, dim // 2 // 2 * 2, 2]), mlp=mlp,
                                      base=r.choice([100.0, 10000.0])))
            continue
        window, keep = r.choice([1, 3, 8, 17, 40, 64, 200]), r.choice([0, 0, 1, 2, 5, 33, 70])
        if owners and r.random() < 0.6:
            src = r.choice(owners)
            m = layers[src]["mixer"]
            entry = {"type": "attention", "mlp": mlp, "mixer": dict(m, mask={"size": window, "keep_first": keep}, kv_from=src, scale=m["scale"] * 0.7)}
            layers.append(entry)
            continue
        g = r.choice([1, 2, 3])
        dim = r.choice([8, 16, 32, 64, 12, 20, 128])
        owners.append(i)
        layers.append(T.attention(g * r.choice([1, 2, 4, 5]), g, dim, r.choice([8, 16, 24, 10, 48]), window, keep, r.choice([dim, dim // 2, 2]),
                                  mlp=mlp, scaled=r.random() < 0.7, base=r.choice([100.0, 10000.0]), factor=r.choice([2.0, 8.0]),
                                  low=r.choice([0.5, 1.0]), high=r.choice([4.0, 32.0]), original=r.choice([16, 64, 1024]),
                                  scale=r.choice([0.5, 1.0, 2.0]) * 2 * dim ** -0.5))
    return T.config(layers, width=r.choice([32, 48, 60, 88]), vocab=r.randint(20, 300), eps=r.choice([1e-5, 1e-6, 1e-3]))


@pytest.mark.parametrize("seed", range(16))
def test_random_configurations_whole_in_portions_decoded_and_side_by_side(tmp_path, seed):
    from lite_llama_amd.executor.ragged import RaggedRunner
    from lite_llama_amd.weights import load_pretrained
    from oracle import kokuvik as O

    cfg = _random_config(seed)
    tens = T.tensors(cfg, seed=seed)
    model = load_pretrained(L.write(tmp_path / "m", cfg, tens), device=DEV, dtype=torch.float32)
    a, b = L.prompt(cfg, 90, seed=seed), L.prompt(cfg, 37, seed=seed + 50)
    wa, wb = O.forward(a, tens, cfg), O.forward(b, tens, cfg)
    runner = RaggedRunner(model, 256, 3, block_size=16, device=DEV)
    _close(_feed(runner, runner.admit(), a, [90]), wa, 5e-5)
    _close(_feed(runner, runner.admit(), a, [2, 1, 7, 3, 1, 30, 1]), wa, 5e-5)
    runner.release([0, 1])
    sa, sb = runner.admit(), runner.admit()            # used slots and pages again, two requests side by side
    got_a, got_b, ia, ib = [], [], 0, 0
    for ca, cb in [(11, 1), (1, 2), (40, 1), (1, 20), (5, 1), (32, 12)]:
        out = runner.step([(sa, a[ia:ia + ca]), (sb, b[ib:ib + cb])], list(range(ca + cb)))
        got_a.append(out[:ca])
        got_b.append(out[ca:])
        ia, ib = ia + ca, ib + cb
    assert ia == 90 and ib == 37
    runner.check_errors()
    _close(torch.cat(got_a), wa, 5e-5)
    _close(torch.cat(got_b), wb, 5e-5)


@pytest.mark.parametrize("seed", range(20, 28))
def test_random_configurations_in_bfloat16_track_the_oracle_and_their_own_portions(tmp_path, seed):
    from lite_llama_amd.executor.ragged import RaggedRunner
    from lite_llama_amd.weights import load_pretrained
    from oracle import kokuvik as O

    cfg = _random_config(seed)
    tens = T.tensors(cfg, seed=seed)
    model = load_pretrained(L.write(tmp_path / "m", cfg, tens), device=DEV, dtype=torch.bfloat16)
    a = L.prompt(cfg, 150, seed=seed)
    want = O.forward(a, tens, cfg)
    runner = RaggedRunner(model, 512, 2, device=DEV)
    whole = _feed(runner, runner.admit(), a, [150]).float().cpu()
    parts = _feed(runner, runner.admit(), a, [2, 9, 40, 1, 65, 1]).float().cpu()
    runner.check_errors()
    # medians over the tokens: a close call of a router may go the other way
    err = lambda x, y: (x.to(F64) - y.to(F64)).pow(2).mean(-1).sqrt().median().item()   # noqa: E731
    assert err(whole, want) < 0.06 * want.std().item()
    assert err(parts, whole) < 0.04 * want.std().item()
