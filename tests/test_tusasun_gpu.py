"""Tusasun on the GPU against the plain CPU restatement (oracle/tusasun.py): each mechanism's kernels alone, then whole models
built from small random checkpoints through the loader, the ragged runner, the paged state cache, the generation engine and the
command line.  float32 runs are held to rounding error; bfloat16 runs to the rounding of their activations.  Where random
weights would hide a fault (a distance one bucket off, a pair written far back into a slowly forgetting state, a weight on the
wrong side of a square), inputs are made so that it shows."""

import json
import os
import subprocess
import sys

import pytest
import torch

from tests import _layered as L
from tests import _tusasun as T
from tests.test_layered_gpu import _close, _feed, _step
from tests.test_nivotar_gpu import LENS, PLAN, _walk, bf, d

pytestmark = pytest.mark.gpu
DEV = "cuda"
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
F64 = torch.float64
_MODELS = {}


# ------------------------------------------------------------------------------------------------------------------- #
# gated delta rule
# ------------------------------------------------------------------------------------------------------------------- #
def _delta_setup(heads, qk_heads, dk, dv, seed=0):
    g = torch.Generator().manual_seed(seed + dk * 7 + dv)
    qk, gk, vw = qk_heads * dk, heads * dk, heads * dv
    cols = 2 * qk + vw + gk + heads
    return g, (qk, gk, vw, cols), bf(torch.randn(gk, generator=g) - 1.0), bf(torch.rand(heads, generator=g) * 3 - 2.5)


def _delta_run(heads, qk_heads, dk, dv, sizes, dt_bias, a_log, state, dtype):
    from lite_llama_amd.kernels.recurrent import delta_scan

    qk, gk, vw, _ = sizes
    return lambda r, step: delta_scan(r[:, :qk], r[:, qk:2 * qk], r[:, 2 * qk:2 * qk + vw], heads, dk, dv, step, state,
                                      gate=r[:, 2 * qk + vw:2 * qk + vw + gk], beta=r[:, 2 * qk + vw + gk:], qk_heads=qk_heads,
                                      dt_bias=dt_bias.to(DEV).to(dtype), a_log=a_log.to(DEV).to(dtype), q_scale=dk ** -0.5)


def _delta_want(rows, heads, qk_heads, dk, dv, sizes, dt_bias, a_log):
    from oracle import tusasun as O

    qk, gk, vw, _ = sizes
    r = rows.to(F64)
    q, k = O.unit(r[:, :qk].view(-1, qk_heads, dk)) * dk ** -0.5, O.unit(r[:, qk:2 * qk].view(-1, qk_heads, dk))
    v, beta = r[:, 2 * qk:2 * qk + vw].view(-1, heads, dv), torch.sigmoid(r[:, 2 * qk + vw + gk:])
    dec = O.channel_decay(r[:, 2 * qk + vw:2 * qk + vw + gk].view(-1, heads, dk), dt_bias.to(F64).view(heads, dk), a_log.to(F64))
    out, last = torch.zeros(r.shape[0], heads, dv, dtype=F64), []
    for h in range(heads):
        j = h // (heads // qk_heads)
        out[:, h], S = O.delta_scan(q[:, j], k[:, j], v[:, h], dec[:, h], beta[:, h])
        last.append(S)
    return out.view(-1, vw), torch.stack(last)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads,qk_heads,dk,dv", [(2, 2, 16, 24), (4, 2, 64, 16), (6, 2, 10, 6), (3, 1, 72, 40), (2, 2, 128, 70),
                                                 (1, 1, 1, 1), (1, 1, 200, 20), (2, 1, 256, 65)])
def test_delta_rule_over_portions_of_every_size_and_stale_slots(dtype, heads, qk_heads, dk, dv):
    """Starts of sequences, single decoded tokens and portions inside a sequence side by side; slots hold another owner's state
    when a sequence starts in them; the state left behind is the oracle's."""
    g, sizes, dt_bias, a_log = _delta_setup(heads, qk_heads, dk, dv)
    state = torch.randn(4, heads, dk, dv, device=DEV)
    untouched = state[1].clone()
    run = _delta_run(heads, qk_heads, dk, dv, sizes, dt_bias, a_log, state, dtype)
    full, got = _walk(PLAN, LENS, dtype, lambda s, n: bf(torch.randn(n, sizes[3], generator=g)), run)
    for s, rows in full.items():
        want, last = _delta_want(rows, heads, qk_heads, dk, dv, sizes, dt_bias, a_log)
        _close(got[s], want, 2e-5)
        _close(state[s], last, 2e-5)
    assert torch.equal(state[1], untouched)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("dk,dv", [(24, 40), (64, 130)])
def test_delta_rule_leaves_the_same_bits_whatever_the_cut_and_the_company(dtype, dk, dv):
    """One prompt in one portion (decays evaluated ahead of the walk), token by token (evaluated inside it), and as one of forty
    sequences of a step (a wider column form): outputs and state bit for bit."""
    heads, n = 8, 37
    g, sizes, dt_bias, a_log = _delta_setup(heads, heads, dk, dv)
    rows = bf(torch.randn(n, sizes[3], generator=g))
    outs, states = [], []
    for plan, slots in (([[(0, 0, n)]], 1), ([[(0, p, 1)] for p in range(n)], 1), ([[(0, 0, n)] + [(s, 0, 2) for s in range(1, 40)]], 40)):
        state = torch.randn(slots, heads, dk, dv, device=DEV)
        run = _delta_run(heads, heads, dk, dv, sizes, dt_bias, a_log, state, dtype)
        _, got = _walk(plan, {s: (n if s == 0 else 2) for s in range(slots)}, dtype, lambda s, m: rows[:m], run, slots=slots)
        outs.append(got[0])
        states.append(state[0].clone())
    for k in (1, 2):
        assert torch.equal(outs[0], outs[k]) and torch.equal(states[0], states[k])


@pytest.mark.parametrize("far", [0, 3, 15, 16, 255])
def test_a_pair_written_far_back_is_read_hundreds_of_tokens_later_and_can_be_overwritten(far):
    """Key entry 3 never forgets; the pair written at ``far`` is read 600 tokens later through portions that end on and off the
    token tiles and through decoded tokens.  A later token with the same key and a full step replaces the value (it is not added)."""
    from oracle import tusasun as O

    heads, dk, dv, total = 1, 16, 8, 720
    g, sizes, _, _ = _delta_setup(heads, heads, dk, dv, seed=far)
    qk, gk, vw, cols = sizes
    dt_bias, a_log = torch.zeros(gk), torch.zeros(heads)
    rows = bf(torch.randn(total, cols, generator=g) * 0.3)
    rows[:, qk + 3] = rows[:, 3] = 0.0                                # nobody else writes or reads entry 3
    rows[:, 2 * qk + vw:2 * qk + vw + gk] = bf(torch.randn(total, gk, generator=g) - 3.0)
    rows[:, 2 * qk + vw + 3] = -40.0                                  # softplus ~ 0: decay 1
    value, other = bf(torch.linspace(-8, 8, dv)), bf(torch.linspace(3, -5, dv))
    for at, v in ((far, value), (690, other)):
        rows[at, qk:2 * qk] = 0.0
        rows[at, qk + 3] = 1.0
        rows[at, 2 * qk:2 * qk + vw] = v
        rows[at, -1] = 40.0                                           # full step
    for probe in (600, 680, 700):
        rows[probe, :qk] = 0.0
        rows[probe, 3] = 1.0
    state = torch.randn(2, heads, dk, dv, device=DEV)
    plan = [[(1, 0, 1)], [(1, 1, 16)], [(1, 17, 47)], [(1, 64, 2)], [(1, 66, 1)], [(1, 67, 500)], [(1, 567, 100)]] \
        + [[(1, p, 1)] for p in range(667, total)]
    run = _delta_run(heads, heads, dk, dv, sizes, dt_bias, a_log, state, torch.float32)
    _, got = _walk(plan, {1: total}, torch.float32, lambda s, n: rows, run, slots=2)
    want, _ = _delta_want(rows, heads, heads, dk, dv, sizes, dt_bias, a_log)
    scale = dk ** -0.5
    assert (want[600] - value.to(F64) * scale).abs().max() < 1e-4 and (want[700] - other.to(F64) * scale).abs().max() < 1e-4
    _close(got[1], want, 2e-5)


def test_delta_decays_from_one_to_zero_and_empty_queries_stay_finite():
    heads, dk, dv, n = 2, 16, 8, 40
    g, sizes, _, _ = _delta_setup(heads, heads, dk, dv, seed=5)
    qk, gk, vw, cols = sizes
    dt_bias = bf(torch.linspace(-60, 60, gk))                         # softplus from 0 to 60: decays from 1 to e^-60 and less
    a_log = torch.tensor([1.0, -1.0])
    rows = bf(torch.randn(n, cols, generator=g))
    rows[7, :2 * qk] = 0.0                                            # a zero query and key: unit norm with its epsilon
    state = torch.randn(1, heads, dk, dv, device=DEV)
    run = _delta_run(heads, heads, dk, dv, sizes, dt_bias, a_log, state, torch.float32)
    _, got = _walk([[(0, 0, 13)], [(0, 13, 27)]], {0: n}, torch.float32, lambda s, m: rows, run, slots=1)
    want, _ = _delta_want(rows, heads, heads, dk, dv, sizes, dt_bias, a_log)
    assert torch.isfinite(got[0]).all()
    _close(got[0], want, 2e-5)


# ------------------------------------------------------------------------------------------------------------------- #
# real-gated recurrence, convolution without an activation
# ------------------------------------------------------------------------------------------------------------------- #
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width,blocks,plan", [(48, 3, "short"), (30, 15, "short"), (1, 1, "short"), (300, 2, "short"), (40, 5, "long"), (264, 1, "long")])
def test_real_gated_recurrence_over_portions_and_long_runs(dtype, width, blocks, plan):
    """Short portions take the token walk, runs of 128 tokens and more the chunked one, next to decoded tokens and starts."""
    from lite_llama_amd.kernels.recurrent import rglru_scan
    from oracle import tusasun as O

    g = torch.Generator().manual_seed(width)
    bs = width // blocks
    steps, lens = (PLAN, LENS) if plan == "short" else \
        ([[(2, 0, 131)], [(2, 131, 1), (0, 0, 300)], [(2, 132, 200), (0, 300, 1), (3, 0, 33)], [(3, 33, 128), (2, 332, 1)]], {2: 333, 0: 301, 3: 161})
    rb, ib, lam = bf(torch.randn(width, generator=g)), bf(torch.randn(width, generator=g)), bf(torch.randn(width, generator=g) * 2 - 3)
    state = torch.randn(4, width, device=DEV)

    def run(r, step):
        gates = r[:, width:3 * width].contiguous().view(-1, blocks, 2, bs)
        to = lambda t: t.to(DEV).to(dtype)  # noqa: E731
        return rglru_scan(r[:, :width], gates, to(rb), to(ib), to(lam), r[:, 3 * width:], step, state)

    full, got = _walk(steps, lens, dtype, lambda s, n: bf(torch.randn(n, 4 * width, generator=g)), run)
    for s, rows in full.items():
        r = rows.to(F64)
        gates = r[:, width:3 * width].view(-1, blocks, 2, bs)
        rr = torch.sigmoid(gates[:, :, 0].reshape(-1, width) + rb.to(F64))
        ii = torch.sigmoid(gates[:, :, 1].reshape(-1, width) + ib.to(F64))
        S, last = O.real_gated_scan(r[:, :width], rr, ii, lam.to(F64))
        _close(got[s], S * O.gelu_tanh(r[:, 3 * width:]), 1e-5 if dtype == torch.float32 else 1e-2)
        _close(state[s], last, 1e-5)


@pytest.mark.parametrize("far", [0, 31, 32, 200])
def test_real_gated_state_holds_a_far_input_and_slow_channels_write_little(far):
    """Channel 0 forgets nothing measurable (a within 1e-6 of 1: what it writes is the square root of twice the distance, which
    1 - a^2 in single precision would lose half of); a large input at ``far`` is still there 500 tokens later."""
    from lite_llama_amd.kernels.recurrent import rglru_scan
    from oracle import tusasun as O

    width, total = 8, 640
    g = torch.Generator().manual_seed(far)
    lam = bf(torch.tensor([-16.0, -12.0, -9.0, -6.0, -3.0, 0.0, 3.0, 20.0]))
    rows = bf(torch.randn(total, 4 * width, generator=g) * 0.3)
    rows[far, :width] = 500.0
    rows[:, 3 * width:] = 2.0
    zero = torch.zeros(width, device=DEV)
    state = torch.randn(1, width, device=DEV)
    run = lambda r, step: rglru_scan(r[:, :width], r[:, width:3 * width].contiguous().view(-1, 1, 2, width), zero, zero, lam.to(DEV),  # noqa: E731
                                     r[:, 3 * width:], step, state)
    plan = [[(0, 0, 33)], [(0, 33, 300)], [(0, 333, 2)], [(0, 335, 129)]] + [[(0, p, 1)] for p in range(464, total)]
    _, got = _walk(plan, {0: total}, torch.float32, lambda s, n: rows, run, slots=1)
    r = rows.to(F64)
    S, _ = O.real_gated_scan(r[:, :width], torch.sigmoid(r[:, width:2 * width]), torch.sigmoid(r[:, 2 * width:3 * width]), lam.to(F64))
    want = S * O.gelu_tanh(r[:, 3 * width:])
    for c in range(width):
        _close(got[0][:, c], want[:, c], 2e-5)
    assert want[far + 400, 0].abs() > 0.9 * want[far, 0].abs()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("channels,taps,biased", [(40, 3, True), (37, 1, True), (24, 4, False), (30, 6, True), (300, 2, False)])
def test_convolution_without_an_activation(dtype, channels, taps, biased):
    from lite_llama_amd.kernels.recurrent import conv_act
    from oracle import tusasun as O

    g = torch.Generator().manual_seed(channels + taps)
    w, b = bf(torch.randn(channels, taps, generator=g) * 0.5), bf(torch.randn(channels, generator=g) * 0.3) if biased else None
    state = torch.randn(2, 4, max(taps - 1, 1), channels, device=DEV).to(dtype) if taps > 1 else None
    run = lambda r, step: conv_act(r, w.to(DEV).to(dtype), b.to(DEV).to(dtype) if biased else None, step, state, act=None)  # noqa: E731
    full, got = _walk(PLAN, LENS, dtype, lambda s, n: bf(torch.randn(n, channels, generator=g)), run)
    for s, rows in full.items():
        _close(got[s], O.causal_conv(rows.to(F64), w.to(F64), b.to(F64) if biased else None), 3e-6 if dtype == torch.float32 else 1e-2)


# ------------------------------------------------------------------------------------------------------------------- #
# attention: capped scores, bias per distance
# ------------------------------------------------------------------------------------------------------------------- #
def _attention_case(total, heads, kv_heads, dk, dv, block, seed, dtype):
    """Random rows, and caches of used pages in random order that hold every position's key and value."""
    g = torch.Generator().manual_seed(seed)
    q, k, v = (bf(torch.randn(total, n, w, generator=g)) for n, w in ((heads, dk), (kv_heads, dk), (kv_heads, dv)))
    pages = -(-total // block)
    order = torch.randperm(pages, generator=g)
    table = torch.zeros(1, pages * block, dtype=torch.int32)
    for p in range(pages * block):
        table[0, p] = int(order[p // block]) * block + p % block
    return q, k, v, table, pages * block


def _attend(plan, q, k, v, table, rows, scale, dtype, **kw):
    from lite_llama_amd.kernels.attention import ragged_attention

    k_cache = torch.randn(rows, *k.shape[1:], device=DEV).to(dtype) * 3
    v_cache = torch.randn(rows, *v.shape[1:], device=DEV).to(dtype) * 3
    where = table[0, :k.shape[0]].long()
    out = []
    for first, count in plan:
        k_cache[where[first:first + count]] = k[first:first + count].to(DEV).to(dtype)
        v_cache[where[first:first + count]] = v[first:first + count].to(DEV).to(dtype)
        out.append(ragged_attention(q[first:first + count].to(DEV).to(dtype).contiguous(), k_cache, v_cache, scale, _step([(0, first, count, 0)], table),
                                    table.to(DEV), **kw))
    return torch.cat(out)


def _want_attention(q, k, v, scale, cap, rel, far):
    from oracle import tusasun as O

    rep = q.shape[1] // k.shape[1]
    heads = []
    for h in range(q.shape[1]):
        s = O.attention_scores(q[:, h].to(F64), k[:, h // rep].to(F64), scale, cap, rel[:, h].to(F64), far)
        heads.append(torch.softmax(s, -1) @ v[:, h // rep].to(F64))
    return torch.cat(heads, -1)


def _spread(rel, far):
    from lite_llama_amd.model_layers import distance_buckets

    return rel.float()[torch.tensor(distance_buckets(rel.shape[0], far))].t().contiguous().to(DEV)


PLANS = {"whole": lambda n: [(0, n)], "portions": lambda n: [(0, 2), (2, 31), (33, 1), (34, 64), (98, 2), (100, n - 100)],
         "decoded": lambda n: [(0, n - 40)] + [(p, 1) for p in range(n - 40, n)]}


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads,kv_heads,dk,dv,rows,far", [(4, 2, 16, 8, 16, 40.0), (3, 1, 12, 10, 6, 9.0), (20, 1, 8, 8, 32, 300.0),
                                                          (2, 2, 64, 96, 8, 280.0), (1, 1, 128, 128, 2, 2.0)])
@pytest.mark.parametrize("plan", sorted(PLANS))
def test_capped_scores_and_distance_bias_in_prompts_portions_and_decoding(dtype, heads, kv_heads, dk, dv, rows, far, plan):
    """Biases of neighbouring buckets differ by several units, so a distance that falls into the wrong bucket, or a table read one
    entry off, changes weights by orders of magnitude; scores reach well into the cap."""
    total, scale, cap = 330, 6.0 * dk ** -0.5, 5.0
    q, k, v, table, n = _attention_case(total, heads, kv_heads, dk, dv, 16, rows + dk, dtype)
    g = torch.Generator().manual_seed(rows)
    rel = bf((torch.arange(rows) % 2 * 5.0)[:, None] + torch.randn(rows, heads, generator=g))
    got = _attend(PLANS[plan](total), q, k, v, table, n, scale, dtype, cap=cap, dist_bias=_spread(rel, far))
    want = _want_attention(q, k, v, scale, cap, rel, far)
    plain = _want_attention(q, k, v, scale, 0.0, rel, far)
    assert (want - plain).abs().max() > 0.3
    _close(got, want, 2e-5 if dtype == torch.float32 else 2e-2)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("hot", [0, 5, 63, 64, 200, 255, 256])
@pytest.mark.parametrize("plan", ["prompt", "decoded"])
def test_one_key_at_every_distance_around_each_bucket_edge(dtype, hot, plan):
    """All keys but one score alike; one key's bias decides by its distance: every second bucket shuts it off, the others let it
    dominate.  Queries on both sides of every edge lie in prompt portions in one plan and are decoded in the other; the last bucket
    (on) still finds the key 300 tokens later, across partitions of the decode form."""
    from oracle import tusasun as O

    heads, dk, dv, rows, far = 2, 16, 8, 8, 50.0
    total = hot + 320
    q, k, v, table, n = _attention_case(total, heads, heads, dk, dv, 16, hot, dtype)
    q[:], k[:] = 1.0, 0.0
    k[hot] = 1.0
    v[hot] = 40.0
    open_ = [b % 2 == 0 or b == rows - 1 for b in range(rows)]
    rel = bf(torch.tensor([12.0 if o else -30.0 for o in open_]))[:, None].repeat(1, heads)
    scale, cap = 40.0 / dk, 16.0                                      # the hot key's score: 16 tanh(40 / 16) ~ 15.8; all others 0
    # (the other keys carry the same biases: what a query sees is the hot key's share of e^(15.8 + bias) against them)
    edges = [x for x in range(1, 60) if O.distance_bucket(x, rows, far) != O.distance_bucket(x - 1, rows, far)]
    plans = {"prompt": [(0, hot + 1), (hot + 1, total - hot - 1)], "decoded": [(0, hot + 1)] + [(p, 1) for p in range(hot + 1, min(hot + 70, total))]
             + [(min(hot + 70, total), total - min(hot + 70, total) - 3)] + [(p, 1) for p in range(total - 3, total)]}
    got = _attend(plans[plan], q, k, v, table, n, scale, dtype, cap=cap, dist_bias=_spread(rel, far))
    want = _want_attention(q, k, v, scale, cap, rel, far)
    seen = 0
    for e in edges:
        before, after = open_[O.distance_bucket(e - 1, rows, far)], open_[O.distance_bucket(e, rows, far)]
        if before != after:
            on, off = (hot + e, hot + e - 1) if after else (hot + e - 1, hot + e)
            assert want[on].mean() > 30.0 > 10.0 > want[off].mean()
            seen += 1
    assert seen >= 5
    assert want[-1].mean() > 30.0
    _close(got, want, 2e-5 if dtype == torch.float32 else 2e-2)


@pytest.mark.parametrize("cap,biased", [(0.0, True), (3.0, False)])
def test_either_half_of_the_score_shape_alone_and_a_mixed_step(cap, biased):
    """A prompt portion beside decoded tokens of other sequences in one step, 16-bit: bias without a cap, cap without a bias."""
    from lite_llama_amd.kernels.attention import ragged_attention

    dtype, heads, kv_heads, dk, dv = torch.bfloat16, 4, 2, 32, 16
    g = torch.Generator().manual_seed(3)
    lens, seqs, block = [90, 40, 300], [(0, 50, 40, 0), (1, 39, 1, 0), (2, 298, 2, 0)], 320
    rel = bf(torch.randn(16, heads, generator=g) * 3)
    bias = _spread(rel, 100.0) if biased else None
    table = (torch.arange(3)[:, None] * block + torch.randperm(block, generator=g)[None, :]).to(torch.int32)
    k_cache, v_cache = torch.zeros(3 * block, kv_heads, dk), torch.zeros(3 * block, kv_heads, dv)
    qs, want = [], []
    for s, n in enumerate(lens):
        q, k, v = (bf(torch.randn(n, h, w, generator=g)) for h, w in ((heads, dk), (kv_heads, dk), (kv_heads, dv)))
        k_cache[table[s, :n].long()], v_cache[table[s, :n].long()] = k, v
        first = seqs[s][1]
        qs.append(q[first:])
        want.append(_want_attention(q, k, v, 0.7, cap, rel if biased else rel * 0, 100.0)[first:])
    out = ragged_attention(torch.cat(qs).to(DEV).to(dtype), k_cache.to(DEV).to(dtype), v_cache.to(DEV).to(dtype), 0.7, _step(seqs, table),
                           table.to(DEV), cap=cap, dist_bias=bias)
    _close(out, torch.cat(want), 2e-2)


# ------------------------------------------------------------------------------------------------------------------- #
# experts
# ------------------------------------------------------------------------------------------------------------------- #
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("experts,top,width", [(6, 3, 96), (5, 5, 58), (1, 1, 18), (60, 4, 40), (16, 1, 128)])
def test_router_weights_are_the_plain_sigmoid_scores(dtype, experts, top, width):
    from lite_llama_amd.kernels.fused_moe import group_router
    from oracle import tusasun as O

    torch.manual_seed(experts * 10 + top)
    n = 33
    h, w, sg = bf(torch.randn(n, width)), bf(torch.randn(experts, width) * 2 * width ** -0.5), bf(torch.randn(1, width) * width ** -0.5)
    ids, weights, shared = group_router(h.to(DEV).to(dtype), w.to(DEV).to(dtype), top, scoring="sigmoid_plain", extra_weight=sg.to(DEV).to(dtype))
    want_ids, want = O.route(h.to(F64), {"router": w}, "", top)
    assert (ids.cpu().long() == want_ids).all()
    _close(weights, want, 1e-5)
    _close(shared, torch.sigmoid(h.to(F64) @ sg[0].to(F64)), 1e-5)
    if top > 1:
        assert (want.sum(-1) - 1).abs().max() > 0.2                   # (scores divided by their sum would be far off)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("experts,top,width,ff,n", [(4, 3, 64, 24, 19), (3, 2, 36, 10, 5), (2, 1, 128, 64, 600), (5, 2, 96, 40, 700), (1, 1, 8, 1, 3)])
def test_weights_multiply_the_experts_inputs_in_all_product_forms(dtype, experts, top, width, ff, n):
    from lite_llama_amd.kernels.fused_moe import sparse_square_experts
    from oracle import tusasun as O

    g = torch.Generator().manual_seed(ff)
    h = bf(torch.randn(n, width, generator=g))
    t = {}
    for e in range(experts):
        t[f"e{e}.up"], t[f"e{e}.down"] = bf(torch.randn(ff, width, generator=g) * width ** -0.5), bf(torch.randn(width, ff, generator=g) * ff ** -0.5)
    ids = torch.stack([torch.randperm(experts, generator=g)[:top] for _ in range(n)]).to(torch.int32)
    weights = torch.rand(n, top, generator=g) * 2.5 + 0.1             # (a weight on the output would enter once instead of squared)
    up, dn = (torch.stack([t[f"e{e}.{k}"] for e in range(experts)]).to(DEV).to(dtype) for k in ("up", "down"))
    y = sparse_square_experts(h.to(DEV).to(dtype), up, dn, ids.to(DEV), weights.to(DEV))
    want = torch.stack([torch.stack([O.square_expert((weights[i, k].to(F64) * h[i].to(F64))[None], t, f"e{int(ids[i, k])}.")[0]
                                     for k in range(top)]) for i in range(n)])
    _close(y, want, 2e-5 if dtype == torch.float32 else 2e-2)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("ff", [40, 37])
def test_relu_square_of_a_column_range(dtype, ff):
    from lite_llama_amd.kernels.norm_act import relu_square

    torch.manual_seed(ff)
    wide = bf(torch.randn(9, ff + 8)).to(DEV).to(dtype)
    _close(relu_square(wide[:, 8:], ff), torch.relu(d(wide[:, 8:])) ** 2, 1e-6 if dtype == torch.float32 else 1e-2)


# ------------------------------------------------------------------------------------------------------------------- #
# streams
# ------------------------------------------------------------------------------------------------------------------- #
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width,streams,parts,shared", [(96, 3, 1, False), (70, 4, 3, True), (2048, 2, 2, True), (3000, 4, 1, True), (4100, 1, 1, False),
                                                      (18, 11, 4, True), (64, 8, 1, False), (64, 5, 2, True), (1024, 1, 1, True)])
def test_streams_update_mix_gather_and_norm_in_one_launch(dtype, width, streams, parts, shared):
    from lite_llama_amd.kernels.norm_act import StreamUpdate, stream_norm
    from oracle import tusasun as O

    torch.manual_seed(width + streams)
    n, eps = 7, 1e-5
    r = lambda *s: bf(torch.randn(*s)).to(DEV).to(dtype)  # noqa: E731
    x0 = torch.randn(n, width, device=DEV)
    gather, gather2, out, mix, scale, w, w2 = r(streams), r(streams), r(streams), r(streams, streams), r(width), r(width), r(width)
    first, same = stream_norm(x0, None, streams, gather, w, eps, 1.0)
    assert same is x0
    xs = d(x0)[None].repeat(streams, 1, 1)
    tol = 3e-6 if dtype == torch.float32 else 1e-2
    _close(first, O.shifted_norm(O.stream_input(xs, d(gather)), d(w), eps), tol)
    x = x0
    for k in range(3):                                                # from the one row, then in place
        y = r(n, parts, width)
        own, own_scale = (r(n, width), torch.rand(n, device=DEV)) if shared else (None, None)
        u = StreamUpdate(y, scale, mix, out, own, own_scale)
        before = x.data_ptr()
        h, x = stream_norm(x, u, streams, gather2 if k else gather, w2, eps, 1.0)
        assert (x.data_ptr() == before) == (k > 0) and tuple(x.shape) == (n, streams, width)
        res = d(y).sum(1) + (d(own_scale)[:, None] * d(own) if shared else 0.0)
        xs = O.stream_update(xs, res * d(scale), d(mix), d(out))
        _close(x.transpose(0, 1), xs, 3e-6)
        _close(h, O.shifted_norm(O.stream_input(xs, d(gather2 if k else gather)), d(w2), eps), 5e-6 if dtype == torch.float32 else 1e-2)
    total, _ = stream_norm(x, None, streams, None, w, eps)             # the plain sum, a plain weight
    _close(total, O.rms(xs.sum(0), eps) * d(w), 5e-6 if dtype == torch.float32 else 1e-2)
    picked = torch.tensor([5, 1], device=DEV)
    sub = x[picked].contiguous()
    h, sub = stream_norm(sub, u.rows(picked), streams, None, w, eps, 1.0)
    want = O.stream_update(xs, res * d(scale), d(mix), d(out))[:, [5, 1]]
    _close(sub.transpose(0, 1), want, 3e-6)


# ------------------------------------------------------------------------------------------------------------------- #
# whole models
# ------------------------------------------------------------------------------------------------------------------- #
def _model(tmp_path_factory, name, dtype):
    from lite_llama_amd.weights import load_pretrained

    if (name, dtype) not in _MODELS:
        cfg = T.on_disk(T.CONFIGS[name])
        tens = T.tensors(T.CONFIGS[name], seed=17)
        folder = L.write(tmp_path_factory.mktemp("tusasun") / name, cfg, tens)
        _MODELS[(name, dtype)] = (load_pretrained(folder, device=DEV, dtype=dtype), cfg, tens, folder)
    return _MODELS[(name, dtype)]


@pytest.mark.parametrize("name", sorted(T.CONFIGS))
def test_whole_prompt_layers_and_logits(tmp_path_factory, name):
    from lite_llama_amd.executor.ragged import RaggedRunner
    from oracle import tusasun as O

    model, cfg, tens, _ = _model(tmp_path_factory, name, torch.float32)
    toks = L.prompt(cfg, 45)
    want, layers = O.forward(toks, tens, cfg)
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
    """Portions down to two tokens, pure token-by-token decoding from the first token on, and a long portion followed by
    decoding; pages of 8 tokens, so portions, taps, buckets, token tiles and pages start and end inside one another."""
    from lite_llama_amd.executor.ragged import RaggedRunner
    from oracle import tusasun as O

    model, cfg, tens, _ = _model(tmp_path_factory, name, torch.float32)
    toks = L.prompt(cfg, 58, seed=1)
    want, _ = O.forward(toks, tens, cfg)
    runner = RaggedRunner(model, 64, 2, block_size=8, device=DEV)
    _close(_feed(runner, runner.admit(), toks, sizes), want, 2e-5)
    runner.check_errors()


@pytest.mark.parametrize("name", ["mix", "odd"])
def test_unequal_requests_in_one_batch_equal_each_alone_and_freed_pages_and_slots_are_used_again(tmp_path_factory, name):
    """Four requests of different lengths ride together in changing portions, three slots and a pool that only holds them
    because finished requests give their pages back; a late request takes over a used slot (with the state and the carried
    rows its last owner left) and used pages."""
    from lite_llama_amd.executor.ragged import RaggedRunner
    from oracle import tusasun as O

    model, cfg, tens, _ = _model(tmp_path_factory, name, torch.float32)
    lens = {"a": 41, "b": 9, "c": 26, "d": 33}
    toks = {k: L.prompt(cfg, n, seed=ord(k)) for k, n in lens.items()}
    want = {k: O.forward(v, tens, cfg)[0] for k, v in toks.items()}
    runner = RaggedRunner(model, 96, 3, block_size=8, device=DEV)      # 12 pages: a + b + c need 12, d needs 5
    sizes = {"a": [5, 1, 1, 9, 2, 30], "b": [2, 1, 3, 1, 1, 1], "c": [1, 13, 2, 2, 8], "d": [16, 1, 1, 15]}
    at, slot, got, k = {x: 0 for x in lens}, {}, {x: [] for x in lens}, 0
    waiting, live = ["a", "b", "c", "d"], []
    while waiting or live:
        while waiting and runner.free_slots and sum(runner.blocks_for(lens[x]) for x in live + waiting[:1]) <= runner.total_blocks:
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


@pytest.mark.parametrize("name", ["mix", "wide"])
def test_long_prompts_and_long_decoding_over_many_pages(tmp_path_factory, name):
    """A prompt long enough for the chunked recurrence and for several attention partitions, decoding past the last bucket's edge."""
    from lite_llama_amd.executor.ragged import RaggedRunner
    from oracle import tusasun as O

    model, cfg, tens, _ = _model(tmp_path_factory, name, torch.float32)
    toks = L.prompt(cfg, 420, seed=5)
    want, _ = O.forward(toks, tens, cfg)
    runner = RaggedRunner(model, 896, 2, block_size=16, device=DEV)
    _close(_feed(runner, runner.admit(), toks, [140, 129, 6, 1]), want, 3e-5)
    _close(_feed(runner, runner.admit(), toks, [420]), want, 3e-5)


@pytest.mark.parametrize("name", sorted(T.CONFIGS))
def test_bfloat16_model_tracks_the_oracle_and_its_own_portions(tmp_path_factory, name):
    from lite_llama_amd.executor.ragged import RaggedRunner
    from oracle import tusasun as O

    model, cfg, tens, _ = _model(tmp_path_factory, name, torch.bfloat16)
    toks = L.prompt(cfg, 70, seed=2)
    want, _ = O.forward(toks, tens, cfg)
    runner = RaggedRunner(model, 160, 2, block_size=16, device=DEV)
    whole = _feed(runner, runner.admit(), toks, [70]).float().cpu()
    parts = _feed(runner, runner.admit(), toks, [2, 9, 1, 1, 30, 1]).float().cpu()
    spread = want.std().item()
    # medians over the tokens: a token whose router sees two experts within a rounding step of each other may choose the other
    err = lambda a, b: (a.to(F64) - b.to(F64)).pow(2).mean(-1).sqrt().median().item()   # noqa: E731
    assert err(whole, want) < 0.06 * spread
    assert err(parts, whole) < 0.04 * spread


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
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
    from oracle import tusasun as O

    model, cfg, tens, _ = _model(tmp_path_factory, "odd", torch.float32)
    prompts = [L.prompt(cfg, n, seed=n) for n in (3, 19, 1, 11, 7)]
    engine = GenerationEngine(model, max_tokens=96, max_requests=3, block_size=8, max_step_tokens=10, device=DEV)
    outs = engine.generate(prompts, SamplingParams(max_new_tokens=6))
    for p, o in zip(prompts, outs):
        assert o == O.greedy(p, 6, tens, cfg)
    captured = GenerationEngine(model, max_tokens=96, max_requests=3, block_size=8, max_step_tokens=10, device=DEV, capture_decode=True)
    assert captured.generate(prompts, SamplingParams(max_new_tokens=6)) == outs and captured.runner.replays > 0
    assert engine.runner.cache.free_blocks == engine.runner.total_blocks and engine.runner.free_slots == 3
    sampled = engine.generate(prompts[:2], SamplingParams(max_new_tokens=5, temperature=0.8, top_p=0.9, repetition_penalty=1.2))
    assert [len(s) for s in sampled] == [5, 5] and all(0 <= t < cfg["vocab"] for s in sampled for t in s)


def test_command_line_generate_and_trace_replay(tmp_path_factory, tmp_path):
    from oracle import tusasun as O

    _, cfg, tens, folder = _model(tmp_path_factory, "wide", torch.float32)
    prompt = L.prompt(cfg, 9, seed=4)
    env = dict(os.environ, PYTHONPATH=ROOT)
    done = subprocess.run([sys.executable, "-m", "lite_llama_amd", "generate", "--model", folder, "--dtype", "float32",
                           "--prompt-ids", ",".join(map(str, prompt)), "--max-new-tokens", "4"],
                          capture_output=True, text=True, env=env, cwd=ROOT, timeout=300)
    assert done.returncode == 0, done.stderr[-2000:]
    line = json.loads(done.stdout.strip().splitlines()[-1])
    assert line["prompt"] == prompt and line["generated"] == O.greedy(prompt, 4, tens, cfg)

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

    la, lb = O.forward(a, tens, cfg)[0], O.forward(b, tens, cfg)[0]
    read = lambda i: torch.from_numpy(np.fromfile(out / f"{i}.f32", dtype="<f4")).view(-1, cfg["vocab"])   # noqa: E731
    _close(read(0), la[[0, 12]], 2e-5)
    _close(read(1), lb[[5]], 2e-5)
    assert not (out / "2.f32").exists()
    _close(read(3), torch.stack([la[30], lb[5]]), 2e-5)


def _random_config(seed):
    """A configuration drawn from the whole range the reader takes: one to five layers of the three mixers in any order, head
    counts and widths with and without the matrix-core forms' multiples, one to seven streams, one to six taps, loops over any
    span, layers without a feed-forward."""
    import random

    r = random.Random(seed)
    layers = []
    for _ in range(r.randint(1, 5)):
        experts = r.randint(1, 9)
        mlp = T.moe(experts, r.randint(1, experts), r.choice([8, 12, 24, 40]), r.choice([8, 14, 32])) if r.random() < 0.8 else None
        mixer = r.choice(["attention", "delta", "rglru"])
        g = r.choice([1, 2, 3])
        if mixer == "attention":
            rows = r.choice([2, 4, 8, 16, 32])
            layers.append(T.attention(g * r.choice([1, 2, 4, 5]), g, r.choice([8, 16, 32, 64, 12, 20, 128]), r.choice([8, 16, 24, 10, 48]), rows,
                                      rows // 2 + r.choice([0.5, 1, 7, 30, 200]), mlp=mlp, cap=r.choice([1.5, 8.0, 50.0])))
        elif mixer == "delta":
            layers.append(T.delta(g * r.choice([1, 2, 3]), g, r.choice([8, 16, 32, 12, 64, 100]), r.choice([8, 16, 10, 40, 72]), r.randint(1, 6),
                                  r.choice([1, 4, 16, 5]), r.choice([1, 8, 3]), mlp=mlp))
        else:
            blocks = r.choice([1, 2, 3, 5])
            layers.append(T.rglru(blocks * r.choice([1, 4, 8, 10, 24]), blocks, r.randint(1, 6), mlp=mlp))
    loop = None
    if r.random() < 0.6:
        start = r.randint(0, len(layers) - 1)
        loop = (start, r.randint(start + 1, len(layers)), r.randint(1, 3))
    return T.config(layers, width=r.choice([32, 48, 58, 88]), vocab=r.randint(20, 300), streams=r.randint(1, 7), loop=loop,
                    eps=r.choice([1e-5, 1e-6, 1e-3]))


@pytest.mark.parametrize("seed", range(12))
def test_random_configurations_whole_in_portions_decoded_and_side_by_side(tmp_path, seed):
    from lite_llama_amd.executor.ragged import RaggedRunner
    from lite_llama_amd.weights import load_pretrained
    from oracle import tusasun as O

    cfg = _random_config(seed)
    tens = T.tensors(cfg, seed=seed)
    cfg = T.on_disk(cfg)
    model = load_pretrained(L.write(tmp_path / "m", cfg, tens), device=DEV, dtype=torch.float32)
    a, b = L.prompt(cfg, 90, seed=seed), L.prompt(cfg, 37, seed=seed + 50)
    wa, wb = O.forward(a, tens, cfg)[0], O.forward(b, tens, cfg)[0]
    runner = RaggedRunner(model, 256, 3, block_size=16, device=DEV)
    _close(_feed(runner, runner.admit(), a, [90]), wa, 3e-5)
    _close(_feed(runner, runner.admit(), a, [2, 1, 7, 3, 1, 30, 1]), wa, 3e-5)
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
    _close(torch.cat(got_a), wa, 3e-5)
    _close(torch.cat(got_b), wb, 3e-5)
