"""Throughput and per-kernel roofline fractions of the Tusasun design (gated delta rule, real-gated recurrence, capped attention
with a bias per distance, squared-relu experts weighted at their input, several mixed residual streams) beside the closest model
of the framework at equal sizes -- the layered family's Nivotar (gated linear attention, windowed attention beside a state-space
mixer, gated experts over the same ragged runner, paged state cache and fp32 residual stream) -- ``python bench.py --tusasun``.

Model level: prefill tokens/s (whole prompts in one ragged step) and decode tokens/s (one token per sequence and step; eager
and captured) for four layers at the widths of a small production model, random weights.  Kernel level: every new kernel of the
design timed alone (HIP events around a loop of launches) with its algorithmic bytes and flops, next to the like kernel of the
framework's other models at the same shape; ``far`` = how many times further from its roofline (HBM 8 TB/s or 2.5 PFLOP/s dense
16-bit MFMA, whichever bounds it) the new kernel is than its counterpart."""

from __future__ import annotations

import torch

from .layered_bench import _entry, _time
from .nivotar_bench import model_points
from .rukedra_bench import _step_of


def kernel_table(dev, dtype, width, streams, heads, kv_heads, dim, vdim, rows, far, cap, d_heads, d_kv, d_dim, d_vdim, taps, rank, gate_rank,
                 lru, blocks, experts, top, eff, shared, prefill=(8, 512), decode=(32, 1024)):
    from lite_llama_amd.kernels.attention import ragged_attention
    from lite_llama_amd.kernels.fused_moe import group_router, sparse_glu_experts, sparse_square_experts
    from lite_llama_amd.kernels.norm_act import GatedUpdate, StreamUpdate, gated_group_norm, glu_act, relu_square, stream_norm
    from lite_llama_amd.kernels.recurrent import conv_act, delta_scan, gated_out_norm, linear_scan, mingru_scan, rglru_scan
    from lite_llama_amd.model_layers import distance_buckets

    es = torch.empty(0, dtype=dtype).element_size()
    out = []
    rnd = lambda *shape: torch.randn(*shape, device=dev).to(dtype)   # noqa: E731
    for phase, (batch, length) in (("prefill", prefill), ("decode", decode)):
        first, count = (0, length) if phase == "prefill" else (length - 1, 1)
        n = batch * count
        step = _step_of(dev, batch, first, count)
        iters = 5 if phase == "prefill" else 20
        state_io = 2 if phase == "decode" else 0

        def add(name, t, moved, flops, like=None):
            out.append(dict(_entry(name, t, moved, flops, like), phase=phase))

        # gated delta rule (+ read-out norm) vs linear attention with a decay per key entry (+ the same norm)
        h, dk, dv = d_heads, d_dim, d_vdim
        qk, gk, vw = d_kv * dk, h * dk, h * dv
        q, k, v, z, gate, b = rnd(n, qk), rnd(n, qk), rnd(n, vw), rnd(n, gk) - 2, rnd(n, vw), rnd(n, h)
        dt_bias, a_log, w_head = rnd(gk), rnd(h) * 0.3, rnd(dv)
        st = torch.zeros(batch, h, dk, dv, device=dev)
        t = _time(lambda: gated_out_norm(delta_scan(q, k, v, h, dk, dv, step, st, gate=z, dt_bias=dt_bias, a_log=a_log, beta=b, qk_heads=d_kv,
                                                    q_scale=dk ** -0.5), w_head, 1e-6, parts=h, gate=gate, gate_kind="sigmoid"), iters=iters)
        t_alone = _time(lambda: delta_scan(q, k, v, h, dk, dv, step, st, gate=z, dt_bias=dt_bias, a_log=a_log, beta=b, qk_heads=d_kv,
                                           q_scale=dk ** -0.5), iters=iters)
        lq, lk = rnd(n, gk) * 0.3, rnd(n, gk) * 0.3
        t_old = _time(lambda: gated_out_norm(linear_scan(lq, lk, v, h, dk, dv, step, st, q_scale=dk ** -0.5, gate=z, gate_bias=dt_bias, tau=8.0),
                                             w_head, 1e-6, parts=h, gate=gate, gate_kind="silu"), iters=iters)
        state_bytes = state_io * batch * h * dk * dv * 4
        like = _entry("linear_scan (decay per key entry) + gated_out_norm", t_old, n * (3 * gk + 3 * vw) * es + state_bytes, n * h * 4.0 * dk * dv)
        moved, flops = n * (2 * qk + gk + 3 * vw + h) * es + state_bytes, n * h * 6.0 * dk * dv
        add(f"delta_scan + gated_out_norm ({h} on {d_kv} x {dk} x {dv})", t, moved, flops, like)
        add("delta_scan alone", t_alone, moved, flops)

        # real-gated recurrence vs minGRU
        u, gates, y = rnd(n, lru), rnd(n, blocks, 2, lru // blocks), rnd(n, lru)
        rb, ib, lam, zb = rnd(lru), rnd(lru), rnd(lru) - 3, rnd(lru)
        st1 = torch.zeros(batch, lru, device=dev)
        t = _time(lambda: rglru_scan(u, gates, rb, ib, lam, y, step, st1), iters=iters)
        zxg = rnd(n, 3 * lru)
        t_old = _time(lambda: mingru_scan(zxg, lru, zb, rb, step, st1), iters=iters)
        like = _entry("mingru_scan", t_old, n * 4 * lru * es + state_io * batch * lru * 4, 0)
        add(f"rglru_scan ({lru} channels, {blocks} blocks)", t, n * 5 * lru * es + state_io * batch * lru * 4, 0, like)
        gw = rnd(blocks, lru // blocks, 2 * (lru // blocks))
        gout = torch.empty(n, blocks, 2 * (lru // blocks), device=dev, dtype=dtype)
        t = _time(lambda: torch.bmm(u.view(n, blocks, -1).transpose(0, 1), gw, out=gout.transpose(0, 1)), iters=iters)
        add("gate product (library batched GEMM)", t, n * 3 * lru * es + gw.numel() * es, n * 4.0 * lru * (lru // blocks))

        # convolution without / with silu
        channels = 2 * qk + vw
        wide = rnd(n, channels + 64)
        cw, cb = rnd(channels, taps), rnd(channels)
        cst = torch.zeros(2, batch, taps - 1, channels, device=dev, dtype=dtype)
        t = _time(lambda: conv_act(wide, cw, cb, step, cst, act=None))
        t_old = _time(lambda: conv_act(wide, cw, cb, step, cst))
        add(f"conv_act without activation ({channels} channels, {taps} taps)", t, n * channels * es * 2, 0,
            _entry("conv_act with silu", t_old, n * channels * es * 2, 0))

        # capped, biased attention vs the same attention without
        ctx = first + count
        kc, vc = rnd(batch * ctx, kv_heads, dim), rnd(batch * ctx, kv_heads, vdim)
        table = torch.arange(batch * ctx, dtype=torch.int32, device=dev).view(batch, ctx)
        qa = rnd(n, heads, dim)
        bias = torch.randn(heads, len(distance_buckets(rows, far)), device=dev)
        t = _time(lambda: ragged_attention(qa, kc, vc, dim ** -0.5, step, table, cap=cap, dist_bias=bias), iters=iters)
        t_old = _time(lambda: ragged_attention(qa, kc, vc, dim ** -0.5, step, table), iters=iters)
        pairs = batch * (count * (count + 1) / 2 if phase == "prefill" else ctx)
        moved = (n * heads * (dim + vdim) + batch * ctx * kv_heads * (dim + vdim)) * es
        flops = pairs * heads * 2.0 * (dim + vdim)
        add(f"ragged_attention, capped + distance bias ({heads} on {kv_heads} x {dim} / {vdim})", t, moved, flops,
            _entry("ragged_attention", t_old, moved, flops))

        # streams: mix + gather + norm vs norm of the result + residual add + cast
        x = torch.randn(n, streams, width, device=dev)
        x1 = torch.randn(n, width, device=dev)
        w, gather, mix = rnd(width), rnd(streams), torch.eye(streams, device=dev).to(dtype)
        for slots in (1, top):
            extra = slots > 1
            own, own_scale = (rnd(n, width), torch.rand(n, device=dev)) if extra else (None, None)
            upd = StreamUpdate(rnd(n, slots, width), w, mix, gather * 0.01, own, own_scale)
            t = _time(lambda: stream_norm(x, upd, streams, gather, w, 1e-6, 1.0))
            old = GatedUpdate(rnd(n, slots, width), w, shared=own, shared_scale=own_scale)
            t_old = _time(lambda: gated_group_norm(x1, old, None, 1e-6, plain=dtype))
            like = _entry(f"gated_group_norm ({slots} rows)", t_old, n * width * (8 + (slots + 1 + extra) * es), 0)
            add(f"stream_norm ({streams} streams, {slots} result rows{' + shared row' if extra else ''})", t,
                n * width * (8 * streams + (slots + 1 + extra) * es), 0, like)

        # experts and router
        hh = rnd(n, width)
        wr, sg = rnd(experts, width) * width ** -0.5, rnd(1, width) * width ** -0.5
        t = _time(lambda: group_router(hh, wr, top, scoring="sigmoid_plain", extra_weight=sg))
        t_old = _time(lambda: group_router(hh, wr, top, extra_weight=sg))
        moved, flops = (n + experts + 1) * width * es, n * (experts + 1) * width * 2.0
        add("group_router (plain sigmoid scores + shared scale)", t, moved, flops, _entry("group_router (renormalised)", t_old, moved, flops))
        ids, wts, _ = group_router(hh, wr, top, scoring="sigmoid_plain", extra_weight=sg)
        up, gu, dn = rnd(experts, eff, width) * 0.02, rnd(experts, 2 * eff, width) * 0.02, rnd(experts, width, eff) * 0.02
        t = _time(lambda: sparse_square_experts(hh, up, dn, ids, wts), iters=iters)
        t_old = _time(lambda: sparse_glu_experts(hh, gu, dn, ids, wts), iters=iters)
        used = min(experts, n * top)
        act = n * (top * (2 * eff + width) + width) * es
        like = _entry("sparse_glu_experts", t_old, used * 3 * eff * width * es + act, n * top * 6.0 * eff * width)
        add(f"sparse_square_experts ({experts} experts, top {top}, ff {eff})", t, used * 2 * eff * width * es + act, n * top * 4.0 * eff * width, like)
        sh = rnd(n, 2 * shared)
        t = _time(lambda: relu_square(sh, shared))
        t_old = _time(lambda: glu_act(sh, shared, "silu"))
        add("relu_square", t, n * shared * 2 * es, 0, _entry("glu_act (silu)", t_old, n * shared * 3 * es, 0))
    return out


def _geometries(width, streams, heads, kv_heads, dim, vdim, rows, far, cap, d_heads, d_kv, d_dim, d_vdim, taps, rank, gate_rank, lru, blocks,
                experts, top, eff, shared, vocab):
    """``(label, stack)`` twice: delta, delta, rglru, attention beside gla, gla, gla, attention + state-space, all with experts."""
    from lite_llama_amd.model_layers import LayeredGeometry, LayerSpec, MixerSpec, MlpSpec, StateSpaceSpec

    delta = MixerSpec("channel_delta", heads=d_heads, dim=d_dim, vdim=d_vdim, kv_heads=d_kv, conv_taps=taps, decay_rank=rank, gate_rank=gate_rank)
    rec = MixerSpec("rglru", width=lru, blocks=blocks, conv_taps=taps)
    att = MixerSpec("distance_attention", heads=heads, dim=dim, vdim=vdim, kv_heads=kv_heads, scale=dim ** -0.5, softcap=cap, bias_rows=rows,
                    bias_max=far)
    moe = MlpSpec("moe", ff=eff, act="relu_square", experts=experts, top=top, scoring="sigmoid_plain", shared_ff=shared)
    new = LayeredGeometry("tusasun", vocab, width, 1e-6, tuple(LayerSpec(m, ff=eff, mlp_kind="moe", mlp=moe) for m in (delta, delta, rec, att)),
                          token_shift=False, loop_mix=False, streams=streams, norm_base=1.0)
    gla = MixerSpec("gla", heads=d_heads, dim=d_dim, vdim=d_vdim, tau=8.0, decay_rank=rank)
    ssd_heads = lru // 64
    par = MixerSpec("attention_ssd", heads=heads, dim=dim, vdim=vdim, kv_heads=kv_heads, scale=dim ** -0.5, window=1 << 20,
                    ssd=StateSpaceSpec(ssd_heads, 64, 64, 4, taps, 4), branch_scales=(0.5, 1.5))
    glu = MlpSpec("moe", ff=eff, act="clamped", limit=7.0, experts=experts, top=top, scoring="softmax_all")
    old = LayeredGeometry("nivotar", vocab, width, 1e-6, tuple(LayerSpec(m, ff=eff, mlp_kind="moe", mlp=glu) for m in (gla, gla, gla, par)),
                          token_shift=False, tied_head=True, post_norm=True)
    return new, old


SIZES = {
    # widths of a 2B-class model: 16 query heads on 4 key/value heads of 128; 16 delta heads of 128 x 128; 2048 recurrent channels
    # in 16 blocks; 32 experts, 4 chosen, and a shared one; four streams
    "compact": dict(width=2048, streams=4, heads=16, kv_heads=4, dim=128, vdim=128, rows=32, far=128.0, cap=30.0, d_heads=16, d_kv=16, d_dim=128,
                    d_vdim=128, taps=4, rank=128, gate_rank=128, lru=2048, blocks=16, experts=32, top=4, eff=704, shared=1408),
    # a wider model: values of 96, grouped delta heads with a narrow key, wider gate blocks, more and smaller experts, two streams
    "wide": dict(width=3072, streams=2, heads=24, kv_heads=8, dim=128, vdim=96, rows=32, far=1024.0, cap=50.0, d_heads=24, d_kv=12, d_dim=64,
                 d_vdim=128, taps=4, rank=64, gate_rank=64, lru=4096, blocks=16, experts=64, top=8, eff=512, shared=1024),
}


def run(dtype_name="bf16", sizes=("compact", "wide"), kernels=True):
    dev = torch.device("cuda", 0)
    dtype = {"bf16": torch.bfloat16, "f16": torch.float16, "f32": torch.float32}[dtype_name]
    line = {"metric": "tusasun_throughput", "dtype": dtype_name, "data": "synthetic", "points": {}}
    for name in sizes:
        s = SIZES[name]
        point = {"sizes": dict(s, layers=4, vocab=32768),
                 "model": model_points(dev, dtype, _geometries(vocab=32768, **s), labels=("tusasun", "nivotar"))}
        if kernels:
            point["kernels"] = kernel_table(dev, dtype, **s)
        line["points"][name] = point
        torch.cuda.empty_cache()
    return line
