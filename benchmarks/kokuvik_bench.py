"""Throughput and per-kernel roofline fractions of the Kokuvik design (retention; windowed attention with kept first keys, a learned
sink, a gate per head and keys / values shared between layers; squared-relu and grouped-softmax expert feed-forwards beside the
mixer) beside the closest models of the framework at equal sizes -- the layered family's Nivotar (linear attention with a fixed decay
per head, windowed attention beside a state-space mixer, gated experts) and Fekanex (the same parallel layer with windowed
attention everywhere) over the same ragged runner, paged state cache and fp32 residual stream -- ``python bench.py --kokuvik``.

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


def kernel_table(dev, dtype, width, heads, kv_heads, dim, vdim, rot, window, keep, r_heads, r_dim, r_vdim, ff, experts, groups, top, eff, shared,
                 prefill=(8, 512), decode=(32, 1024)):
    from lite_llama_amd.kernels.attention import conv_rope_cache, ragged_attention, rotation_table, rownorm_rope_cache
    from lite_llama_amd.kernels.fused_moe import group_router
    from lite_llama_amd.kernels.norm_act import glu_act, relu_square
    from lite_llama_amd.kernels.recurrent import gated_out_norm, linear_scan, retention

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

        # retention (rotation, scan, head norm, gate) vs the scan with a fixed decay per head + read-out norm and gate
        for h, dk, dv, what in ((r_heads, r_dim, r_vdim, ""), (r_heads // 2, 256, 256, ", wide heads")):
            qk, vw = h * dk, h * dv
            rows = rnd(n, 2 * qk + 2 * vw) * 0.3
            st = torch.zeros(batch, h, dk, dv, device=dev)
            dec = torch.rand(h, device=dev) * 0.1 + 0.9
            freq = torch.rand(dk // 2, device=dev)
            table = rotation_table(step, freq, dk // 2)
            q, k, v, g = rows[:, :qk], rows[:, qk:2 * qk], rows[:, 2 * qk:2 * qk + vw], rows[:, 2 * qk + vw:]
            t = _time(lambda: retention(q, k, v, h, dk, dv, step, st, decay=dec, gate=g, eps=1e-6, k_scale=dk ** -0.5, half=dk // 2,
                                        rot_table=table), iters=iters)
            t_old = _time(lambda: gated_out_norm(linear_scan(q, k, v, h, dk, dv, step, st, head_decay=dec), None, 1e-6, parts=h, gate=g,
                                                 gate_kind="silu"), iters=iters)
            moved, flops = n * (2 * qk + 3 * vw) * es + state_io * batch * h * dk * dv * 4, n * h * 4.0 * dk * dv
            add(f"retention ({h} x {dk} x {dv}{what})", t, moved + n * dk * 4, flops,
                _entry("linear_scan (fixed decay) + gated_out_norm (no rotation)", t_old, moved, flops))

        # rotation + cache write, and of queries alone, vs the half-split rotation + cache write
        channels = (heads + kv_heads) * dim + kv_heads * vdim
        ctx = first + count
        kc, vc = rnd(batch * ctx, kv_heads, dim), rnd(batch * ctx, kv_heads, vdim)
        freq = torch.rand(rot // 2, device=dev)
        table = rotation_table(step, freq, rot // 2)
        wide = rnd(n, channels + ff + 8)
        t = _time(lambda: conv_rope_cache(wide, heads, kv_heads, dim, vdim, step, kc, vc, freq=freq, pairs=rot // 2, rot_table=table))
        t_q = _time(lambda: conv_rope_cache(wide, heads, 0, dim, vdim, step, None, None, freq=freq, pairs=rot // 2, rot_table=table))
        t_old = _time(lambda: rownorm_rope_cache(wide, heads, kv_heads, dim, vdim, step, kc, vc, freq=freq, pairs=rot // 2))
        like = _entry("rownorm_rope_cache (no norms)", t_old, n * channels * 2 * es, 0)
        add("conv_rope_cache (rotation + cache write)", t, n * (channels * 2 * es + rot * 4), 0, like)
        add("conv_rope_cache (queries alone)", t_q, n * (heads * dim * 2 * es + rot * 4), 0, like)

        # attention with a gate per head vs the same without
        tt = torch.arange(batch * ctx, dtype=torch.int32, device=dev).view(batch, ctx)
        qa, sink = rnd(n, heads, dim), rnd(heads)
        gate = rnd(n, channels + heads)[:, channels:]
        mixed = torch.empty(n, heads * vdim + ff, device=dev, dtype=dtype)
        kw = dict(sink=sink, window=window, keep_first=keep, out=mixed[:, :heads * vdim])
        t = _time(lambda: ragged_attention(qa, kc, vc, dim ** -0.5, step, tt, head_gate=gate, **kw), iters=iters)
        t_old = _time(lambda: ragged_attention(qa, kc, vc, dim ** -0.5, step, tt, **kw), iters=iters)
        span = min(window + keep, length)
        pairs = batch * (length * span - span * (span - 1) / 2) if phase == "prefill" else batch * span
        moved = (n * heads * (dim + vdim) + batch * (ctx if phase == "prefill" else span) * kv_heads * (dim + vdim)) * es
        flops = pairs * heads * 2.0 * (dim + vdim)
        add(f"ragged_attention (sink, window {window} + {keep} kept, gate per head)", t, moved + n * heads * es, flops,
            _entry("ragged_attention (sink, window, kept keys)", t_old, moved, flops))

        # router and activation
        hh = rnd(n, width)
        wr = rnd(experts, width) * width ** -0.5
        t = _time(lambda: group_router(hh, wr, top, groups, max(groups // 2, 1), scoring="softmax_groups"))
        t_old = _time(lambda: group_router(hh, wr, top, groups, max(groups // 2, 1)))
        moved, flops = (n + experts) * width * es, n * experts * width * 2.0
        add(f"group_router (softmax over {experts}, {groups} groups)", t, moved, flops, _entry("group_router (sigmoid, groups)", t_old, moved, flops))
        t = _time(lambda: relu_square(wide[:, channels:channels + ff], ff, out=mixed[:, heads * vdim:]))
        act = rnd(n, 2 * ff)
        t_old = _time(lambda: glu_act(act, ff, "silu", out=mixed[:, heads * vdim:]))
        add("relu_square (column ranges)", t, n * ff * 2 * es, 0, _entry("glu_act (silu)", t_old, n * ff * 3 * es, 0))
    return out


def _geometries(width, heads, kv_heads, dim, vdim, rot, window, keep, r_heads, r_dim, r_vdim, ff, experts, groups, top, eff, shared, vocab):
    """Three stacks of four layers: attention + dense, retention + experts, attention over the first layer's keys + experts, retention +
    experts; the same with Nivotar's layers (windowed attention beside a state-space mixer for the attention layers, linear
    attention with a fixed decay for retention) and with Fekanex's (attention in every layer)."""
    from lite_llama_amd.model_layers import LayeredGeometry, LayerSpec, MixerSpec, MlpSpec, RotarySpec, StateSpaceSpec

    stack = lambda pairs: tuple(LayerSpec(m, ff=f.ff, mlp_kind=f.kind, mlp=f) for m, f in pairs)   # noqa: E731
    at = dict(heads=heads, dim=dim, vdim=vdim, kv_heads=kv_heads, scale=dim ** -0.5, window=window)
    decay = tuple(1.0 - 2.0 ** -(5 + 3 * i / max(r_heads - 1, 1)) for i in range(r_heads))
    own = MixerSpec("window_attention", rotary=RotarySpec(rot, 10000.0, 8.0, 4096.0, low=1.0, high=4.0), keep_first=keep, **at)
    borrowed = MixerSpec("window_attention", rotary=own.rotary, keep_first=keep, kv_from=0, **at)
    ret = MixerSpec("retention", heads=r_heads, dim=r_dim, vdim=r_vdim, rotary=RotarySpec(r_dim, 10000.0), decay=decay)
    dense = MlpSpec("dense", ff=ff, act="relu_square", bias=True)
    moe = MlpSpec("moe", ff=eff, act="silu", experts=experts, top=top, scoring="softmax_groups", group_count=groups,
                  group_keep=max(groups // 2, 1), shared_ff=shared)
    new = LayeredGeometry("kokuvik", vocab, width, 1e-6, stack(((own, dense), (ret, moe), (borrowed, moe), (ret, moe))), token_shift=False,
                          parallel=True)
    par = MixerSpec("attention_ssd", rotary=RotarySpec(rot, 10000.0), ssd=StateSpaceSpec(r_heads, r_vdim, 64, 4, 4, 4), branch_scales=(0.5, 1.5),
                    **at)
    lin = MixerSpec("decay_linear", heads=r_heads, dim=r_dim, vdim=r_vdim, decay=decay)
    niv_moe = MlpSpec("moe", ff=eff, act="clamped", limit=7.0, experts=experts, top=top, scoring="softmax_all")
    niv = LayeredGeometry("nivotar", vocab, width, 1e-6,
                          stack(((par, MlpSpec("dense", ff=ff, act="silu", bias=True)), (lin, niv_moe), (par, niv_moe), (lin, niv_moe))),
                          token_shift=False, tied_head=True, post_norm=True)
    conv = MixerSpec("conv_attention", rotary=RotarySpec(rot, 10000.0, 8.0, 4096.0, 32.0, 1.0), keep_first=keep, bias=True, conv_taps=4,
                     unit_norm=True, unit_sink=True, value_mix=True, **at)
    fek_moe = MlpSpec("moe", ff=eff, act="silu", experts=experts, top=top, scoring="softmax_chosen")
    fek = LayeredGeometry("fekanex", vocab, width, 1e-6,
                          stack(((conv, MlpSpec("dense", ff=ff, act="clamped", limit=7.0)), (conv, fek_moe), (conv, fek_moe), (conv, fek_moe))),
                          token_shift=False, parallel=True, tied_head=True)
    return new, niv, fek


SIZES = {
    # widths of a 2B-class model: 16 query heads on 4 key/value heads of 128, a window of 256 keys plus 4 kept; 16 retention heads of
    # 128 x 128; 32 experts in 4 groups, 4 chosen, and a shared one
    "compact": dict(width=2048, heads=16, kv_heads=4, dim=128, vdim=128, rot=64, window=256, keep=4, r_heads=16, r_dim=128, r_vdim=128, ff=5632,
                    experts=32, groups=4, top=4, eff=704, shared=1408),
    # a wider model: values of 96, a window of 512 plus 16 kept; 24 retention heads with narrow keys; more and smaller experts
    "wide": dict(width=3072, heads=24, kv_heads=8, dim=128, vdim=96, rot=128, window=512, keep=16, r_heads=24, r_dim=64, r_vdim=128, ff=8192,
                 experts=64, groups=8, top=8, eff=512, shared=1024),
}


def run(dtype_name="bf16", sizes=("compact", "wide"), kernels=True):
    dev = torch.device("cuda", 0)
    dtype = {"bf16": torch.bfloat16, "f16": torch.float16, "f32": torch.float32}[dtype_name]
    line = {"metric": "kokuvik_throughput", "dtype": dtype_name, "data": "synthetic", "points": {}}
    for name in sizes:
        s = SIZES[name]
        point = {"sizes": dict(s, layers=4, vocab=32768),
                 "model": model_points(dev, dtype, _geometries(vocab=32768, **s), labels=("kokuvik", "nivotar", "fekanex"))}
        if kernels:
            point["kernels"] = kernel_table(dev, dtype, **s)
        line["points"][name] = point
        torch.cuda.empty_cache()
    return line
