"""Small random Tusasun checkpoints for tests: configurations, tensors under the checkpoint's names (values exactly
representable in bfloat16, so a bf16 file holds the same numbers the float64 oracle reads).  Files are written with
``tests._layered.write``."""

import torch


def attention(heads, kv_heads, dim, vdim, rows, bias_max, mlp=None, scale=None, cap=15.0):
    """(``rows`` is not part of a checkpoint's configuration: it is the row count of ``mix.rel`` and read from there.)"""
    return {"type": "attention", "mlp": mlp, "_rows": rows, "mixer": {
        "heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale if scale is not None else 1.5 * dim ** -0.5,
        "softcap": cap, "bias_max": bias_max}}


def delta(heads, kv_heads, dim, vdim, conv, rank, gate_rank, mlp=None):
    """(The two ranks are the row counts of ``mix.a1`` and ``mix.g1``.)"""
    return {"type": "channel_delta", "mlp": mlp, "_ranks": (rank, gate_rank),
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


def rglru(width, blocks, conv, mlp=None):
    return {"type": "rglru", "mlp": mlp, "mixer": {"width": width, "blocks": blocks, "conv": conv}}


def moe(experts, top, ff, shared):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}, "shared": {"ff": shared}}


def config(layers, width, vocab, streams, loop=None, eps=1e-5):
    cfg = {"architecture": "Tusasun", "layers": layers, "norm": {"eps": eps}, "vocab": vocab, "width": width, "streams": streams}
    if loop is not None:
        cfg["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return cfg


def on_disk(cfg):
    """The configuration as a checkpoint folder holds it (without the test's bookkeeping keys)."""
    return dict(cfg, layers=[{k: v for k, v in entry.items() if not k.startswith("_")} for entry in cfg["layers"]])


CONFIGS = {
    # sizes that are multiples of 8 (the 16-bit matrix-core forms run); every mixer; grouped heads in both attention kinds; several
    # experts per token; the looped span holds a recurrent and an attention layer
    "mix": config([delta(4, 2, 16, 24, 4, 8, 16, mlp=moe(6, 3, 24, 40)),
                   attention(4, 2, 16, 8, 16, 40.0, mlp=moe(4, 2, 16, 24)),
                   rglru(48, 3, 3, mlp=moe(5, 1, 32, 16)),
                   attention(2, 2, 24, 16, 8, 20.0)], width=96, vocab=83, streams=4, loop=(1, 3, 2)),
    # odd sizes: heads of 12 / 10 entries (the plain attention form), widths off every 8- and 16-byte border, one tap (no carried
    # rows), six taps, all experts chosen, unequal ranks, three query heads on one key head, one block per channel pair
    "odd": config([rglru(30, 15, 6, mlp=moe(5, 5, 12, 20)),
                   delta(6, 2, 10, 6, 1, 5, 3, mlp=moe(3, 1, 10, 6)),
                   attention(3, 1, 12, 10, 6, 9.0, mlp=moe(7, 2, 14, 18), cap=4.0),
                   delta(3, 3, 14, 10, 6, 1, 7)], width=58, vocab=47, streams=3, loop=(0, 2, 3), eps=1e-6),
    # twenty query heads on one key/value head (two column tiles of the grouped decode form), wide state heads, five streams, one
    # large block, no loop
    "wide": config([attention(20, 1, 8, 8, 32, 300.0, mlp=moe(8, 4, 8, 8)),
                    delta(2, 1, 72, 40, 3, 24, 4, mlp=moe(2, 1, 40, 8)),
                    rglru(64, 1, 2)], width=64, vocab=71, streams=5),
    # everything that can be 1: one head, one entry, one block of one channel, one expert, one stream, a loop of one pass; two
    # distance buckets; a width that is no multiple of 4
    "one": config([attention(1, 1, 2, 1, 2, 2.0, mlp=moe(1, 1, 1, 1), scale=1.0), delta(1, 1, 1, 1, 1, 1, 1, mlp=moe(1, 1, 8, 1)),
                   rglru(1, 1, 1)], width=18, vocab=11, streams=1, loop=(1, 2, 1)),
}


def tensors(cfg, seed=0):
    g = torch.Generator().manual_seed(seed)
    W, V, P = cfg["width"], cfg["vocab"], cfg["streams"]

    def rnd(*shape, std=1.0, mean=0.0):
        return (torch.randn(*shape, generator=g) * std + mean).to(torch.bfloat16).float()

    def uni(*shape, lo=0.0, hi=1.0):
        return (torch.rand(*shape, generator=g) * (hi - lo) + lo).to(torch.bfloat16).float()

    def lin(out, inp, gain=1.0):
        return rnd(out, inp, std=gain * inp ** -0.5)

    t = {"embed": rnd(V, W), "final.norm": rnd(W, std=0.1), "head": lin(V, W)}
    for i, entry in enumerate(cfg["layers"]):
        p, m = f"l{i}.mix.", entry["mixer"]
        subs = (1, 2) if entry["mlp"] is not None else (1,)
        for n in subs:
            t[f"l{i}.norm{n}"], t[f"l{i}.ls{n}"] = rnd(W, std=0.1), uni(W, lo=0.3, hi=1.5)
            t[f"l{i}.hc{n}.in"], t[f"l{i}.hc{n}.out"] = rnd(P, std=0.3, mean=0.6), rnd(P, std=0.4, mean=0.7)
            t[f"l{i}.hc{n}.mix"] = (torch.eye(P) * 0.8 + torch.randn(P, P, generator=g) * 0.2).to(torch.bfloat16).float()
        if entry["type"] == "attention":
            H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            for name, rows in (("q", H * d), ("k", G * d), ("v", G * dv)):
                t[p + name], t[p + name + ".b"] = lin(rows, W), rnd(rows, std=0.4)
            t[p + "q.norm"], t[p + "k.norm"] = rnd(d, std=0.2, mean=1.2), rnd(d, std=0.2, mean=1.2)
            t[p + "rel"] = rnd(entry["_rows"], H, std=1.0)
            t[p + "o"], t[p + "o.b"] = lin(W, H * dv), rnd(W, std=0.3)
        elif entry["type"] == "channel_delta":
            H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            ra, rg = entry["_ranks"]
            for name, rows in (("q", G * d), ("k", G * d), ("v", H * dv)):
                t[p + name], t[p + name + ".conv"] = lin(rows, W), rnd(rows, m["conv"], std=0.6, mean=0.3)
            t[p + "b"], t[p + "A_log"], t[p + "norm"] = lin(H, W), uni(H, lo=-3.0, hi=0.5), rnd(dv, std=0.1, mean=1.0)
            t[p + "a1"], t[p + "a2"], t[p + "dt_bias"] = lin(ra, W), lin(H * d, ra), rnd(H * d, mean=-1.5)
            t[p + "g1"], t[p + "g2"] = lin(rg, W), lin(H * dv, rg, 2.0)
            t[p + "o"] = lin(W, H * dv)
        else:
            C, B = m["width"], m["blocks"]
            for name in ("y", "x"):
                t[p + name], t[p + name + ".b"] = lin(C, W), rnd(C, std=0.4)
            t[p + "conv"], t[p + "conv.b"] = rnd(C, m["conv"], std=0.5, mean=0.3), rnd(C, std=0.3)
            for name in ("ra", "ri"):
                t[p + name], t[p + name + ".b"] = rnd(B, C // B, C // B, std=(C // B) ** -0.5), rnd(B, C // B, std=0.5)
            t[p + "lam"] = rnd(C, std=1.5, mean=-3.0)
            t[p + "o"] = lin(W, C)
        mlp = entry["mlp"]
        if mlp is None:
            continue
        p = f"l{i}.mlp."
        t[p + "router"] = lin(mlp["router"]["experts"], W, 1.5)
        for name, ff in [(f"e{e}", mlp["expert"]["ff"]) for e in range(mlp["router"]["experts"])] + [("shared", mlp["shared"]["ff"])]:
            t[f"{p}{name}.up"], t[f"{p}{name}.down"] = lin(ff, W, 1.2), lin(W, ff, 1.2)
        t[p + "shared.sg"] = lin(1, W)
    return t
