"""Small random Kokuvik checkpoints for tests: configurations, tensors under the checkpoint's names (values exactly representable
in bfloat16, so a bf16 file holds the same numbers the float64 oracle reads).  Files are written with ``tests._layered.write``."""

import torch


def rot(dims, base=100.0, scaled=True, factor=4.0, low=0.5, high=4.0, original=64):
    out = {"base": base, "dims": dims}
    if scaled:
        out["scaling"] = {"factor": factor, "high": high, "low": low, "original": original}
    return out


def attention(heads, kv_heads, dim, vdim, window, keep, rot_dims, mlp=None, scale=None, kv_from=None, **rot_kw):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": window, "keep_first": keep},
             "rot": rot(rot_dims, **rot_kw), "scale": scale if scale is not None else 1.5 * dim ** -0.5}
    if kv_from is not None:
        mixer["kv_from"] = kv_from
    return {"type": "attention", "mixer": mixer, "mlp": mlp}


def retention(heads, dim, vdim, rot_dims, mlp=None, base=100.0, decay=None):
    decay = decay if decay is not None else [1.0 - 2.0 ** -(2 + 2 * i) for i in range(heads)]
    return {"type": "retention", "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay, "rot": {"base": base, "dims": rot_dims}}}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, shared=0, groups=None):
    out = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if groups is not None:
        out["router"]["groups"] = {"count": groups[0], "keep": groups[1]}
    if shared:
        out["shared"] = {"ff": shared}
    return out


def config(layers, width, vocab, eps=1e-5):
    return {"architecture": "Kokuvik", "layers": layers, "norm": {"eps": eps}, "vocab": vocab, "width": width}


CONFIGS = {
    # sizes that are multiples of 8 (the 16-bit matrix-core and 16-byte forms run); every feed-forward kind and a layer without one; a
    # layer that borrows keys and values with another window than their owner's; a part of the retention heads rotated
    "mix": config([attention(4, 2, 16, 8, 9, 3, 8, mlp=dense(72)),
                   retention(3, 16, 24, 16, mlp=moe(6, 2, 24, shared=40, groups=(3, 2))),
                   attention(4, 2, 16, 8, 14, 0, 8, kv_from=0, mlp=moe(4, 4, 16)),
                   retention(2, 32, 16, 16)], width=96, vocab=83),
    # odd sizes: heads of 10 / 6 and 12 / 10 entries (the plain forms), feed-forward and shared widths that are no multiple of 8
    # (activations and gates off every 16-byte border), a layer whose keys and values two others borrow, frequencies without
    # bands, groups of one expert, one expert chosen, decays of 1 and far below 1/2
    "odd": config([retention(5, 10, 6, 4, mlp=dense(44), decay=[1.0, 0.25, 0.0625, 0.96875, 0.5]),
                   attention(3, 1, 12, 10, 7, 2, 6, mlp=moe(9, 1, 12, shared=13, groups=(9, 4)), scaled=False),
                   attention(3, 1, 12, 10, 5, 6, 6, kv_from=1, mlp=dense(37), scaled=False, scale=1.0),
                   attention(3, 1, 12, 10, 30, 1, 6, kv_from=1, mlp=moe(8, 3, 6, groups=(4, 2)), scaled=False)], width=58, vocab=47,
                  eps=1e-6),
    # twenty query heads on one key/value head (two column tiles of the grouped decode form), wide state heads, values wider and
    # narrower than keys, more kept keys than a window holds, several heads that borrow, a deep band scaling
    "wide": config([attention(20, 1, 8, 16, 21, 40, 8, mlp=dense(40), factor=16.0, original=512),
                    retention(2, 72, 40, 72, mlp=moe(8, 4, 8, shared=8, groups=(2, 1))),
                    attention(20, 1, 8, 16, 3, 5, 8, kv_from=0, mlp=moe(2, 1, 16), factor=16.0, original=512),
                    retention(1, 136, 8, 64)], width=64, vocab=71),
    # everything that can be 1: one head of one pair, one value entry, a window of one key plus one kept key, one expert of one hidden
    # entry in one group, one shared entry; a width that is no multiple of 4
    "one": config([attention(1, 1, 2, 1, 1, 1, 2, mlp=moe(1, 1, 1, shared=1, groups=(1, 1)), scale=1.0),
                   retention(1, 2, 1, 2, mlp=dense(1)), attention(1, 1, 2, 1, 4, 0, 2, kv_from=0)], width=18, vocab=11),
}


def tensors(cfg, seed=0):
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]

    def rnd(*shape, std=1.0, mean=0.0):
        return (torch.randn(*shape, generator=g) * std + mean).to(torch.bfloat16).float()

    def lin(out, inp, gain=1.0):
        return rnd(out, inp, std=gain * inp ** -0.5)

    t = {"embed": rnd(V, W), "final.norm": rnd(W, std=0.1, mean=1.0), "head": lin(V, W)}
    for i, entry in enumerate(cfg["layers"]):
        p, m = f"l{i}.mix.", entry["mixer"]
        t[f"l{i}.norm1"] = rnd(W, std=0.1, mean=1.0)
        H, d, dv = m["heads"], m["dim"], m["vdim"]
        if entry["type"] == "retention":
            for name, rows in (("q", H * d), ("k", H * d), ("v", H * dv), ("g", H * dv)):
                t[p + name] = lin(rows, W)
        else:
            G = m["kv_heads"]
            t[p + "q"], t[p + "g"], t[p + "sink"] = lin(H * d, W, 1.5), lin(H, W, 1.5), rnd(H)
            if m.get("kv_from") is None:
                t[p + "k"], t[p + "v"] = lin(G * d, W, 1.5), lin(G * dv, W)
        t[p + "o"] = lin(W, H * dv)
        mlp = entry["mlp"]
        if mlp is None:
            continue
        p = f"l{i}.mlp."
        if mlp["kind"] == "dense":
            t[p + "up"], t[p + "up.b"] = lin(mlp["ff"], W), rnd(mlp["ff"], std=0.4)
            t[p + "down"], t[p + "down.b"] = lin(W, mlp["ff"], 0.7), rnd(W, std=0.4)
            continue
        t[p + "router"] = lin(mlp["router"]["experts"], W, 1.5)
        members = [(f"e{e}", mlp["expert"]["ff"]) for e in range(mlp["router"]["experts"])]
        for name, ff in members + ([("shared", mlp["shared"]["ff"])] if mlp.get("shared") else []):
            t[f"{p}{name}.gate"], t[f"{p}{name}.up"], t[f"{p}{name}.down"] = lin(ff, W, 1.2), lin(ff, W, 1.2), lin(W, ff, 1.2)
    return t
