"""Plain, slow restatement of the Kokuvik design on the CPU, in float64 unless told otherwise: one function per mechanism,
written from the equations, consuming the checkpoint's tensor names and ``config.json`` directly.  It shares no code with
lite_llama_amd/ (no kernels, no model classes, no cache): whole sequences only, full score matrices, the retention state token
by token, every expert evaluated for every token.

Notation: T tokens, W width, H query heads on G key/value heads, d query/key entries and dv value entries per head, E experts,
rn(y) = y / sqrt(mean(y^2) + eps).

  * layer          h = rn(x) * w;  x <- x + (mixer(h) + feed_forward(h))
  * retention      q, k (H x d), v (H x dv);  entry i < dims / 2 of a q / k head rotated with entry i + dims / 2 by position * f_i;
                   k times d^(-1/2);  S <- lambda_h S + k v^T, o = S^T q;  heads rn(o) side by side, times silu(W_g h);  W_o
  * attention      pairs (2i, 2i + 1) of the first `dims` entries of q / k heads rotated by position * f_i (f_i rescaled by wavelength
                   bands);  scores q . k * scale over keys j <= i with i - j < size or j < keep_first;  weights
                   exp(s) / (exp(sink_h) + sum exp(s));  head h times sigmoid(W_g h)_h;  W_o.  A layer may read the keys (rotated)
                   and values of an earlier layer
  * feed-forward   dense: W_d relu(W_u h + b_u)^2 + b_d
                   experts: softmax over all router logits; a group of neighbouring experts scores as its best member, the best
                   groups stay, the `top` best experts in them weigh in with score / sum of chosen scores:
                   sum of weight * W_d(silu(W_g h) * W_u h), plus a shared expert of the same form
  * output         logits = head (rn(x) * w_final)
"""

from __future__ import annotations

import math

import torch


# ------------------------------------------------------------------------------------- #
# norm, rotation
# ------------------------------------------------------------------------------------- #
def rms_norm(x, weight, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis, times ``weight`` (``None``: no weight)."""
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if weight is None else y * weight


def banded_frequencies(rot):
    """``f [dims / 2]`` of ``{"base", "dims", "scaling": {factor, low, high, original} | None}``: with wavelength l = 2 pi / f a
    frequency stays where l < original / high, is divided by ``factor`` where l > original / low, and is blended in between."""
    dims, base = int(rot["dims"]), float(rot["base"])
    out = []
    sc = rot.get("scaling")
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if sc:
            factor, low, high, original = (float(sc[k]) for k in ("factor", "low", "high", "original"))
            wavelength = 2 * math.pi / f
            if wavelength > original / low:
                f = f / factor
            elif not wavelength < original / high:
                s = (original / wavelength - low) / (high - low)
                f = (1 - s) * f / factor + s * f
        out.append(f)
    return torch.tensor(out, dtype=torch.float64)


def _angles(positions, rot, dtype, angle_dtype):
    f = banded_frequencies(rot)
    ang = (positions.to(angle_dtype)[:, None] * f.to(angle_dtype)[None, :]).to(torch.float64)
    return torch.cos(ang).to(dtype)[:, None, :], torch.sin(ang).to(dtype)[:, None, :]


def rotate_interleaved(v, positions, rot, angle_dtype=torch.float64):
    """``v [T, heads, n]``: entry 2i with entry 2i + 1 of the first ``dims`` entries; the rest passes."""
    dims = int(rot["dims"])
    cos, sin = _angles(positions, rot, v.dtype, angle_dtype)
    a, b = v[..., 0:dims:2], v[..., 1:dims:2]
    out = v.clone()
    out[..., 0:dims:2] = a * cos - b * sin
    out[..., 1:dims:2] = b * cos + a * sin
    return out


def rotate_halves(v, positions, rot, angle_dtype=torch.float64):
    """``v [T, heads, n]``: entry i with entry i + dims / 2 of the first ``dims`` entries; the rest passes."""
    dims = int(rot["dims"])
    cos, sin = _angles(positions, {"dims": dims, "base": rot["base"]}, v.dtype, angle_dtype)
    a, b = v[..., :dims // 2], v[..., dims // 2:dims]
    out = v.clone()
    out[..., :dims // 2] = a * cos - b * sin
    out[..., dims // 2:dims] = b * cos + a * sin
    return out


# ------------------------------------------------------------------------------------- #
# retention
# ------------------------------------------------------------------------------------- #
def retention_scan(q, k, v, decay, state=None):
    """``q, k [T, H, d]``, ``v [T, H, dv]``, ``decay [H]``: token by token S <- decay_h S + k v^T, o = S^T q.  Returns
    ``(o [T, H, dv], S [H, d, dv])``."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[-1], dtype=q.dtype) if state is None else state.clone()
    lam = torch.as_tensor(decay, dtype=q.dtype)[:, None, None]
    out = []
    for t in range(T):
        S = lam * S + k[t][:, :, None] * v[t][:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return (torch.stack(out) if out else v.new_zeros(0, H, v.shape[-1])), S


def retention(h, t, p, m, eps, angle_dtype=torch.float64):
    T = h.shape[0]
    H, d, dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    w = lambda leaf: t[p + leaf].to(h.dtype)  # noqa: E731
    q, k, v = (h @ w("q").T).view(T, H, d), (h @ w("k").T).view(T, H, d), (h @ w("v").T).view(T, H, dv)
    if m.get("rot"):
        pos = torch.arange(T)
        q, k = rotate_halves(q, pos, m["rot"], angle_dtype), rotate_halves(k, pos, m["rot"], angle_dtype)
    o, _ = retention_scan(q, k * d ** -0.5, v, m["decay"])
    o = rms_norm(o, None, eps).reshape(T, H * dv)
    g = h @ w("g").T
    return (o * (g * torch.sigmoid(g))) @ w("o").T


# ------------------------------------------------------------------------------------- #
# attention
# ------------------------------------------------------------------------------------- #
def visible(T, size, keep_first):
    """``[T, T]`` bool: query i sees key j when j <= i and (i - j < size or j < keep_first)."""
    i = torch.arange(T)[:, None]
    j = torch.arange(T)[None, :]
    return (j <= i) & ((i - j < size) | (j < keep_first))


def sink_softmax(scores, mask, sink):
    """exp(s_j) / (exp(sink) + sum over visible j of exp(s_j))."""
    s = scores.masked_fill(~mask, -math.inf)
    m = torch.clamp(s.max(-1, keepdim=True).values, min=float(sink))
    e = torch.exp(s - m)
    return e / (torch.exp(sink - m) + e.sum(-1, keepdim=True))


def attention(h, t, p, m, kv=None, angle_dtype=torch.float64):
    """One attention mixer over a whole sequence.  ``kv``: ``(keys, values)`` of the layer it borrows them from, or ``None``.
    Returns ``(output [T, W], (keys [T, G, d] after rotation, values [T, G, dv]))``."""
    T = h.shape[0]
    H, G, d, dv = int(m["heads"]), int(m.get("kv_heads") or m["heads"]), int(m["dim"]), int(m["vdim"])
    w = lambda leaf: t[p + leaf].to(h.dtype)  # noqa: E731
    pos = torch.arange(T)
    turn = (lambda x: rotate_interleaved(x, pos, m["rot"], angle_dtype)) if m.get("rot") else (lambda x: x)
    q = turn((h @ w("q").T).view(T, H, d))
    if kv is None:
        kv = turn((h @ w("k").T).view(T, G, d)), (h @ w("v").T).view(T, G, dv)
    k, v = kv
    mask_cfg = m.get("mask") or {}
    mask = visible(T, int(mask_cfg.get("size") or T + 1), int(mask_cfg.get("keep_first") or 0))
    gate = torch.sigmoid(h @ w("g").T)
    heads = []
    for a in range(H):
        g = a // (H // G)
        weights = sink_softmax(q[:, a] @ k[:, g].T * float(m["scale"]), mask, w("sink")[a])
        heads.append(weights @ v[:, g] * gate[:, a:a + 1])
    return torch.cat(heads, -1) @ w("o").T, kv


# ------------------------------------------------------------------------------------- #
# feed-forwards
# ------------------------------------------------------------------------------------- #
def square_mlp(h, t, p):
    u = torch.relu(h @ t[p + "up"].to(h.dtype).T + t[p + "up.b"].to(h.dtype))
    return (u * u) @ t[p + "down"].to(h.dtype).T + t[p + "down.b"].to(h.dtype)


def glu_expert(h, t, p):
    z = h @ t[p + "gate"].to(h.dtype).T
    return (z * torch.sigmoid(z) * (h @ t[p + "up"].to(h.dtype).T)) @ t[p + "down"].to(h.dtype).T


def route(h, router, top, groups=None):
    """``(ids [T, top], weights [T, top])``: softmax scores, the best groups by their best member, the best experts in them,
    weights divided by their sum."""
    s = torch.softmax(h @ router.to(h.dtype).T, -1)
    ranked = s
    count, keep = int((groups or {}).get("count", 1)), int((groups or {}).get("keep", 1))
    if count > 1:
        best = s.view(s.shape[0], count, -1).max(-1).values
        kept = torch.zeros_like(best, dtype=torch.bool).scatter_(1, torch.topk(best, keep, dim=-1).indices, True)
        ranked = s.masked_fill(~kept.repeat_interleave(s.shape[1] // count, 1), -1.0)
    ids = torch.topk(ranked, top, dim=-1).indices
    w = s.gather(1, ids)
    return ids, w / (w.sum(-1, keepdim=True) + 1e-20)


def moe(h, t, p, mlp):
    r = mlp["router"]
    ids, w = route(h, t[p + "router"], int(r["top"]), r.get("groups"))
    y = torch.zeros(h.shape[0], t[p + "e0.down"].shape[0], dtype=h.dtype)
    for e in range(int(r["experts"])):
        y = y + glu_expert(h, t, f"{p}e{e}.") * ((ids == e) * w).sum(-1, keepdim=True)
    return y + glu_expert(h, t, p + "shared.") if mlp.get("shared") else y


def feed_forward(h, t, p, mlp):
    if mlp is None:
        return torch.zeros_like(h)
    return square_mlp(h, t, p) if mlp.get("kind", "dense") == "dense" else moe(h, t, p, mlp)


# ------------------------------------------------------------------------------------- #
# the model
# ------------------------------------------------------------------------------------- #
def forward(tokens, t, cfg, dtype=torch.float64, angle_dtype=torch.float64, layers_out: list | None = None):
    """Logits ``[T, vocab]`` of one whole sequence.  ``layers_out`` receives the residual stream after every layer."""
    eps = float(cfg["norm"]["eps"])
    x = t["embed"].to(dtype)[torch.tensor(list(tokens))]
    cached = {}
    for i, entry in enumerate(cfg["layers"]):
        p, m = f"l{i}.", entry["mixer"]
        h = rms_norm(x, t[p + "norm1"].to(dtype), eps)
        if entry["type"] == "retention":
            y = retention(h, t, p + "mix.", m, eps, angle_dtype)
        else:
            source = m.get("kv_from")
            y, cached[i] = attention(h, t, p + "mix.", m, None if source is None else cached[int(source)], angle_dtype)
        x = x + (y + feed_forward(h, t, p + "mlp.", entry.get("mlp")))
        if layers_out is not None:
            layers_out.append(x.clone())
    return rms_norm(x, t["final.norm"].to(dtype), eps) @ t["head"].to(dtype).T


def greedy(prompt, t, cfg, new_tokens, dtype=torch.float64):
    """Greedy continuation by recomputing the whole sequence per token."""
    seq, out = list(prompt), []
    for _ in range(new_tokens):
        nxt = int(forward(seq, t, cfg, dtype)[-1].argmax())
        seq.append(nxt)
        out.append(nxt)
    return out
