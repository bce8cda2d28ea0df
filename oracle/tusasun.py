"""Plain, slow restatement of the Tusasun design on the CPU, in float64 unless told otherwise: one function per mechanism,
written from the equations, consuming the checkpoint's tensor names and ``config.json`` directly.  It shares no code with
lite_llama_amd/ (no kernels, no model classes, no cache): whole sequences only, full score matrices, token loops for every
recurrence, every expert evaluated for every token.

Notation: T tokens, W width, H heads on G key/value heads, d / dv key / value entries per head, P streams, E experts, eps the
norm epsilon, rn(y) = y / sqrt(mean(y^2) + eps).

  * streams         x_1 .. x_P all start as the embedding row.  A sublayer f with in [P], mix [P, P], out [P]:
                    u = sum_s in_s x_s;  y = ls * f(rn(u) (1 + w));  x_t <- sum_s mix[s, t] x_s + out_t y  (all t from the old x)
  * rglru           y = gelu(W_y h + b_y);  u = conv(W_x h + b_x) + b_c;  in each of the equal parts of u:
                    r = sigmoid(R u + b_r), i = sigmoid(I u + b_i);  log a = -8 r softplus(lam);
                    S <- a S + sqrt(1 - a^2) i u;  W_o (S y)
  * attention       q, k, v = W h + b;  q, k heads rn'd with one weight [d] each;  s = q . k scale, s <- cap tanh(s / cap),
                    s += rel[bucket(i - j), h];  causal softmax;  W_o + b_o
  * channel_delta   q, k, v through a causal convolution per channel and silu;  q, k heads divided by sqrt(sum + 1e-6), q times
                    d^(-1/2);  beta = sigmoid(W_b h);  g = exp(-exp(A_log_h) softplus(W_a2 W_a1 h + dt_bias)) per key entry;
                    S <- diag(g) S;  S <- S + k (beta (v - S^T k))^T;  o = S^T q;
                    every head rn'd times one weight [dv], times sigmoid(W_g2 W_g1 h);  W_o
  * experts         s = sigmoid(W_r h);  the `top` largest;  sum of e(s h), e(z) = W_down relu(W_up z)^2;
                    plus sigmoid(W_sg h) times a shared expert of the same form
  * output          logits = head (rn(sum of the streams) (1 + w_f))
"""

from __future__ import annotations

import math

import torch


def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def shifted_norm(x, w, eps):
    """RMS norm whose weight is stored around zero."""
    return rms(x, eps) * (1.0 + w)


def silu(x):
    return x * torch.sigmoid(x)


def gelu_tanh(x):
    return 0.5 * x * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (x + 0.044715 * x ** 3)))


def softplus(x):
    return torch.where(x > 30.0, x, torch.log1p(torch.exp(torch.clamp(x, max=30.0))))


def causal_conv(u, w, b=None):
    """``u [T, C]``, ``w [C, taps]``: y_t = b + sum_j w[:, j] u_(t - taps + 1 + j), zeros in front of the sequence."""
    T, taps = u.shape[0], w.shape[1]
    y = torch.zeros_like(u)
    for j in range(taps):
        back = taps - 1 - j
        if back < T:
            y[back:] += w[:, j] * u[:T - back]
    return y if b is None else y + b


# ------------------------------------------------------------------------------------- #
# streams
# ------------------------------------------------------------------------------------- #
def stream_input(xs, w_in):
    """``xs [P, T, W]`` -> the sublayer's input before its norm."""
    return (w_in[:, None, None] * xs).sum(0)


def stream_update(xs, y, mix, out):
    """New streams, every one from the old ones: ``mix[from, to]``."""
    return torch.stack([sum(mix[s, t] * xs[s] for s in range(xs.shape[0])) + out[t] * y for t in range(xs.shape[0])])


# ------------------------------------------------------------------------------------- #
# mixers
# ------------------------------------------------------------------------------------- #
def real_gated_scan(u, r, i, lam):
    """``u, r, i [T, C]``, ``lam [C]``, token by token.  Returns ``(S of every token [T, C], the last S)``."""
    S = torch.zeros_like(u[0])
    out = torch.zeros_like(u)
    for t in range(u.shape[0]):
        a = torch.exp(-8.0 * r[t] * softplus(lam))
        S = a * S + torch.sqrt(1.0 - a * a) * i[t] * u[t]
        out[t] = S
    return out, S


def block_gates(u, w, b):
    """``u [T, C]`` in equal parts, each through its own square matrix ``w [parts, out, in]`` with bias ``b [parts, out]``."""
    T, parts = u.shape[0], w.shape[0]
    up = u.view(T, parts, -1)
    return torch.sigmoid(torch.stack([up[:, p] @ w[p].T + b[p] for p in range(parts)], 1)).reshape(T, -1)


def rglru(h, t, p, m, eps):
    dt = h.dtype
    y = gelu_tanh(h @ t[p + "y"].to(dt).T + t[p + "y.b"].to(dt))
    u = causal_conv(h @ t[p + "x"].to(dt).T + t[p + "x.b"].to(dt), t[p + "conv"].to(dt), t[p + "conv.b"].to(dt))
    r = block_gates(u, t[p + "ra"].to(dt), t[p + "ra.b"].to(dt))
    i = block_gates(u, t[p + "ri"].to(dt), t[p + "ri.b"].to(dt))
    S, _ = real_gated_scan(u, r, i, t[p + "lam"].to(dt))
    return (S * y) @ t[p + "o"].to(dt).T


def distance_bucket(n, rows, far):
    """Bucket of the distance ``n >= 0`` among ``rows`` buckets: one per distance below ``rows / 2``, then logarithmic up to ``far``."""
    half = rows // 2
    if n < half:
        return n
    return min(rows - 1, half + math.floor(math.log(n / half) / math.log(far / half) * (rows - half)))


def attention_scores(q, k, scale, cap, rel_h, far):
    """One head: ``q, k [T, d]``, ``rel_h [rows]`` -> ``[T, T]`` scores with -inf above the diagonal."""
    T = q.shape[0]
    s = (q @ k.T) * scale
    if cap:
        s = cap * torch.tanh(s / cap)
    by_distance = torch.stack([rel_h[distance_bucket(n, rel_h.shape[0], far)] for n in range(T)])
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    s = s + by_distance[(i - j).clamp(min=0)]
    return s.masked_fill(j > i, -math.inf)


def attention(h, t, p, m, eps):
    T, dt = h.shape[0], h.dtype
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    proj = lambda name: h @ t[p + name].to(dt).T + t[p + name + ".b"].to(dt)  # noqa: E731
    q = rms(proj("q").view(T, H, d), eps) * t[p + "q.norm"].to(dt)
    k = rms(proj("k").view(T, G, d), eps) * t[p + "k.norm"].to(dt)
    v = proj("v").view(T, G, dv)
    rel = t[p + "rel"].to(dt)
    heads = []
    for n in range(H):
        g = n // (H // G)
        s = attention_scores(q[:, n], k[:, g], float(m["scale"]), float(m["softcap"]), rel[:, n], float(m["bias_max"]))
        heads.append(torch.softmax(s, -1) @ v[:, g])
    return torch.cat(heads, -1) @ t[p + "o"].to(dt).T + t[p + "o.b"].to(dt)


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_scan(q, k, v, g, beta):
    """One head, token by token: ``q, k, g [T, d]``, ``v [T, dv]``, ``beta [T]``.  Returns ``(o [T, dv], the last S)``."""
    S = torch.zeros(k.shape[1], v.shape[1], dtype=q.dtype)
    o = torch.zeros(k.shape[0], v.shape[1], dtype=q.dtype)
    for t in range(k.shape[0]):
        S = g[t][:, None] * S
        u = beta[t] * (v[t] - S.T @ k[t])
        S = S + torch.outer(k[t], u)
        o[t] = S.T @ q[t]
    return o, S


def channel_decay(z, dt_bias, a_log):
    """``z, dt_bias [.., H, d]``, ``a_log [H]``."""
    return torch.exp(-torch.exp(a_log)[:, None] * softplus(z + dt_bias))


def channel_delta(h, t, p, m, eps):
    T, dt = h.shape[0], h.dtype
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    short = lambda name: silu(causal_conv(h @ t[p + name].to(dt).T, t[p + name + ".conv"].to(dt)))  # noqa: E731
    q = unit(short("q").view(T, G, d)) * d ** -0.5
    k = unit(short("k").view(T, G, d))
    v = short("v").view(T, H, dv)
    beta = torch.sigmoid(h @ t[p + "b"].to(dt).T)
    z = ((h @ t[p + "a1"].to(dt).T) @ t[p + "a2"].to(dt).T).view(T, H, d)
    g = channel_decay(z, t[p + "dt_bias"].to(dt).view(H, d), t[p + "A_log"].to(dt))
    o = torch.zeros(T, H, dv, dtype=dt)
    for n in range(H):
        c = n // (H // G)
        o[:, n], _ = delta_scan(q[:, c], k[:, c], v[:, n], g[:, n], beta[:, n])
    o = (rms(o, eps) * t[p + "norm"].to(dt)).view(T, H * dv)
    o = o * torch.sigmoid((h @ t[p + "g1"].to(dt).T) @ t[p + "g2"].to(dt).T)
    return o @ t[p + "o"].to(dt).T


MIXERS = {"rglru": rglru, "attention": attention, "channel_delta": channel_delta}


# ------------------------------------------------------------------------------------- #
# feed-forward
# ------------------------------------------------------------------------------------- #
def square_expert(z, t, p):
    return torch.relu(z @ t[p + "up"].to(z.dtype).T) ** 2 @ t[p + "down"].to(z.dtype).T


def route(h, t, p, top):
    """``(ids [T, top], weights [T, top])``: the largest sigmoid scores, not renormalised."""
    s = torch.sigmoid(h @ t[p + "router"].to(h.dtype).T)
    w, ids = torch.topk(s, top, dim=-1)
    return ids, w


def moe(h, t, p, mlp):
    ids, w = route(h, t, p, int(mlp["router"]["top"]))
    y = torch.zeros_like(h)
    for i in range(h.shape[0]):
        for e, we in zip(ids[i].tolist(), w[i]):
            y[i] += square_expert((we * h[i])[None], t, f"{p}e{e}.")[0]
    if mlp.get("shared"):
        y = y + torch.sigmoid(h @ t[p + "shared.sg"].to(h.dtype).T) * square_expert(h, t, p + "shared.")
    return y


# ------------------------------------------------------------------------------------- #
# the model
# ------------------------------------------------------------------------------------- #
def layer_order(cfg):
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return list(range(n))
    a, b = int(loop["start"]), int(loop["stop"])
    return list(range(a)) + list(range(a, b)) * int(loop["times"]) + list(range(b, n))


def forward(tokens, t, cfg, dtype=torch.float64):
    """``(logits [T, vocab], sum of the streams after every layer run [runs, T, W])`` of one whole sequence."""
    eps = float(cfg["norm"]["eps"])
    x = t["embed"].to(dtype)[torch.tensor(list(tokens))]
    xs = torch.stack([x] * int(cfg["streams"]))
    layers = []
    for index in layer_order(cfg):
        entry, p = cfg["layers"][index], f"l{index}."
        sub = [(1, lambda h: MIXERS[entry["type"]](h, t, p + "mix.", entry["mixer"], eps))]
        if entry.get("mlp") is not None:
            sub.append((2, lambda h: moe(h, t, p + "mlp.", entry["mlp"])))
        for n, f in sub:
            hc = {k: t[f"{p}hc{n}.{k}"].to(dtype) for k in ("in", "out", "mix")}
            y = f(shifted_norm(stream_input(xs, hc["in"]), t[f"{p}norm{n}"].to(dtype), eps)) * t[f"{p}ls{n}"].to(dtype)
            xs = stream_update(xs, y, hc["mix"], hc["out"])
        layers.append(xs.sum(0))
    h = shifted_norm(xs.sum(0), t["final.norm"].to(dtype), eps)
    return h @ t["head"].to(dtype).T, torch.stack(layers)


def greedy(prompt, steps, t, cfg, dtype=torch.float64):
    """``steps`` tokens after ``prompt``, each the argmax of the last position's logits."""
    toks = list(prompt)
    out = []
    for _ in range(steps):
        logits, _ = forward(toks, t, cfg, dtype)
        out.append(int(torch.argmax(logits[-1])))
        toks.append(out[-1])
    return out
