"""A plain float64 implementation of the Domelix design, one function per
mechanism, for the tests to compare the serving path against. It shares no code
with the package: whole sequences only, no cache, no batching, python loops
where they are clearest.

Weights are a dict name -> float64 tensor with the checkpoint's names ('embed',
'l<i>.norm1', 'l<i>.mix.left.q', ...); the config is the dict that config.json
holds.
"""

from __future__ import annotations

import math

import torch

F64 = torch.float64


def unit_rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last dimension."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm_about_one(x, w, eps):
    """RMS norm with a weight stored as its distance from 1."""
    return unit_rms(x, eps) * (1.0 + w)


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


# -- softmax attention with a distance bias ------------------------------------------


def bucket(n, rows, limit):
    """The row of the bias table for a key n positions back: one row each for the
    first rows // 2 distances, then rows that widen with the logarithm until
    `limit`, the last one for everything beyond."""
    near = rows // 2
    if n < near:
        return n
    step = math.log(n / near) / math.log(limit / near) * (rows - near)
    return min(rows - 1, near + math.floor(step + 1e-9))


def bias_scores(h, w, p, mx):
    """Scores [heads, n, n] (query, key), scaled and biased; no mask."""
    n = h.shape[0]
    H, G, d = mx["heads"], mx.get("kv_heads", mx["heads"]), mx["dim"]
    q = (h @ w[p + "q"].T).view(n, H, d)
    k = (h @ w[p + "k"].T).view(n, G, d)
    rel = w[p + "rel"]
    s = torch.zeros(H, n, n, dtype=F64)
    rows = [bucket(m, rel.shape[0], mx["bias_max"]) for m in range(n)]
    for a in range(H):
        s[a] = q[:, a] @ k[:, a * G // H].T * mx["scale"]
        for i in range(n):
            for j in range(i + 1):
                s[a, i, j] += rel[rows[i - j], a]
    return s


def sink_weights(s, sink):
    """Causal softmax over the keys with one more term exp(sink_h) in every
    denominator; [heads, n, n]."""
    n = s.shape[1]
    out = torch.zeros_like(s)
    for a in range(s.shape[0]):
        for i in range(n):
            top = max(float(s[a, i, : i + 1].max()), float(sink[a]))
            e = torch.exp(s[a, i, : i + 1] - top)
            out[a, i, : i + 1] = e / (e.sum() + math.exp(float(sink[a]) - top))
    return out


def bias_attention(h, w, p, mx):
    n = h.shape[0]
    H, G = mx["heads"], mx.get("kv_heads", mx["heads"])
    dv = mx.get("vdim", mx["dim"])
    a = sink_weights(bias_scores(h, w, p, mx), w[p + "sink"])
    v = (h @ w[p + "v"].T).view(n, G, dv)
    o = torch.cat([a[i] @ v[:, i * G // H] for i in range(H)], dim=-1)
    return (o * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


# -- linear attention with a fixed decay ---------------------------------------------


def decayed_sum(q, k, v, decay):
    """One head, summed out: o_i = sum_{j <= i} decay^(i - j) (q_i . k_j) v_j."""
    n = q.shape[0]
    lag = torch.arange(n).view(n, 1) - torch.arange(n).view(1, n)
    keep = torch.tensor(float(decay), dtype=F64) ** lag.clamp(min=0)
    return ((q @ k.T) * keep * (lag >= 0)) @ v


def decayed_state(k, v, decay):
    """The state such a head ends with, [d, dv]."""
    n = k.shape[0]
    keep = torch.tensor(float(decay), dtype=F64) ** torch.arange(n - 1, -1, -1)
    return (k * keep.view(n, 1)).T @ v


def lightning(h, w, p, mx, eps, states=False):
    n, H = h.shape[0], mx["heads"]
    q, k, v = (silu(h @ w[p + x].T).view(n, H, -1) for x in "qkv")
    o = torch.cat([decayed_sum(q[:, a], k[:, a], v[:, a], mx["decay"][a]) for a in range(H)], -1)
    y = (unit_rms(o, eps) * w[p + "norm"] * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T
    if states:
        return y, [decayed_state(k[:, a], v[:, a], mx["decay"][a]) for a in range(H)]
    return y


def rotate_halves(x, positions, base, dims):
    """x [n, ..., d]: dimension i turned with dimension i + dims / 2 by
    position * base^(-2 i / dims); the rest passes."""
    half = dims // 2
    y = x.clone()
    for i in range(half):
        ang = positions.to(F64) * base ** (-2.0 * i / dims)
        shape = [-1] + [1] * (x.dim() - 2)
        c, s = torch.cos(ang).view(shape), torch.sin(ang).view(shape)
        y[..., i] = x[..., i] * c - x[..., i + half] * s
        y[..., i + half] = x[..., i + half] * c + x[..., i] * s
    return y


def retention(h, w, p, mx, eps, states=False):
    n, H, d = h.shape[0], mx["heads"], mx["dim"]
    q, k, v = ((h @ w[p + x].T).view(n, H, -1) for x in "qkv")
    rot = mx.get("rot")
    if rot:
        pos = torch.arange(n)
        q = rotate_halves(q, pos, rot["base"], rot["dims"])
        k = rotate_halves(k, pos, rot["base"], rot["dims"])
    k = k / math.sqrt(d)
    o = torch.cat([unit_rms(decayed_sum(q[:, a], k[:, a], v[:, a], mx["decay"][a]), eps)
                   for a in range(H)], -1)
    y = (o * silu(h @ w[p + "g"].T)) @ w[p + "o"].T
    if states:
        return y, [decayed_state(k[:, a], v[:, a], mx["decay"][a]) for a in range(H)]
    return y


# -- gated delta rule ------------------------------------------------------------------


def causal_conv(x, taps):
    """x [n, C], taps [C, K]: every channel's weighted sum of its last K inputs
    (the last weight for the current one, zeros before the start), then silu."""
    n, K = x.shape[0], taps.shape[1]
    y = torch.zeros_like(x)
    for t in range(n):
        for i in range(K):
            src = t - (K - 1) + i
            if src >= 0:
                y[t] = y[t] + taps[:, i] * x[src]
    return silu(y)


def delta_cell(q, k, v, beta, g):
    """One head, token by token; returns (o [n, dv], the final state)."""
    S = torch.zeros(k.shape[1], v.shape[1], dtype=F64)
    out = []
    for t in range(q.shape[0]):
        S = g[t] * S
        read = k[t] @ S
        S = S + torch.outer(k[t], beta[t] * (v[t] - read))
        out.append(q[t] @ S)
    return torch.stack(out), S


def delta_parts(h, w, p, mx):
    """(q, k [n, G, d] as unit vectors, v [n, H, dv], beta, g [n, H])."""
    n, H = h.shape[0], mx["heads"]
    G = mx.get("kv_heads", H)
    q, k, v = (causal_conv(h @ w[p + x].T, w[p + x + ".conv"]) for x in "qkv")
    q, k, v = q.view(n, G, -1), k.view(n, G, -1), v.view(n, H, -1)
    q = q / torch.sqrt((q * q).sum(-1, keepdim=True) + 1e-6) / math.sqrt(mx["dim"])
    k = k / torch.sqrt((k * k).sum(-1, keepdim=True) + 1e-6)
    rate = torch.log1p(torch.exp(h @ w[p + "a"].T + w[p + "dt_bias"]))
    return q, k, v, sigmoid(h @ w[p + "b"].T), torch.exp(-torch.exp(w[p + "A_log"]) * rate)


def delta(h, w, p, mx, eps, states=False):
    H = mx["heads"]
    G = mx.get("kv_heads", H)
    q, k, v, beta, g = delta_parts(h, w, p, mx)
    outs, ends = [], []
    for a in range(H):
        o, S = delta_cell(q[:, a * G // H], k[:, a * G // H], v[:, a], beta[:, a], g[:, a])
        outs.append(unit_rms(o, eps) * w[p + "norm"])
        ends.append(S)
    y = (torch.cat(outs, -1) * silu(h @ w[p + "g"].T)) @ w[p + "o"].T
    return (y, ends) if states else y


# -- feed-forward ----------------------------------------------------------------------


def route(h, w, p, router):
    """Per token: [(expert, weight), ...], best first."""
    s = torch.softmax(h @ w[p + "router"].T, -1)
    E = router["experts"]
    groups = router.get("groups") or {"count": 1, "keep": 1}
    size = E // groups["count"]
    out = []
    for row in s.tolist():
        best = sorted(range(groups["count"]),
                      key=lambda a: -max(row[a * size:(a + 1) * size]))[: groups["keep"]]
        allowed = [e for e in range(E) if e // size in best]
        chosen = sorted(allowed, key=lambda e: -row[e])[: router["top"]]
        total = sum(row[e] for e in chosen) + 1e-20
        out.append([(e, row[e] / total) for e in chosen])
    return out


def moe(h, w, p, mlp):
    y = torch.zeros_like(h)
    for t, picks in enumerate(route(h, w, p, mlp["router"])):
        for e, s in picks:
            q = p + "e%d." % e
            y[t] += s * (w[q + "down"] @ (silu(w[q + "gate"] @ h[t]) * (w[q + "up"] @ h[t])))
    return y


# -- the stack -------------------------------------------------------------------------


def mixer(h, w, p, spec, eps):
    mx = spec["mixer"]
    if spec["type"] == "retention":
        return retention(h, w, p, mx, eps)
    if spec["type"] == "delta":
        return delta(h, w, p, mx, eps)
    a = unit_rms(bias_attention(h, w, p + "left.", mx["left"]), eps) * w[p + "left.out"]
    b = unit_rms(lightning(h, w, p + "right.", mx["right"], eps), eps) * w[p + "right.out"]
    return (a + b) / 2.0


def forward(cfg, w, ids, return_layers=False):
    """Logits [n, vocab] (and the stream after every layer)."""
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.tensor(ids)]
    layers = []
    for i, spec in enumerate(cfg["layers"]):
        p = "l%d." % i
        add = mixer(norm_about_one(x, w[p + "norm1"], eps), w, p + "mix.", spec, eps)
        if spec.get("mlp") is not None:
            add = add + moe(norm_about_one(x, w[p + "norm2"], eps), w, p + "mlp.", spec["mlp"])
        x = x + add
        layers.append(x)
    logits = norm_about_one(x, w["final.norm"], eps) @ w["head"].T
    return (logits, layers) if return_layers else logits


def random_weights(cfg, seed=0):
    """bf16-representable float64 weights under the checkpoint's names."""
    g = torch.Generator().manual_seed(seed)
    W, w = cfg["width"], {}

    def put(name, *shape, scale=None, shift=0.0):
        s = shape[-1] ** -0.5 if scale is None else scale
        w[name] = (torch.randn(*shape, generator=g) * s + shift).bfloat16().to(F64)

    put("embed", cfg["vocab"], W, scale=1.0)
    for i, spec in enumerate(cfg["layers"]):
        p, mx = "l%d." % i, spec["mixer"]
        put(p + "norm1", W, scale=0.2)

        def decaying(q, m, plain_norm):
            H, d, dv = m["heads"], m["dim"], m.get("vdim", m["dim"])
            for x, n in (("q", d), ("k", d), ("v", dv), ("g", dv)):
                put(q + x, H * n, W)
            put(q + "o", W, H * dv)
            if plain_norm:
                put(q + "norm", H * dv, scale=0.2, shift=1.0)

        if spec["type"] == "retention":
            decaying(p + "mix.", mx, False)
        elif spec["type"] == "parallel":
            q, m = p + "mix.left.", mx["left"]
            H, G = m["heads"], m.get("kv_heads", m["heads"])
            d, dv = m["dim"], m.get("vdim", m["dim"])
            put(q + "q", H * d, W)
            put(q + "k", G * d, W)
            put(q + "v", G * dv, W)
            put(q + "g", H * dv, W)
            put(q + "o", W, H * dv)
            put(q + "rel", m["rows"], H, scale=1.0)
            put(q + "sink", H, scale=1.0)
            put(q + "out", W, scale=0.2, shift=1.0)
            decaying(p + "mix.right.", mx["right"], True)
            put(p + "mix.right.out", W, scale=0.2, shift=1.0)
        else:
            H, G = mx["heads"], mx.get("kv_heads", mx["heads"])
            d, dv = mx["dim"], mx.get("vdim", mx["dim"])
            q = p + "mix."
            for x, n in (("q", G * d), ("k", G * d), ("v", H * dv)):
                put(q + x, n, W)
                put(q + x + ".conv", n, mx["conv"], scale=0.5)
            put(q + "g", H * dv, W)
            put(q + "a", H, W)
            put(q + "b", H, W)
            put(q + "A_log", H, scale=0.5)
            put(q + "dt_bias", H, scale=0.5, shift=-3.0)
            put(q + "norm", dv, scale=0.2, shift=1.0)
            put(q + "o", W, H * dv)
        mlp = spec.get("mlp")
        if mlp is not None:
            put(p + "norm2", W, scale=0.2)
            E, ff = mlp["router"]["experts"], mlp["expert"]["ff"]
            put(p + "mlp.router", E, W, scale=2.0 * W ** -0.5)
            for e in range(E):
                put(p + "mlp.e%d.gate" % e, ff, W)
                put(p + "mlp.e%d.up" % e, ff, W)
                put(p + "mlp.e%d.down" % e, W, ff)
    put("final.norm", W, scale=0.2)
    put("head", cfg["vocab"], W)
    return w
