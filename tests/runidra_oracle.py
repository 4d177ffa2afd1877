"""A plain float64 implementation of the Runidra design, one function per
mechanism, for the tests to compare the serving path against. It shares no
code with the package: whole sequences only, no cache, no batching, python
loops where they are clearest.

Weights are a dict name -> float64 tensor with the checkpoint's names
('embed', 'l<i>.norm1', 'l<i>.mix.q', 'l<i>.hc1.in', ...); the config is the
dict that config.json holds.
"""

from __future__ import annotations

import math

import torch

F64 = torch.float64


def rms_norm(x, w, eps):
    """x / sqrt(mean(x^2) + eps) * w over the last dimension (w None: 1)."""
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if w is None else y * w


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def silu(z):
    return z / (1.0 + torch.exp(-z))


def layer_order(cfg):
    """Indices of the layers in the order they run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return list(range(n))
    order = []
    for i in range(loop["start"]):
        order.append(i)
    for _ in range(loop["times"]):
        for i in range(loop["start"], loop["stop"]):
            order.append(i)
    for i in range(loop["stop"], n):
        order.append(i)
    return order


def hyper_read(streams, coef):
    """streams [S, n, W] -> sum_s coef[s] x_s."""
    u = torch.zeros_like(streams[0])
    for s in range(streams.shape[0]):
        u = u + coef[s] * streams[s]
    return u


def hyper_write(streams, mix, write, y):
    """x_t <- sum_s mix[s, t] x_s + write[t] y, mix[from, to]."""
    out = []
    for t in range(streams.shape[0]):
        x = write[t] * y
        for s in range(streams.shape[0]):
            x = x + mix[s, t] * streams[s]
        out.append(x)
    return torch.stack(out)


def mlstm_gates(h, w, p, cap):
    """(log input gate, log forget gate), each [n, heads]."""
    i = cap * torch.tanh((h @ w[p + "i"].T + w[p + "i.b"]) / cap)
    z = cap * torch.tanh((h @ w[p + "f"].T + w[p + "f.b"]) / cap)
    return i, -torch.log1p(torch.exp(-z))


def mlstm_cell(q, k, v, i, f):
    """One head, token by token: q, k [n, d] (q scaled), v [n, dv], i, f [n].
    Returns (o [n, dv], S, n, m at the end)."""
    d, dv = k.shape[1], v.shape[1]
    S, nrm, m = torch.zeros(d, dv, dtype=F64), torch.zeros(d, dtype=F64), 0.0
    out = []
    for t in range(q.shape[0]):
        m_new = max(float(f[t]) + m, float(i[t]))
        keep, add = math.exp(float(f[t]) + m - m_new), math.exp(float(i[t]) - m_new)
        S = keep * S + add * torch.outer(k[t], v[t])
        nrm = keep * nrm + add * k[t]
        m = m_new
        den = max(abs(float(nrm @ q[t])), math.exp(-m)) + 1e-6
        out.append((S.T @ q[t]) / den)
    return torch.stack(out), S, nrm, m


def mlstm(h, w, p, mx, eps, return_state=False):
    H, d, dv = mx["heads"], mx["dim"], mx["vdim"]
    q = (h @ w[p + "q"].T).view(-1, H, d) * d ** -0.5
    k = (h @ w[p + "k"].T).view(-1, H, d)
    v = (h @ w[p + "v"].T).view(-1, H, dv)
    i, f = mlstm_gates(h, w, p, mx["gate_cap"])
    heads = [mlstm_cell(q[:, a], k[:, a], v[:, a], i[:, a], f[:, a]) for a in range(H)]
    o = torch.cat([rms_norm(c[0], None, eps) for c in heads], dim=-1)
    o = o * w[p + "norm"] * torch.sigmoid(h @ w[p + "g"].T)
    y = o @ w[p + "o"].T
    return (y, [c[1:] for c in heads]) if return_state else y


def rotate_pairs(x, positions, base):
    """x [n, ..., dims]: pair (2i, 2i + 1) turned by p * base^(-2i / dims)."""
    dims = x.shape[-1]
    out = x.clone()
    for i in range(dims // 2):
        ang = positions.to(F64) * base ** (-2.0 * i / dims)
        c, s = torch.cos(ang), torch.sin(ang)
        while c.dim() < x.dim() - 1:
            c, s = c.unsqueeze(-1), s.unsqueeze(-1)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def latent_scores(h, w, p, mx, eps):
    """(scores [heads, n, n], values [n, heads, dv])."""
    H, d, r, dv, R = mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"], mx["kv_rank"]
    pos = torch.arange(h.shape[0])
    base = mx["rot"]["base"]
    cq = rms_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], eps)
    q = (cq @ w[p + "uq"].T).view(-1, H, d + r)
    down = h @ w[p + "dkv"].T
    c = rms_norm(down[:, :R], w[p + "dkv.norm"], eps)
    k_rot = rotate_pairs(down[:, R:], pos, base)
    k = (c @ w[p + "uk"].T).view(-1, H, d)
    v = (c @ w[p + "uv"].T).view(-1, H, dv)
    q_rot = rotate_pairs(q[..., d:], pos, base)
    s = torch.stack([q[:, a, :d] @ k[:, a].T + q_rot[:, a] @ k_rot.T for a in range(H)])
    return s * mx["scale"], v


def sink_softmax(s, sink, window):
    """s [heads, n, n] -> weights; query i sees i - window < j <= i; the
    denominator also holds exp(sink)."""
    n = s.shape[-1]
    i = torch.arange(n)
    dist = i[:, None] - i[None, :]
    seen = (dist >= 0) & (dist < window)
    s = s.masked_fill(~seen, float("-inf"))
    top = torch.maximum(s.max(-1, keepdim=True).values, sink.view(-1, 1, 1))
    e = torch.exp(s - top)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink.view(-1, 1, 1) - top))


def latent_attention(h, w, p, mx, eps):
    s, v = latent_scores(h, w, p, mx, eps)
    a = sink_softmax(s, w[p + "sink"], mx["mask"]["size"])
    o = torch.cat([a[x] @ v[:, x] for x in range(mx["heads"])], dim=-1)
    return o @ w[p + "o"].T


def dense_ff(h, w, p):
    g = gelu_tanh(h @ w[p + "gate"].T + w[p + "gate.b"])
    return (g * (h @ w[p + "up"].T + w[p + "up.b"])) @ w[p + "down"].T + w[p + "down.b"]


def expert(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route(h, w, p, top):
    """Per token [(expert, weight), ...]: softmax over the chosen logits."""
    z = h @ w[p + "router"].T + w[p + "router.b"]
    out = []
    for t in range(h.shape[0]):
        best = sorted(range(z.shape[1]), key=lambda e: -float(z[t, e]))[:top]
        e = [math.exp(float(z[t, b] - z[t, best[0]])) for b in best]
        out.append([(b, x / sum(e)) for b, x in zip(best, e)])
    return out


def moe(h, w, p, mlp):
    y = torch.zeros_like(h)
    for t, chosen in enumerate(route(h, w, p, mlp["router"]["top"])):
        for e, weight in chosen:
            y[t] = y[t] + weight * expert(h[t], w, p + "e%d." % e)
    if mlp.get("shared"):
        y = y + torch.sigmoid(h @ w[p + "shared.sg"].T) * expert(h, w, p + "shared.")
    return y


def forward(cfg, w, tokens, return_layers=False):
    """Logits [n, vocab] (and the sum of the streams after every layer run)."""
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.tensor(tokens)]
    streams = torch.stack([x for _ in range(cfg["streams"])])
    layers = []
    for n in layer_order(cfg):
        sp, p = cfg["layers"][n], "l%d." % n
        h = rms_norm(hyper_read(streams, w[p + "hc1.in"]), w[p + "norm1"], eps)
        mixer = mlstm if sp["type"] == "mlstm" else latent_attention
        y = mixer(h, w, p + "mix.", sp["mixer"], eps)
        streams = hyper_write(streams, w[p + "hc1.mix"], w[p + "hc1.out"], y)
        mlp = sp["mlp"]
        if mlp is not None:
            h = rms_norm(hyper_read(streams, w[p + "hc2.in"]), w[p + "norm2"], eps)
            y = dense_ff(h, w, p + "mlp.") if mlp["kind"] == "dense" \
                else moe(h, w, p + "mlp.", mlp)
            streams = hyper_write(streams, w[p + "hc2.mix"], w[p + "hc2.out"], y)
        layers.append(streams.sum(0))
    z = rms_norm(streams.sum(0), w["final.norm"], eps) @ w["head"].T * cfg["logit_scale"]
    cap = cfg["logit_softcap"]
    z = cap * torch.tanh(z / cap)
    return (z, layers) if return_layers else z


def random_weights(cfg, seed):
    """Weights that a bf16 checkpoint holds exactly."""
    g = torch.Generator().manual_seed(seed)
    w = {}

    def put(name, *shape, scale=None, shift=0.0):
        s = scale if scale is not None else shape[-1] ** -0.5
        w[name] = (torch.randn(*shape, generator=g) * s + shift).bfloat16().to(F64)

    W, V, S = cfg["width"], cfg["vocab"], cfg["streams"]
    put("embed", V, W, scale=1.0)
    put("head", V, W)
    put("final.norm", W, scale=0.2, shift=1.0)
    for n, sp in enumerate(cfg["layers"]):
        p, mx, mlp = "l%d." % n, sp["mixer"], sp["mlp"]
        H, d, dv = mx["heads"], mx["dim"], mx["vdim"]
        for q in ("1", "2") if mlp is not None else ("1",):
            put(p + "norm" + q, W, scale=0.2, shift=1.0)
            put(p + "hc%s.in" % q, S, scale=0.4, shift=0.6)
            put(p + "hc%s.out" % q, S, scale=0.15, shift=0.3)
            put(p + "hc%s.mix" % q, S, S, scale=0.25)
            w[p + "hc%s.mix" % q] += 0.75 * torch.eye(S, dtype=F64)
            w[p + "hc%s.mix" % q] = w[p + "hc%s.mix" % q].bfloat16().to(F64)
        m = p + "mix."
        if sp["type"] == "mlstm":
            put(m + "q", H * d, W)
            put(m + "k", H * d, W)
            put(m + "v", H * dv, W)
            put(m + "g", H * dv, W)
            put(m + "norm", H * dv, scale=0.2, shift=1.0)
            put(m + "o", W, H * dv)
            put(m + "i", H, W)
            put(m + "i.b", H)
            put(m + "f", H, W)
            put(m + "f.b", H, scale=1.0, shift=3.0)
        else:
            Q, R, r = mx["q_rank"], mx["kv_rank"], mx["rot_dim"]
            put(m + "dq", Q, W)
            put(m + "dq.norm", Q, scale=0.2, shift=1.0)
            put(m + "uq", H * (d + r), Q)
            put(m + "dkv", R + r, W)
            put(m + "dkv.norm", R, scale=0.2, shift=1.0)
            put(m + "uk", H * d, R)
            put(m + "uv", H * dv, R)
            put(m + "sink", H, scale=1.0)
            put(m + "o", W, H * dv)
        if mlp is None:
            continue
        m = p + "mlp."
        if mlp["kind"] == "dense":
            for name, a, b in (("gate", mlp["ff"], W), ("up", mlp["ff"], W),
                               ("down", W, mlp["ff"])):
                put(m + name, a, b)
                put(m + name + ".b", a, scale=0.3)
        else:
            E, ff = mlp["router"]["experts"], mlp["expert"]["ff"]
            put(m + "router", E, W)
            put(m + "router.b", E, scale=0.5)
            parts = [("e%d." % e, ff) for e in range(E)]
            if mlp.get("shared"):
                parts.append(("shared.", mlp["shared"]["ff"]))
                put(m + "shared.sg", 1, W)
            for name, f in parts:
                put(m + name + "gate", f, W)
                put(m + name + "up", f, W)
                put(m + name + "down", W, f)
    return w
