"""Tabedra in plain float64 torch, one function per mechanism, written from the design's equations for the tests to compare the
engine against.  Nothing here is shared with the product path: every sequence is run whole, with an explicit list of what each
position sees; convolutions, streams and experts are walked one term at a time.

    W: checkpoint-named tensors (float64), cfg: the config.json dict, tokens: one sequence.
"""
import math

import torch

D = torch.float64


def layer_norm(x, w, b, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w + b


def unit(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def bigram_row(prev, token, spec):
    """Row of the bigram table for `token` after `prev` (None: the token opens its sequence)."""
    return spec["buckets"] if prev is None else (prev * spec["mul_prev"] + token * spec["mul_cur"]) % spec["buckets"]


def embed(W, cfg, tokens):
    rows = []
    for p, t in enumerate(tokens):
        r = bigram_row(tokens[p - 1] if p else None, t, cfg["embedding"]["bigram"])
        rows.append(W["embed"][t] + W["bigram"][r] + W["pos"][p])
    return torch.stack(rows)


def causal_conv(u, w):
    """u [T, C], w [C, taps]: the last tap lies on the token itself."""
    T, taps = u.shape[0], w.shape[1]
    y = torch.zeros_like(u)
    for t in range(T):
        for j in range(taps):
            at = t - taps + 1 + j
            if at >= 0:
                y[t] += w[:, j] * u[at]
    return y


def bucket(n, rows, reach):
    half = rows // 2
    if n < half:
        return n
    return min(rows - 1, half + math.floor(math.log(n / half) / math.log(reach / half) * (rows - half)))


def softmax_mix(scores, values):
    e = torch.exp(scores - scores.max())
    return (e[:, None] * values).sum(0) / e.sum()


def attend(q, k, v, scale, rel, reach, window, only=None):
    """q [T, H, d], k [T, G, d], v [T, G, dv] -> [T, H, dv]; position i sees the `window` positions up to itself (0: all of them); the
    bias rel [rows, H] is added to the scaled score.  `only`: the positions to compute (others stay zero)."""
    T, H, G = q.shape[0], q.shape[1], k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=D)
    of_distance = [bucket(n, rel.shape[0], reach) for n in range(T)]
    for i in range(T) if only is None else only:
        first = max(0, i - window + 1) if window else 0
        rows = torch.tensor([of_distance[i - j] for j in range(first, i + 1)])
        for h in range(H):
            g = h // (H // G)
            s = (k[first:i + 1, g] @ q[i, h]) * scale + rel[rows, h]
            out[i, h] = softmax_mix(s, v[first:i + 1, g])
    return out


def attention(W, p, m, h, eps, kept):
    """`kept`: (keys, values) of another layer, or None; returns the result and what this layer attended over."""
    T, H, G, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]

    def projected(leaf):
        return causal_conv(h @ W[p + leaf].T, W[p + leaf + ".conv"])

    q = unit(projected("q").view(T, H, d), eps)
    if kept is None:
        kept = unit(projected("k").view(T, G, d), eps), projected("v").view(T, G, dv)
    o = attend(q, kept[0], kept[1], m["scale"], W[p + "rel"], m["bias_max"], m["mask"]["size"] if m.get("mask") else 0)
    return (o.reshape(T, H * dv) * torch.sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T, kept


def expert(W, name, x):
    return torch.clamp(x @ W[name + ".up"].T, min=0.0) ** 2 @ W[name + ".down"].T


def route(logits, correction, top):
    """[(expert, weight)] of one token."""
    s = torch.softmax(logits, -1)
    chosen = sorted(range(len(s)), key=lambda e: (-float(s[e] + correction[e]), e))[:top]
    total = sum(float(s[e]) for e in chosen) + 1e-20
    return [(e, float(s[e]) / total) for e in chosen]


def experts(W, p, m, h):
    out = expert(W, p + "shared", h) if m.get("shared") else torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in route(W[p + "router"] @ h[t], W[p + "correction"], m["router"]["top"]):
            out[t] = out[t] + w * expert(W, f"{p}e{e}", h[t])
    return out


def around(W, p, q, streams, sublayer, eps):
    """One sublayer between the streams: what it reads, and what every stream becomes."""
    u = sum(W[f"{p}hc{q}.in"][s] * x for s, x in enumerate(streams))
    y = sublayer(layer_norm(u, W[f"{p}norm{q}"], W[f"{p}norm{q}.b"], eps))
    return [sum(W[f"{p}hc{q}.mix"][s, t] * x for s, x in enumerate(streams)) + W[f"{p}hc{q}.out"][t] * y for t in range(len(streams))]


def forward(W, cfg, tokens, collect=None):
    """fp64 logits [T, vocab]; `collect` (a list) receives the sum of the streams after every layer."""
    eps = cfg["norm"]["eps"]
    streams = [embed(W, cfg, tokens)] * cfg["streams"]
    kept = {}
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]

        def mixer(h):
            y, kept[i] = attention(W, p + "mix.", m, h, eps, kept[m["kv_from"]] if m.get("kv_from") is not None else None)
            return y

        streams = around(W, p, 1, streams, mixer, eps)
        if L.get("mlp"):
            streams = around(W, p, 2, streams, lambda h: experts(W, p + "mlp.", L["mlp"], h), eps)
        if collect is not None:
            collect.append(sum(streams))
    return layer_norm(sum(streams), W["final.norm"], W["final.norm.b"], eps) @ W["head"].T
