"""Mopalorn in plain float64 torch, one function per mechanism, written from the design's equations for the tests to compare the
engine against.  Nothing here is shared with the product path: every sequence is run whole, with an explicit list of what each
position sees; the keys and values of the latent attention are formed per head.

    W: checkpoint-named tensors (float64), cfg: the config.json dict, tokens: one sequence.
"""
import math

import torch

D = torch.float64


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def rotate_halves(x, rot):
    """x [T, heads, size]: entries (i, i + dims/2) of every head are turned by position * base^(-2i/dims), i < dims/2."""
    half = rot["dims"] // 2
    freq = torch.tensor([rot["base"] ** (-2.0 * i / rot["dims"]) for i in range(half)], dtype=D)
    ang = torch.arange(x.shape[0], dtype=D)[:, None, None] * freq
    c, s = torch.cos(ang), torch.sin(ang)
    out = x.clone()
    a, b = x[..., :half], x[..., half:2 * half]
    out[..., :half], out[..., half:2 * half] = a * c - b * s, b * c + a * s
    return out


def temperature(p, spec):
    """What the query at position p is multiplied by."""
    return 1.0 + spec["coef"] * math.log((p + 1) // spec["every"] + 1) if spec else 1.0


def softcap(s, cap):
    return cap * torch.tanh(s / cap) if cap else s


def pooled_blocks(i, size, pool):
    """How many whole blocks of `pool` positions lie before the window of the query at position i."""
    return max(0, (i - size + 1) // pool)


def block_mean(x, b, pool):
    return x[b * pool:(b + 1) * pool].mean(0)


def softmax_mix(scores, values, sink=None):
    """Softmax of `scores` [n] over `values` [n, dv], with an optional logit that only the denominator sees."""
    top = float(scores.max())
    if sink is not None:
        top = max(top, float(sink))
    e = torch.exp(scores - top)
    den = e.sum() + (math.exp(float(sink) - top) if sink is not None else 0.0)
    return (e[:, None] * values).sum(0) / den


def attend(q, k, v, scale, window=0, pool=0, sinks=None, cap=0.0, q_temp=None):
    """q [T, H, d], k [T, G, d], v [T, G, dv] -> [T, H, dv].  window > 0: the last `window` positions; with `pool` also one mean key
    and value per block of `pool` positions that lies wholly before the window."""
    T, H = q.shape[0], q.shape[1]
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=D)
    for g in range(G):
        kb = torch.stack([block_mean(k[:, g], b, pool) for b in range(T // pool)]) if pool and T >= pool else k[:0, g]
        vb = torch.stack([block_mean(v[:, g], b, pool) for b in range(T // pool)]) if pool and T >= pool else v[:0, g]
        for h in range(g * (H // G), (g + 1) * (H // G)):
            for i in range(T):
                first = max(0, i - window + 1) if window else 0
                n = pooled_blocks(i, window, pool) if pool else 0
                keys = torch.cat([kb[:n], k[first:i + 1, g]])
                vals = torch.cat([vb[:n], v[first:i + 1, g]])
                s = softcap((keys @ (q[i, h] * temperature(i, q_temp))) * scale, cap)
                out[i, h] = softmax_mix(s, vals, None if sinks is None else sinks[h])
    return out


def latent_attention(W, p, m, h, eps):
    T, H, d, r, dv, n = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = (h @ W[p + "q"].T).view(T, H, d + r)
    down = h @ W[p + "dkv"].T
    c = rms_norm(down[:, :n], W[p + "dkv.norm"], eps)
    k_rot = rotate_halves(down[:, n:].view(T, 1, r), m["rot"]).expand(T, H, r)
    k = torch.cat([(c @ W[p + "uk"].T).view(T, H, d), k_rot], -1)
    v = (c @ W[p + "uv"].T).view(T, H, dv)
    q = torch.cat([q[..., :d], rotate_halves(q[..., d:], m["rot"])], -1)
    o = attend(q, k, v, m["scale"], window=m["mask"]["size"] if m.get("mask") else 0)
    return (o.reshape(T, H * dv) * torch.sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


def mixed_values(v, lam, first):
    return v if first is None else (1.0 - lam) * v + lam * first


def head_attention(W, p, m, h, kind, first_values):
    """The two attentions with keys and values per head; returns the result and this layer's own values as projected."""
    T, H, d = h.shape[0], m["heads"], m["dim"]
    G, dv = m["kv_heads"], m["vdim"]
    q, k, own = (h @ W[p + "q"].T).view(T, H, d), (h @ W[p + "k"].T).view(T, G, d), h @ W[p + "v"].T
    v = mixed_values(own, W.get(p + "vmix"), first_values if m.get("v_mix") else None).view(T, G, dv)
    if kind == "attention":
        o = attend(q, k, v, m["scale"], cap=m.get("softcap") or 0.0, q_temp=m.get("q_temp"))
    else:
        o = attend(q, k, v, m["scale"], window=m["mask"]["size"], pool=m["mask"]["pool"], sinks=W[p + "sink"])
    return o.reshape(T, H * dv) @ W[p + "o"].T, own


def xielu(z, p, q):
    sp = lambda t: math.log1p(math.exp(float(t)))
    return torch.where(z > 0, sp(p) * z * z + z / 2, (0.5 + sp(q)) * (torch.exp(torch.clamp(z, max=0.0)) - 1 - z) + z / 2)


def feed_forward(W, p, h):
    return xielu(h @ W[p + "up"].T, W[p + "act"][0], W[p + "act"][1]) @ W[p + "down"].T


def forward(W, cfg, tokens, collect=None):
    """fp64 logits [T, vocab]; `collect` (a list) receives the stream after every layer."""
    eps = cfg["norm"]["eps"]
    x = W["embed"][torch.tensor(tokens)]
    first_values = None
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        h = rms_norm(x, W[p + "norm1"], eps)
        if L["type"] == "latent_attention":
            y = latent_attention(W, p + "mix.", m, h, eps)
        else:
            y, own = head_attention(W, p + "mix.", m, h, L["type"], first_values)
            if m.get("v_mix") and first_values is None:
                first_values = own
        x = x + rms_norm(y, W[p + "norm1b"], eps)
        if L.get("mlp"):
            x = x + rms_norm(feed_forward(W, p + "mlp.", rms_norm(x, W[p + "norm2"], eps)), W[p + "norm2b"], eps)
        if collect is not None:
            collect.append(x.clone())
    return rms_norm(x, W["final.norm"], eps) @ W["embed"].T * cfg["logit_scale"]
