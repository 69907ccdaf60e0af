"""A plain, slow implementation of the Puvirax design: torch on the CPU in float64, one function per mechanism, every expert and
every head a loop.  It shares nothing with the engine.

The design: a token's embedding plus a row of a second table that the token and the one before it pick enters the residual
stream; layers of softmax attention and a feed-forward, each behind a norm, add to it; the model's norm and the embedding
table, times a constant, give the logits.  Three kinds of attention, chosen layer by layer:
    rotated      all earlier keys; the first entries of q and k turn with the position (frequencies by bands), then every head of
                 q and k is divided by its root mean square; a head's output is multiplied by the logistic function of a number
    windowed     the last keys only; head norms with one weight for all heads; a learned number a head and distance class
    unrotated    all earlier keys; one norm over all heads' entries together; a learned number a head and distance class
In layers that mix values, all but the first of them blend their values with that first one's.
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm(x, w, eps):
    return rms(x, eps) * w.to(F64)


def squared_relu(z):
    return torch.clamp(z, min=0.0) ** 2


def bigram_rows(b, tokens):
    """The row of the second table for every token of a sequence: a hash of the token and its predecessor; the last row for
    the first token."""
    return [b["buckets"] if i == 0 else (tokens[i - 1] * b["mul_prev"] + tokens[i] * b["mul_cur"]) % b["buckets"] for i in range(len(tokens))]


def embed(cfg, w, tokens):
    x = w["embed"].to(F64)[torch.tensor(tokens)]
    b = cfg.get("embedding", {}).get("bigram")
    return x + w["bigram"].to(F64)[torch.tensor(bigram_rows(b, tokens))] if b else x


def frequencies(rot):
    """f [dims / 2].  With a scaling, the wavelength decides: short ones keep their frequency, long ones are divided by the factor,
    a linear blend over original / wavelength lies between."""
    out = []
    for i in range(rot["dims"] // 2):
        f = rot["base"] ** (-2.0 * i / rot["dims"])
        sc = rot.get("scaling")
        if sc:
            length = 2.0 * math.pi / f
            if length > sc["original"] / sc["low"]:
                f = f / sc["factor"]
            elif length >= sc["original"] / sc["high"]:
                s = (sc["original"] / length - sc["low"]) / (sc["high"] - sc["low"])
                f = (1.0 - s) * f / sc["factor"] + s * f
        out.append(f)
    return torch.tensor(out, dtype=F64)


def rotate(x, rot):
    """x [T, heads, dim]: entries i and i + dims/2 of the first dims form a pair; the others stay."""
    half = rot["dims"] // 2
    ang = torch.arange(x.shape[0], dtype=F64)[:, None] * frequencies(rot)[None, :]
    cos, sin = torch.cos(ang)[:, None, :], torch.sin(ang)[:, None, :]
    u, v, rest = x[..., :half], x[..., half:2 * half], x[..., 2 * half:]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, rest], dim=-1)


def distance_class(n, rows, far):
    """Which of `rows` classes the distance n falls in: one each for the first half, logarithmic ones for the rest."""
    half = rows // 2
    if n < half:
        return n
    return min(rows - 1, half + math.floor(math.log(n / half) / math.log(far / half) * (rows - half)))


def visible(T, window=None):
    """[T, T]: whether row i sees key j: itself and everything before it, or the window - 1 keys before it."""
    back = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    return (back >= 0) & (back < (window or T + 1))


def qk_rotated(m, w, p, q, k, eps):
    return rms(rotate(q, m["rot"]), eps), rms(rotate(k, m["rot"]), eps)


def qk_head_norm(m, w, p, q, k, eps):
    return norm(q, w[p + "q.norm"], eps), norm(k, w[p + "k.norm"], eps)


def qk_whole_norm(m, w, p, q, k, eps):
    return norm(q.flatten(1), w[p + "q.norm"], eps).view_as(q), norm(k.flatten(1), w[p + "k.norm"], eps).view_as(k)


QK = {"attention": qk_rotated, "attention_2": qk_head_norm, "attention_3": qk_whole_norm}


def mix_values(v, first, share):
    """v, first [T, entries]: the blend with the first mixing layer's values of the same token."""
    return (1.0 - share) * v + share * first


def attend(q, k, v, scale, see, bias=None):
    """q [T, H, d], k [T, G, d], v [T, G, dv]; bias [T, T, H] or None -> [T, H, dv]."""
    T, H, G = q.shape[0], q.shape[1], k.shape[1]
    out = torch.zeros(T, H, v.shape[-1], dtype=F64)
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * scale
        if bias is not None:
            s = s + bias[:, :, h]
        out[:, h] = torch.softmax(s.masked_fill(~see, -math.inf), dim=-1) @ v[:, g]
    return out


def distance_bias(table, far, T):
    """[T, T, H]; entries for keys after the row stay zero."""
    cls = torch.tensor([distance_class(n, table.shape[0], far) for n in range(T)])
    back = (torch.arange(T)[:, None] - torch.arange(T)[None, :]).clamp(min=0)
    return table.to(F64)[cls[back]]


def attention(kind, m, w, p, h, eps, first):
    """Attention of one sequence from position 0; h [T, width].  first: {"v": values of the first mixing layer} or {} so far."""
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].to(F64).T).view(T, H, d)
    k = (h @ w[p + "k"].to(F64).T).view(T, G, d)
    v = h @ w[p + "v"].to(F64).T
    q, k = QK[kind](m, w, p, q, k, eps)
    if m.get("v_mix"):
        if "v" in first:
            v = mix_values(v, first["v"], w[p + "vmix"].to(F64))
        else:
            first["v"] = v
    mask = m.get("mask")
    bias = None if kind == "attention" else distance_bias(w[p + "rel"], m["bias_max"], T)
    out = attend(q, k, v.view(T, G, dv), m["scale"], visible(T, mask["size"] if mask else None), bias)
    if kind == "attention":
        out = out * torch.sigmoid(h @ w[p + "g"].to(F64).T)[:, :, None]
    return out.reshape(T, H * dv) @ w[p + "o"].to(F64).T


def dense(w, p, h):
    return squared_relu(h @ w[p + "up"].to(F64).T) @ w[p + "down"].to(F64).T


def route(router, w, p, h):
    """The chosen experts [T, top] (largest choice score first) and their weights: the logistic scores without the correction."""
    E, top = router["experts"], router["top"]
    groups = router.get("groups") or {"count": 1, "keep": 1}
    size = E // groups["count"]
    s = torch.sigmoid(h @ w[p + "router"].to(F64).T)
    choice = s + w[p + "correction"].to(F64)
    idx = torch.zeros(h.shape[0], top, dtype=torch.long)
    for t in range(h.shape[0]):
        def worth(g):
            return sum(sorted(choice[t, g * size:(g + 1) * size].tolist(), reverse=True)[:2])
        best = sorted(range(groups["count"]), key=lambda g: -worth(g))[:groups["keep"]]
        allowed = [e for e in range(E) if e // size in best]
        idx[t] = torch.tensor(sorted(allowed, key=lambda e: -float(choice[t, e]))[:top])
    return idx, torch.gather(s, 1, idx)


def experts(mlp, w, p, h):
    idx, wts = route(mlp["router"], w, p, h)
    out = dense(w, p + "shared.", h) if mlp.get("shared") else torch.zeros_like(h)
    for e in range(mlp["router"]["experts"]):
        rows, place = (idx == e).nonzero(as_tuple=True)
        if len(rows):
            out[rows] += wts[rows, place][:, None] * dense(w, f"{p}e{e}.", h[rows])
    return out


def forward(cfg, w, tokens, streams=None):
    """Logits [T, vocab] in float64 for one sequence from position 0.  streams: a list that receives the residual stream
    after every layer."""
    eps = cfg["norm"]["eps"]
    x = embed(cfg, w, list(tokens))
    first = {}
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        x = x + attention(layer["type"], layer["mixer"], w, p + "mix.", norm(x, w[p + "norm1"], eps), eps, first)
        mlp = layer.get("mlp")
        if mlp:
            h = norm(x, w[p + "norm2"], eps)
            x = x + (dense(w, p + "mlp.", h) if mlp["kind"] == "dense" else experts(mlp, w, p + "mlp.", h))
        if streams is not None:
            streams.append(x)
    return norm(x, w["final.norm"], eps) @ w["embed"].to(F64).T * cfg.get("logit_scale", 1.0)


def generate_greedy(cfg, w, prompt, n):
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(torch.argmax(forward(cfg, w, seq)[-1])))
    return seq[len(prompt):]
