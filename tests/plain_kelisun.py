"""A plain, slow implementation of the Kelisun design: torch on the CPU in float64, one function per mechanism, keys and
values expanded from the latent, every expert a loop.  It shares nothing with the engine.

The design: the normed embedding enters `streams` equal copies of the residual.  Around a sublayer (the layer's attention,
then its experts), with the sublayer's coefficients a (s numbers), b (s numbers) and M (s x s):
    u = sum over s of a[s] x_s;  y = sublayer(norm(u));  x_t <- sum over s of M[s, t] x_s + b[t] y   (all t at once)
The attention goes through a latent, sees a window of the last keys, rotates one shared key part by stretched frequencies,
and counts a learned number a head as one more entry of the softmax's denominator.  The experts are chosen by groups.  A
layer may use another layer's weights.  At the end the streams are added, normed and projected to the vocabulary.
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w.to(F64)


def silu(z):
    return z * torch.sigmoid(z)


def frequencies(rot):
    """(f [dims / 2], the factor on cosine and sine).  A pair whose wavelength is short against the trained length keeps its
    frequency, a long one is divided by the factor, and a ramp over the pairs' indices lies between."""
    dims, base = rot["dims"], rot["base"]
    f = base ** (-2.0 * torch.arange(dims // 2, dtype=F64) / dims)
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0

    def index_of(turns):
        return dims * math.log(sc["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    low = max(math.floor(index_of(sc["fast"])), 0)
    high = min(math.ceil(index_of(sc["slow"])), dims - 1)
    ramp = ((torch.arange(dims // 2, dtype=F64) - low) / max(high - low, 0.001)).clamp(0.0, 1.0)
    return f / sc["factor"] * ramp + f * (1.0 - ramp), 0.1 * math.log(sc["factor"]) + 1.0


def rotate_halves(x, positions, rot):
    """x [T, heads, dims]: entries i and i + dims/2 form a pair that turns by position * f_i and is stretched by the factor."""
    f, mag = frequencies(rot)
    half = rot["dims"] // 2
    ang = positions.to(F64)[:, None] * f[None, :]
    cos, sin = (torch.cos(ang) * mag)[:, None, :], (torch.sin(ang) * mag)[:, None, :]
    u, v = x[..., :half], x[..., half:]
    return torch.cat([u * cos - v * sin, v * cos + u * sin], dim=-1)


def visible(T, window):
    """[T, T]: whether row i sees key j: itself and the window - 1 keys before it."""
    back = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    return (back >= 0) & (back < window)


def latent_attention(m, w, p, h, eps):
    """Attention of one sequence from position 0; h [T, width]."""
    T = h.shape[0]
    H, d, dr, dv, r = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    positions = torch.arange(T)
    q = (h @ w[p + "q"].to(F64).T).view(T, H, d + dr)
    q_flat, q_rot = q[..., :d], rotate_halves(q[..., d:], positions, m["rot"])
    down = h @ w[p + "dkv"].to(F64).T
    c = norm(down[:, :r], w[p + "dkv.norm"], eps)
    k_rot = rotate_halves(down[:, None, r:], positions, m["rot"])[:, 0]
    k = (c @ w[p + "uk"].to(F64).T).view(T, H, d)
    v = (c @ w[p + "uv"].to(F64).T).view(T, H, dv)
    see = visible(T, m["mask"]["size"])
    out = torch.zeros(T, H, dv, dtype=F64)
    for head in range(H):
        s = (q_flat[:, head] @ k[:, head].T + q_rot[:, head] @ k_rot.T) * m["scale"]
        s = s.masked_fill(~see, -math.inf)
        sink = w[p + "sink"][head].to(F64)
        top = torch.maximum(s.max(dim=1).values, sink)
        e = torch.exp(s - top[:, None])
        out[:, head] = (e @ v[:, head]) / (e.sum(1) + torch.exp(sink - top))[:, None]
    return out.reshape(T, H * dv) @ w[p + "o"].to(F64).T


def expert(w, p, h):
    return (silu(h @ w[p + "gate"].to(F64).T) * (h @ w[p + "up"].to(F64).T)) @ w[p + "down"].to(F64).T


def route(router, w, p, h):
    """The chosen experts [T, top] (largest score first) and their weights: softmax scores over all experts times the scale."""
    E, top = router["experts"], router["top"]
    groups = router.get("groups") or {"count": 1, "keep": 1}
    size = E // groups["count"]
    s = torch.softmax(h @ w[p + "router"].to(F64).T, dim=-1)
    idx = torch.zeros(h.shape[0], top, dtype=torch.long)
    for t in range(h.shape[0]):
        best = sorted(range(groups["count"]), key=lambda g: -float(s[t, g * size:(g + 1) * size].max()))[:groups["keep"]]
        allowed = [e for e in range(E) if e // size in best]
        idx[t] = torch.tensor(sorted(allowed, key=lambda e: -float(s[t, e]))[:top])
    return idx, torch.gather(s, 1, idx) * router.get("scale", 1.0)


def experts(mlp, w, p, h):
    idx, wts = route(mlp["router"], w, p, h)
    out = torch.zeros_like(h)
    for e in range(mlp["router"]["experts"]):
        rows, place = (idx == e).nonzero(as_tuple=True)
        if len(rows):
            out[rows] += wts[rows, place][:, None] * expert(w, f"{p}e{e}.", h[rows])
    return out


def hyper(streams, w, p, sublayer):
    """One sublayer around s streams [s, T, width]: read a mixture of them, write its output back while they mix."""
    a, b, M = w[p + "in"].to(F64), w[p + "out"].to(F64), w[p + "mix"].to(F64)
    u = torch.einsum("s,stw->tw", a, streams)
    y = sublayer(u)
    return torch.einsum("sz,stw->ztw", M, streams) + b[:, None, None] * y[None]


def source(cfg, i):
    """The layer whose tensors layer i uses."""
    while cfg["layers"][i].get("weights_of") is not None:
        i = cfg["layers"][i]["weights_of"]
    return i


def forward(cfg, w, tokens, streams=None):
    """Logits [T, vocab] in float64 for one sequence from position 0.  streams: a list that receives the sum of the
    residual streams after every layer."""
    eps = cfg["norm"]["eps"]
    x = norm(w["embed"].to(F64)[torch.tensor(tokens)], w["embed.norm"], eps)
    xs = x[None].repeat(cfg["streams"], 1, 1)
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{source(cfg, i)}."
        if layer["type"] != "latent_attention":
            raise ValueError(layer["type"])
        xs = hyper(xs, w, p + "hc1.", lambda u: latent_attention(layer["mixer"], w, p + "mix.", norm(u, w[p + "norm1"], eps), eps))
        if layer.get("mlp"):
            xs = hyper(xs, w, p + "hc2.", lambda u: experts(layer["mlp"], w, p + "mlp.", norm(u, w[p + "norm2"], eps)))
        if streams is not None:
            streams.append(xs.sum(0))
    return norm(xs.sum(0), w["final.norm"], eps) @ w["head"].to(F64).T


def generate_greedy(cfg, w, prompt, n):
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(torch.argmax(forward(cfg, w, seq)[-1])))
    return seq[len(prompt):]
