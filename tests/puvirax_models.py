"""Small Puvirax models for the tests: configurations that differ from each other in every size and option, and random
weights for them, written as a model folder (config.json, model.safetensors in bfloat16)."""
from __future__ import annotations

import json
from pathlib import Path

import torch
from safetensors.torch import save_file


def rotated(heads, kv_heads, dim, vdim, dims, base=10000.0, scaling=None, scale=None, mix=True):
    """Every earlier key, a rotation of the first `dims` entries, unit heads, a gate a head.  scaling: (factor, original, low, high)."""
    rot = {"base": base, "dims": dims}
    if scaling:
        rot["scaling"] = dict(zip(("factor", "original", "low", "high"), scaling))
    m = {"dim": dim, "heads": heads, "kv_heads": kv_heads, "rot": rot, "scale": scale if scale is not None else 3.0 / dim, "v_mix": mix, "vdim": vdim}
    return "attention", m


def windowed(heads, kv_heads, dim, vdim, window, far, scale=None, mix=True):
    """The last keys, head norms, a bias by distance."""
    return "attention_2", {"bias_max": far, "dim": dim, "heads": heads, "kv_heads": kv_heads, "mask": {"size": window},
                           "scale": scale if scale is not None else 0.5 * dim ** -0.5, "v_mix": mix, "vdim": vdim}


def unrotated(heads, kv_heads, dim, vdim, far, scale=None, mix=True):
    """Every earlier key, one norm over all heads, a bias by distance."""
    return "attention_3", {"bias_max": far, "dim": dim, "heads": heads, "kv_heads": kv_heads, "scale": scale if scale is not None else 0.5 * dim ** -0.5,
                           "v_mix": mix, "vdim": vdim}


def dense(ff):
    return {"ff": ff, "kind": "dense"}


def moe(experts, top, ff, groups=None, shared=None):
    """groups: (count, keep) or None; shared: the shared expert's size or None."""
    router = {"experts": experts, "top": top}
    if groups:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    mlp = {"expert": {"ff": ff}, "kind": "moe", "router": router}
    if shared:
        mlp["shared"] = {"ff": shared}
    return mlp


def layer(mixer, mlp=None):
    return {"type": mixer[0], "mixer": mixer[1], "mlp": mlp}


def config(layers, width=64, vocab=97, eps=1e-5, buckets=37, mul_prev=5, mul_cur=11, logit_scale=1.0):
    return {"architecture": "Puvirax", "embedding": {"bigram": {"buckets": buckets, "mul_cur": mul_cur, "mul_prev": mul_prev}}, "layers": layers,
            "logit_scale": logit_scale, "norm": {"eps": eps}, "vocab": vocab, "width": width}


# Layers that differ from each other: head sizes that are no multiples of 8 or 16, values wider and narrower than keys, one key
# head for all, as many as query heads, more heads than a tile has rows, windows shorter than a page, equal to one and longer,
# distances that reach their last class early, late and beyond the sequences of the tests, full, partial and banded rotations,
# layers that mix values and some that do not (the first of all among those), a layer that cuts its values into other heads,
# layers without a feed-forward, experts with and without groups and a shared one.
MIXED = config([
    layer(rotated(3, 1, 12, 20, dims=8, base=500.0, scaling=(3.0, 40, 1.0, 4.0), mix=False), dense(40)),
    layer(windowed(4, 2, 20, 12, window=10, far=9), moe(3, 3, 40, shared=24)),
    layer(unrotated(18, 1, 8, 24, far=300), dense(72)),
    layer(windowed(2, 2, 16, 16, window=33, far=64, mix=False)),
    layer(rotated(6, 3, 10, 8, dims=10, base=77.0, scale=0.6)),
    layer(unrotated(5, 5, 14, 20, far=25, mix=False), dense(8)),
    # The routers that choose stand last: where two experts all but tie, the 16-bit engine may choose the other one, and a
    # token that went to another expert in an early layer would change the keys that later tokens read.
    layer(rotated(4, 4, 24, 6, dims=6, base=900.0, scaling=(8.0, 100, 0.5, 2.0)), moe(10, 3, 24, groups=(5, 3))),
    layer(windowed(1, 1, 32, 24, window=16, far=40), moe(8, 2, 12, groups=(2, 1), shared=56)),
], width=64, vocab=97, logit_scale=0.75)
# Heads of the sizes that the shared tiles take, and one between; a width whose vectors do not fill a wave; more buckets than
# tokens; multipliers of one and of nothing.
WIDE = config([
    layer(windowed(4, 2, 64, 64, window=100, far=130), dense(104)),
    layer(rotated(4, 1, 128, 128, dims=64, base=400000.0, scaling=(4.0, 256, 1.0, 4.0), mix=False), dense(64)),
    layer(unrotated(8, 4, 48, 32, far=48), moe(6, 2, 48, groups=(3, 1), shared=64)),
    layer(rotated(2, 2, 256, 64, dims=256, scale=0.02, mix=True)),
    layer(windowed(2, 1, 200, 128, window=64, far=20), moe(16, 5, 64, groups=(4, 2))),
], width=104, vocab=130, buckets=487, mul_prev=1, mul_cur=0, logit_scale=3.0, eps=1e-6)
CONFIGS = {"MIXED": MIXED, "WIDE": WIDE}


def random_weights(cfg, seed, classes=None):
    """classes: rows of every distance table (by default they differ from layer to layer)."""
    g = torch.Generator().manual_seed(seed)

    def normal(*shape, std=1.0):
        return torch.randn(*shape, generator=g) * std

    def uniform(*shape, lo=-1.0, hi=1.0):
        return torch.rand(*shape, generator=g) * (hi - lo) + lo

    W, V = cfg["width"], cfg["vocab"]
    w = {"embed": normal(V, W), "bigram": normal(cfg["embedding"]["bigram"]["buckets"] + 1, W, std=0.7), "final.norm": uniform(W, lo=0.5, hi=1.5)}
    mixing = 0
    for i, spec in enumerate(cfg["layers"]):
        p = f"l{i}."
        m = spec["mixer"]
        H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        w[p + "norm1"] = uniform(W, lo=0.5, hi=1.5)
        w[p + "mix.q"] = normal(H * d, W, std=W ** -0.5)
        w[p + "mix.k"] = normal(G * d, W, std=W ** -0.5)
        w[p + "mix.v"] = normal(G * dv, W, std=W ** -0.5)
        w[p + "mix.o"] = normal(W, H * dv, std=(H * dv) ** -0.5)
        if spec["type"] == "attention":
            w[p + "mix.g"] = normal(H, W, std=1.5 * W ** -0.5)
        else:
            whole = spec["type"] == "attention_3"
            w[p + "mix.q.norm"] = uniform(H * d if whole else d, lo=0.5, hi=2.0)
            w[p + "mix.k.norm"] = uniform(G * d if whole else d, lo=0.5, hi=2.0)
            w[p + "mix.rel"] = normal(classes or (6, 16, 11, 32, 2)[i % 5], H, std=1.5)
        if m.get("v_mix"):
            # The first layer that mixes holds a share as well, and does not use it.
            w[p + "mix.vmix"] = uniform(1, lo=0.2, hi=0.9)[0] if mixing else torch.tensor(7.0)
            mixing += 1
        mlp = spec.get("mlp")
        if not mlp:
            continue
        w[p + "norm2"] = uniform(W, lo=0.5, hi=1.5)

        def relu2(name, F, std):
            w[p + name + ".up"] = normal(F, W, std=W ** -0.5)
            w[p + name + ".down"] = normal(W, F, std=std * F ** -0.5)
        if mlp["kind"] == "dense":
            relu2("mlp", mlp["ff"], 0.7)
            continue
        E = mlp["router"]["experts"]
        w[p + "mlp.router"] = normal(E, W, std=2.0 * W ** -0.5)
        w[p + "mlp.correction"] = uniform(E, lo=-1.5, hi=0.5)          # choice scores on both sides of nothing
        # The experts write less than the attention: an expert chosen otherwise by the 16-bit engine, where two all but
        # tie, then moves a row less (in 32-bit every row is held to rounding anyway).
        for e in range(E):
            relu2(f"mlp.e{e}", mlp["expert"]["ff"], 0.3)
        if mlp.get("shared"):
            relu2("mlp.shared", mlp["shared"]["ff"], 0.5)
    # What the file stores is what both sides compute with.
    return {n: t.to(torch.bfloat16).contiguous() for n, t in w.items()}


def write_model(folder, cfg, weights):
    folder = Path(folder)
    folder.mkdir(parents=True, exist_ok=True)
    (folder / "config.json").write_text(json.dumps(cfg))
    save_file(weights, str(folder / "model.safetensors"))
    return folder
