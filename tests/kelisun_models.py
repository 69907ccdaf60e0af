"""Small Kelisun models for the tests: configurations that differ from each other in every size and option, and random
weights for them, written as a model folder (config.json, model.safetensors in bfloat16)."""
from __future__ import annotations

import json
from pathlib import Path

import torch
from safetensors.torch import save_file


def latent(heads, dim, rot_dim, vdim, kv_rank, window, base=10000.0, scaling=None, scale=None):
    """scaling: (factor, original, fast, slow) or None."""
    rot = {"base": base, "dims": rot_dim}
    if scaling:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return {"dim": dim, "heads": heads, "kv_rank": kv_rank, "mask": {"size": window}, "rot": rot, "rot_dim": rot_dim,
            "scale": scale if scale is not None else (dim + rot_dim) ** -0.5, "vdim": vdim}


def moe(experts, top, ff, groups=None, scale=1.0):
    """groups: (count, keep) or None."""
    router = {"experts": experts, "scale": scale, "top": top}
    if groups:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"expert": {"ff": ff}, "kind": "moe", "router": router}


def layer(mixer, mlp=None):
    return {"type": "latent_attention", "mixer": mixer, "mlp": mlp}


def again(layers, i):
    """A layer that uses layer i's weights."""
    return dict(layers[i], weights_of=i)


def config(layers, width=64, vocab=97, streams=2, eps=1e-5):
    return {"architecture": "Kelisun", "layers": layers, "norm": {"eps": eps}, "streams": streams, "vocab": vocab, "width": width}


# Layers that differ from each other: head and value sizes and latents that are no multiples of 8 or 16, more heads than a
# tile has rows, one head, windows shorter than a page, equal to one and longer, stretched and plain rotations, layers
# without a feed-forward, one expert of one, all experts chosen, one group of several, three of five; three layers that
# share weights, one of them with a layer that comes later.
_LATER = layer(latent(18, 8, 4, 8, kv_rank=16, window=33, scaling=(8.0, 64, 16.0, 1.0)))
_M = [layer(latent(3, 12, 6, 20, kv_rank=20, window=10, base=500.0, scaling=(3.0, 40, 8.0, 0.5)), moe(3, 3, 40, scale=1.5)),
      dict(_LATER, weights_of=5)]
_M += [again(_M, 0), layer(latent(2, 16, 16, 40, kv_rank=48, window=64, base=77.0, scale=0.3), moe(1, 1, 16, scale=0.7))]
_M += [again(_M, 3), _LATER,
       # The two routers that choose stand last: where two experts all but tie, the 16-bit engine may choose the other one,
       # and a token that went to another expert in an early layer would change the keys that later tokens read.
       layer(latent(1, 24, 10, 24, kv_rank=13, window=16, base=900.0), moe(10, 3, 24, groups=(5, 3), scale=2.5)),
       layer(latent(4, 10, 8, 12, kv_rank=30, window=21, scaling=(2.0, 100, 4.0, 1.0)), moe(8, 2, 12, groups=(2, 1)))]
MIXED = config(_M, width=64, vocab=97, streams=3)
# A cached row that fills the widest shared tiles of one size, one that fills the widest of all, and one between; a width
# whose vectors do not fill a wave; two streams.
_W = [layer(latent(4, 32, 16, 32, kv_rank=112, window=100, base=400000.0, scaling=(4.0, 256, 32.0, 1.0)), moe(16, 5, 64, groups=(4, 2), scale=1.25)),
      layer(latent(5, 48, 24, 56, kv_rank=200, window=70))]
_W += [again(_W, 0), layer(latent(2, 64, 32, 48, kv_rank=224, window=128, scaling=(16.0, 128, 16.0, 2.0)), moe(6, 2, 48, groups=(3, 1), scale=0.5))]
WIDE = config(_W, width=104, vocab=130, streams=2)
CONFIGS = {"MIXED": MIXED, "WIDE": WIDE}


def random_weights(cfg, seed):
    g = torch.Generator().manual_seed(seed)

    def normal(*shape, std=1.0):
        return torch.randn(*shape, generator=g) * std

    def uniform(*shape, lo=-1.0, hi=1.0):
        return torch.rand(*shape, generator=g) * (hi - lo) + lo

    W, S = cfg["width"], cfg["streams"]
    w = {"embed": normal(cfg["vocab"], W), "embed.norm": uniform(W, lo=0.5, hi=1.5), "final.norm": uniform(W, lo=0.5, hi=1.5),
         "head": normal(cfg["vocab"], W, std=2.0 * W ** -0.5)}
    for i, spec in enumerate(cfg["layers"]):
        if spec.get("weights_of") is not None:
            continue
        p = f"l{i}."
        m = spec["mixer"]
        H, d, dr, dv, r = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
        w[p + "norm1"] = uniform(W, lo=0.5, hi=1.5)
        w[p + "mix.q"] = normal(H * (d + dr), W, std=W ** -0.5)
        w[p + "mix.dkv"] = normal(r + dr, W, std=W ** -0.5)
        w[p + "mix.dkv.norm"] = uniform(r, lo=0.5, hi=2.0)
        w[p + "mix.uk"] = normal(H * d, r, std=r ** -0.5)
        w[p + "mix.uv"] = normal(H * dv, r, std=r ** -0.5)
        w[p + "mix.sink"] = uniform(H, lo=-1.0, hi=3.0)
        w[p + "mix.o"] = normal(W, H * dv, std=(H * dv) ** -0.5)
        subs = ["hc1."]
        mlp = spec.get("mlp")
        if mlp:
            subs.append("hc2.")
            E, F = mlp["router"]["experts"], mlp["expert"]["ff"]
            w[p + "norm2"] = uniform(W, lo=0.5, hi=1.5)
            w[p + "mlp.router"] = normal(E, W, std=2.0 * W ** -0.5)
            for e in range(E):
                w[p + f"mlp.e{e}.gate"] = normal(F, W, std=W ** -0.5)
                w[p + f"mlp.e{e}.up"] = normal(F, W, std=W ** -0.5)
                w[p + f"mlp.e{e}.down"] = normal(W, F, std=F ** -0.5)
        for s in subs:
            w[p + s + "in"] = uniform(S, lo=0.3, hi=1.2)
            # The experts write less than the attention: an expert chosen otherwise by the 16-bit engine, where two all but
            # tie, then moves a row less (in 32-bit every row is held to rounding anyway).
            w[p + s + "out"] = uniform(S, lo=0.4, hi=1.4) if s == "hc1." else uniform(S, lo=0.2, hi=0.5)
            w[p + s + "mix"] = torch.eye(S) * 0.9 + uniform(S, S, lo=-0.3, hi=0.3)
    # What the file stores is what both sides compute with.
    return {n: t.to(torch.bfloat16).contiguous() for n, t in w.items()}


def write_model(folder, cfg, weights):
    folder = Path(folder)
    folder.mkdir(parents=True, exist_ok=True)
    (folder / "config.json").write_text(json.dumps(cfg))
    save_file(weights, str(folder / "model.safetensors"))
    return folder
