"""The Kelisun architecture on the CPU: what the native library makes of its config.json, and the plain implementation's
own pieces against torch's routines and equations written out."""
import json
import math
import subprocess

import numpy as np
import pytest
import torch

import plain_kelisun as plain
from kelisun_models import MIXED, again, config, latent, layer, moe, random_weights, write_model
from vosti_amd.config import ConfigError, config_from_dict
from vosti_amd.kernels import build

F64 = torch.float64


def test_description_of_a_configuration():
    c = config_from_dict(MIXED)
    assert c.architecture == "Kelisun" and c.vocab == 97 and c.width == 64 and c.layers == 8 and c.streams == 3
    spec = c.model_spec()
    # Five layers with weights of their own, run eight times, every run with a cache of its own.
    assert [l.block for l in spec.layers] == ["hyper_streams"] * 5
    assert [l.feed_forward.kind for l in spec.layers] == ["routed_experts", "routed_experts", "none", "routed_experts", "routed_experts"]
    assert [(e.layer, e.cache_from) for e in spec.schedule] == [(0, None), (2, None), (0, None), (1, None), (1, None), (2, None), (3, None), (4, None)]
    assert spec.embedding.kind == "token_embedding_normed" and spec.embedding.params["eps"] == 1e-5
    assert spec.final_norm.params == {"size": 64, "eps": 1e-5} and "softcap" not in spec.head.params
    f = spec.layers[3].feed_forward.params
    assert (f["experts"], f["top"], f["intermediate_size"], f["gated"], f["score"], f["groups"], f["keep_groups"], f["weight_scale"]) == (10, 3, 24, 1, 2, 5, 3, 2.5)
    assert not {"limit", "router_bias", "shared_size", "weigh_input", "up_shift", "glu_slope"} & set(f)
    assert (spec.layers[0].feed_forward.params["groups"], spec.layers[0].feed_forward.params["keep_groups"]) == (1, 1)
    n = spec.layers[4].names
    assert n["mixer.q_proj.weight"] == "l7.mix.q" and n["mixer.kv_down_norm.weight"] == "l7.mix.dkv.norm" and n["mixer.sinks"] == "l7.mix.sink"
    assert n["norms.mixer_in.weight"] == "l7.norm1" and n["norms.ffn_in.weight"] == "l7.norm2"
    assert n["hyper_mixer.in"] == "l7.hc1.in" and n["hyper_ffn.mix"] == "l7.hc2.mix" and n["feed_forward.experts.7.down_proj.weight"] == "l7.mlp.e7.down"
    assert "norms.ffn_in.weight" not in spec.layers[2].names and "hyper_ffn.in" not in spec.layers[2].names


def test_the_parts_in_the_library_s_own_words():
    from vosti_amd.config.registry import describe
    d = describe(MIXED)
    a = d["layers"][0]["mixer"]
    n = a["numbers"]
    assert a["kind"] == "latent_attention"
    assert (n["num_heads"], n["head_dim"], n["rotary_dim"], n["value_dim"], n["kv_rank"], n["q_rank"], n["window"], n["sink"]) == (3, 12, 6, 20, 20, 0, 10, 1)
    assert "output_gate" not in n
    r = a["parts"]["position"]
    assert r["kind"] == "rotary_stretched" and "neighbours" not in r["numbers"]
    assert [r["numbers"][k] for k in ("rotary_dim", "theta", "factor", "original", "fast", "slow")] == [6, 500, 3, 40, 8, 0.5]
    plain_rot = d["layers"][1]["mixer"]["parts"]["position"]["numbers"]
    assert plain_rot["theta"] == 77 and "factor" not in plain_rot
    assert d["layers"][0]["block_numbers"] == {"hidden_size": 64, "streams": 3}
    assert d["ignored_names"] == ["l5.norm2", "l5.hc2.in", "l5.hc2.out", "l5.hc2.mix"]
    assert d["names"]["embedding.norm.weight"] == "embed.norm" and d["names"]["head.weight"] == "head"
    # A layer without a mask sees every earlier key.
    free = json.loads(json.dumps(MIXED))
    for i in (3, 4):
        del free["layers"][i]["mixer"]["mask"]
    assert describe(free)["layers"][1]["mixer"]["numbers"]["window"] == 0


@pytest.mark.parametrize("change, text", [
    (lambda c: c["layers"][5].update(type="serial"), "unknown mixer type"),
    (lambda c: c["layers"][5].pop("type"), "type"),
    (lambda c: c["layers"][5].pop("mixer"), "mixer"),
    (lambda c: c["layers"][3]["mixer"].update(heads=0), "heads"),
    (lambda c: c["layers"][3]["mixer"]["rot"].update(dims=8), "rot_dim"),
    (lambda c: c["layers"][3]["mixer"].update(rot_dim=5, rot={"base": 10.0, "dims": 5}), "even"),
    (lambda c: c["layers"][3]["mixer"]["rot"].update(base=1.0), "base"),
    (lambda c: c["layers"][3]["mixer"].pop("scale"), "scale"),
    (lambda c: c["layers"][3]["mixer"].pop("rot"), "rot"),
    (lambda c: c["layers"][3]["mixer"]["mask"].update(size=0), "size"),
    (lambda c: c["layers"][7]["mixer"]["rot"]["scaling"].pop("slow"), "slow"),
    (lambda c: c["layers"][7]["mixer"]["rot"]["scaling"].update(factor=0), "factor"),
    (lambda c: c["layers"][7]["mlp"]["router"].update(top=5), "kept groups"),
    (lambda c: c["layers"][7]["mlp"]["router"]["groups"].update(count=3), "divide"),
    (lambda c: c["layers"][7]["mlp"]["router"]["groups"].update(keep=3), "keep"),
    (lambda c: c["layers"][3]["mlp"].update(kind="dense"), "moe"),
    (lambda c: c["layers"][3]["mlp"]["expert"].pop("ff"), "ff"),
    (lambda c: c["layers"][2].update(weights_of=2), "weights_of"),
    (lambda c: c["layers"][2].update(weights_of=8), "weights_of"),
    (lambda c: c["layers"][2].update(weights_of=1), "differs"),
    (lambda c: c["layers"][2]["mixer"].update(scale=0.7), "differs"),
    (lambda c: c["layers"][2].update(mlp=None), "differs"),
    (lambda c: c.pop("streams"), "streams"),
    (lambda c: c.pop("norm"), "norm"),
])
def test_configuration_errors_name_the_key(change, text):
    cfg = json.loads(json.dumps(MIXED))
    change(cfg)
    with pytest.raises(ConfigError, match=text):
        config_from_dict(cfg)


def test_a_layer_may_use_the_weights_of_one_that_uses_another_s():
    layers = [layer(latent(1, 8, 4, 8, kv_rank=8, window=5))]
    layers += [again(layers, 0)]
    layers += [again(layers, 1)]
    spec = config_from_dict(config(layers)).model_spec()
    assert [e.layer for e in spec.schedule] == [0, 0, 0] and len(spec.layers) == 1
    layers[0]["weights_of"] = 2
    with pytest.raises(ConfigError, match="weights_of"):
        config_from_dict(config(layers))


def test_tensor_names_are_the_files(tmp_path):
    """The program's own description of a model folder lists exactly the tensors that such a file holds."""
    w = random_weights(MIXED, 1)
    folder = write_model(tmp_path / "m", MIXED, w)
    program = str(build.ensure("engine", verbose=False))
    r = subprocess.run([program, "--kind", "describe", "--model-path", str(folder)], capture_output=True, text=True)
    assert r.returncode == 0, r.stderr
    got = json.loads(r.stdout)
    assert got["architecture"] == "Kelisun"
    assert got["tensor_names"] == sorted(w)


def test_the_rotation_frequencies_are_the_plain_ones():
    from vosti_amd.cache.host import rotary_stretched_frequencies
    for rot in (latent(1, 8, 16, 8, 8, 4, base=10000.0, scaling=(4.0, 64, 16.0, 1.0))["rot"], latent(1, 8, 40, 8, 8, 4, base=77.0, scaling=(2.5, 300, 8.0, 0.5))["rot"],
                latent(1, 8, 6, 8, 8, 4, base=500.0)["rot"]):
        f, mag = plain.frequencies(rot)
        got, got_mag = rotary_stretched_frequencies(rot["base"], rot["dims"], **rot.get("scaling", {}))
        assert np.allclose(got, f.numpy(), rtol=1e-7, atol=0) and abs(got_mag - mag) < 1e-6


# ------------------------------------------------------------------------- the plain implementation's own pieces
def test_norm_and_silu_against_torch():
    x = torch.randn(5, 12, dtype=F64, generator=torch.Generator().manual_seed(0))
    w = torch.randn(12, dtype=F64, generator=torch.Generator().manual_seed(1))
    assert torch.allclose(plain.norm(x, w, 1e-5), torch.nn.functional.rms_norm(x, (12,), eps=1e-5) * w, atol=1e-12)
    assert torch.allclose(plain.silu(x), torch.nn.functional.silu(x), atol=1e-12)


def test_stretched_rotation_written_out():
    """A ramp with a first, a middle and a last part: short wavelengths keep their frequency, long ones are divided."""
    rot = {"base": 10000.0, "dims": 16, "scaling": {"factor": 4.0, "original": 64, "fast": 4.0, "slow": 0.5}}
    f, mag = plain.frequencies(rot)
    whole = [10000.0 ** (-2 * i / 16) for i in range(8)]
    at = lambda t: 16 * math.log(64 / (2 * math.pi * t)) / (2 * math.log(10000.0))
    lo, hi = math.floor(at(4.0)), math.ceil(at(0.5))
    assert (lo, hi) == (0, 3)
    for i in range(8):
        ramp = min(max((i - lo) / (hi - lo), 0.0), 1.0)
        assert math.isclose(float(f[i]), whole[i] * (1 - ramp) + whole[i] / 4.0 * ramp, rel_tol=1e-12)
    assert float(f[0]) == whole[0] and math.isclose(float(f[7]), whole[7] / 4)
    assert math.isclose(mag, 0.1 * math.log(4.0) + 1.0)
    x = torch.randn(5, 2, 16, dtype=F64, generator=torch.Generator().manual_seed(0))
    y = plain.rotate_halves(x, torch.arange(5), rot)
    a = 3 * float(f[2])
    assert torch.allclose(y[3, :, 2], (x[3, :, 2] * math.cos(a) - x[3, :, 10] * math.sin(a)) * mag)
    assert torch.allclose(y[3, :, 10], (x[3, :, 10] * math.cos(a) + x[3, :, 2] * math.sin(a)) * mag)
    assert torch.allclose(y[0], x[0] * mag)
    plain_rot = {"base": 10000.0, "dims": 16}
    assert plain.frequencies(plain_rot)[1] == 1.0 and torch.allclose(plain.frequencies(plain_rot)[0], torch.tensor(whole, dtype=F64))


def test_a_window_is_the_last_keys():
    see = plain.visible(6, 3)
    assert [[j for j in range(6) if see[i, j]] for i in range(6)] == [[0], [0, 1], [0, 1, 2], [1, 2, 3], [2, 3, 4], [3, 4, 5]]
    assert torch.equal(plain.visible(4, 1), torch.eye(4, dtype=torch.bool))


def one_layer(mixer, mlp=None, width=8, streams=2):
    cfg = config([layer(mixer, mlp)], width=width, vocab=10, streams=streams)
    return cfg, {n: t.double() for n, t in random_weights(cfg, 2).items()}


def test_latent_attention_written_out_over_the_cached_row():
    """The scores and outputs from the cached row alone: (W_uk^T q_flat) . c + q_rot . k_rot and W_uv (sum p c), with the sink
    as one more entry of the softmax that carries nothing."""
    cfg, w = one_layer(latent(2, 4, 2, 6, kv_rank=5, window=3, base=50.0, scaling=(2.0, 16, 2.0, 0.25)))
    m, p = cfg["layers"][0]["mixer"], "l0.mix."
    h = torch.randn(7, 8, dtype=F64, generator=torch.Generator().manual_seed(1))
    got = plain.latent_attention(m, w, p, h, 1e-5)
    down = h @ w[p + "dkv"].T
    c = down[:, :5] / torch.sqrt((down[:, :5] ** 2).mean(-1, keepdim=True) + 1e-5) * w[p + "dkv.norm"]
    turn = lambda x, i: plain.rotate_halves(x[None, None], torch.tensor([i]), m["rot"])[0, 0]
    shared = torch.stack([turn(down[i, 5:], i) for i in range(7)])
    q = (h @ w[p + "q"].T).view(7, 2, 6)
    out = torch.zeros(7, 2, 6, dtype=F64)
    for head in range(2):
        uk, uv = w[p + "uk"][head * 4:(head + 1) * 4], w[p + "uv"][head * 6:(head + 1) * 6]
        for i in range(7):
            j = list(range(max(0, i - 2), i + 1))
            s = (c[j] @ (uk.T @ q[i, head, :4]) + shared[j] @ turn(q[i, head, 4:], i)) * m["scale"]
            weights = torch.softmax(torch.cat([s, w[p + "sink"][head:head + 1]]), 0)[:-1]
            out[i, head] = uv @ (weights @ c[j])
    assert torch.allclose(got, out.reshape(7, 12) @ w[p + "o"].T, atol=1e-12)
    # The factor on cosine and sine stays off the part that is not rotated: with that part alone it changes nothing.
    flat = dict(w)
    flat[p + "q"] = w[p + "q"].clone().view(2, 6, 8)
    flat[p + "q"][:, 4:] = 0
    flat[p + "q"] = flat[p + "q"].view(12, 8)
    bare = json.loads(json.dumps(m))
    del bare["rot"]["scaling"]
    assert torch.allclose(plain.latent_attention(m, flat, p, h, 1e-5), plain.latent_attention(bare, flat, p, h, 1e-5), atol=1e-12)
    assert not torch.allclose(got, plain.latent_attention(bare, w, p, h, 1e-5), atol=1e-3)


def test_routing_by_groups_keeps_the_softmax_over_all():
    cfg, w = one_layer(latent(1, 2, 2, 2, kv_rank=4, window=4), moe(8, 3, 6, groups=(4, 2), scale=2.5))
    mlp, p = cfg["layers"][0]["mlp"], "l0.mlp."
    h = torch.randn(40, 8, dtype=F64, generator=torch.Generator().manual_seed(3)) * 2
    idx, wt = plain.route(mlp["router"], w, p, h)
    z = h @ w[p + "router"].T
    got = plain.experts(mlp, w, p, h)
    differs = 0
    for t in range(40):
        s = torch.exp(z[t]) / torch.exp(z[t]).sum()
        kept = sorted(range(4), key=lambda g: -float(max(s[2 * g], s[2 * g + 1])))[:2]
        order = sorted([e for g in kept for e in (2 * g, 2 * g + 1)], key=lambda e: -float(s[e]))[:3]
        assert idx[t].tolist() == order and torch.allclose(wt[t], 2.5 * s[order])
        differs += set(order) != set(torch.argsort(s, descending=True)[:3].tolist())
        want = torch.zeros(8, dtype=F64)
        for e in order:
            g = w[p + f"e{e}.gate"] @ h[t]
            want += 2.5 * s[e] * (w[p + f"e{e}.down"] @ (g / (1 + torch.exp(-g)) * (w[p + f"e{e}.up"] @ h[t])))
        assert torch.allclose(got[t], want, atol=1e-12)
    assert differs > 3                                   # the groups do change the choice here
    assert float((wt / 2.5).sum(1).min()) < 0.95         # and the chosen scores are not divided by their sum


def test_streams_and_the_order_of_a_layer():
    """A layer of three streams written out one stream after the other; both sublayers see a mixture of all streams."""
    cfg, w = one_layer(latent(1, 4, 2, 6, kv_rank=5, window=3), moe(2, 1, 6), streams=3)
    layers = cfg["layers"] + [dict(cfg["layers"][0], weights_of=0)]
    cfg = dict(cfg, layers=layers)
    tokens = [1, 2, 3, 1]
    sums = []
    logits = plain.forward(cfg, w, tokens, sums)
    x = w["embed"][torch.tensor(tokens)]
    x = x / torch.sqrt((x * x).mean(-1, keepdim=True) + 1e-5) * w["embed.norm"]
    xs = [x, x, x]
    for _ in range(2):
        for sub, fn, norm in (("hc1", lambda h: plain.latent_attention(layers[0]["mixer"], w, "l0.mix.", h, 1e-5), "norm1"),
                              ("hc2", lambda h: plain.experts(layers[0]["mlp"], w, "l0.mlp.", h), "norm2")):
            a, b, M = (w[f"l0.{sub}.{n}"] for n in ("in", "out", "mix"))
            u = a[0] * xs[0] + a[1] * xs[1] + a[2] * xs[2]
            y = fn(plain.norm(u, w[f"l0.{norm}"], 1e-5))
            xs = [M[0, t] * xs[0] + M[1, t] * xs[1] + M[2, t] * xs[2] + b[t] * y for t in range(3)]
    total = xs[0] + xs[1] + xs[2]
    assert torch.allclose(sums[1], total, atol=1e-10) and len(sums) == 2
    assert torch.allclose(logits, plain.norm(total, w["final.norm"], 1e-5) @ w["head"].T, atol=1e-10)
    turned = {n: (t.T.contiguous() if n.endswith(".mix") else t) for n, t in w.items()}
    assert not torch.allclose(plain.forward(cfg, turned, tokens), logits, atol=1e-3)      # [from, to], not [to, from]
