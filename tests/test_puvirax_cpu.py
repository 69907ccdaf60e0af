"""The Puvirax architecture on the CPU: what the native library makes of its config.json, the rules it shares with every
host, the tokens that the cache manager remembers, and the plain implementation's own pieces against torch's routines and
equations written out."""
import json
import math
import subprocess

import numpy as np
import pytest
import torch

import plain_puvirax as plain
from puvirax_models import MIXED, config, dense, layer, moe, random_weights, rotated, unrotated, windowed, write_model
from vosti_amd.config import ConfigError, config_from_dict
from vosti_amd.kernels import build

F64 = torch.float64


def test_description_of_a_configuration():
    c = config_from_dict(MIXED)
    assert c.architecture == "Puvirax" and c.vocab == 97 and c.width == 64 and c.layers == 8 and c.logit_scale == 0.75 and c.bigram_buckets == 37
    spec = c.model_spec()
    assert [l.block for l in spec.layers] == ["prenorm"] * 8
    assert [l.feed_forward.kind for l in spec.layers] == ["squared_relu", "routed_experts", "squared_relu", "none", "none", "squared_relu", "routed_experts",
                                                          "routed_experts"]
    assert [(e.layer, e.cache_from) for e in spec.schedule] == [(i, None) for i in range(8)]
    assert spec.embedding.kind == "token_embedding_bigram"
    assert [spec.embedding.params[k] for k in ("buckets", "mul_prev", "mul_cur")] == [37, 5, 11]
    assert spec.final_norm.params == {"size": 64, "eps": 1e-5, "scale": 0.75}
    f = spec.layers[6].feed_forward.params
    assert (f["experts"], f["top"], f["intermediate_size"], f["score"], f["choice_correction"], f["groups"], f["keep_groups"], f["group_score"]) == (10, 3, 24, 1, 1, 5, 3, 1)
    assert not {"limit", "router_bias", "shared_size", "weigh_input", "gated", "weight_eps"} & set(f)
    assert spec.layers[7].feed_forward.params["shared_size"] == 56 and spec.layers[1].feed_forward.params["groups"] == 1
    n = spec.layers[7].names
    assert n["mixer.q_proj.weight"] == "l7.mix.q" and n["mixer.k_norm.weight"] == "l7.mix.k.norm" and n["mixer.distance_bias"] == "l7.mix.rel"
    assert n["mixer.value_share"] == "l7.mix.vmix" and n["feed_forward.router.correction"] == "l7.mlp.correction"
    assert n["feed_forward.experts.7.down_proj.weight"] == "l7.mlp.e7.down" and n["feed_forward.shared.up_proj.weight"] == "l7.mlp.shared.up"
    assert spec.layers[0].names["mixer.head_gate.weight"] == "l0.mix.g" and "norms.post_mixer.weight" not in spec.layers[3].names


def test_the_parts_in_the_library_s_own_words():
    from vosti_amd.config.registry import describe
    d = describe(MIXED)
    mixers = [d["layers"][i]["mixer"] for i in range(8)]
    assert all(m["kind"] == "attention" and m["numbers"]["exact_weights"] == 1 for m in mixers)
    # The first layer that mixes is the second of the model; those that do not, and that one, need no share.
    assert [m["numbers"]["value_mix"] for m in mixers] == [0, 1, 2, 0, 2, 0, 2, 2]
    assert d["ignored_names"] == ["l0.mix.vmix", "l1.mix.vmix", "l3.mix.vmix", "l3.norm2", "l4.norm2", "l5.mix.vmix"]
    r = mixers[0]["parts"]["position"]
    assert r["kind"] == "rotary_stretched" and [r["numbers"][k] for k in ("rotary_dim", "theta", "band_factor", "original", "band_low", "band_high")] == [8, 500, 3, 40, 1, 4]
    assert "band_factor" not in mixers[4]["parts"]["position"]["numbers"]
    assert (mixers[0]["numbers"]["unit_norm"], mixers[0]["numbers"]["head_gate"], mixers[0]["numbers"]["eps"]) == (1, 1, 1e-5)
    assert "window" not in mixers[0]["numbers"] and mixers[1]["numbers"]["window"] == 10 and "window" not in mixers[2]["numbers"]
    assert mixers[1]["numbers"]["bias_max"] == 9 and "whole_norm" not in mixers[1]["numbers"] and mixers[2]["numbers"]["whole_norm"] == 1
    assert mixers[1]["parts"]["q_norm"]["numbers"]["size"] == 20 and mixers[2]["parts"]["q_norm"]["numbers"]["size"] == 144 and mixers[2]["parts"]["k_norm"]["numbers"]["size"] == 8
    assert d["names"]["head.weight"] == d["names"]["embedding.weight"] == "embed" and d["names"]["embedding.bigram"] == "bigram"


@pytest.mark.parametrize("change, text", [
    (lambda c: c["layers"][5].update(type="serial"), "unknown mixer type"),
    (lambda c: c["layers"][5].pop("type"), "type"),
    (lambda c: c["layers"][5].pop("mixer"), "mixer"),
    (lambda c: c["layers"][3]["mixer"].update(heads=0), "heads"),
    (lambda c: c["layers"][1]["mixer"].update(kv_heads=3), "multiple"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=14), "dims"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7), "even"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(base=0), "base"),
    (lambda c: c["layers"][0]["mixer"].pop("rot"), "rot"),
    (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("low"), "low"),
    (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(factor=0), "factor"),
    (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(low=5.0), "low"),
    (lambda c: c["layers"][3]["mixer"].pop("scale"), "scale"),
    (lambda c: c["layers"][3]["mixer"].update(scale=0), "scale"),
    (lambda c: c["layers"][3]["mixer"]["mask"].update(size=0), "size"),
    (lambda c: c["layers"][3]["mixer"].pop("bias_max"), "bias_max"),
    (lambda c: c["layers"][2]["mixer"].update(bias_max=-1), "bias_max"),
    (lambda c: c["layers"][2]["mixer"].update(v_mix=1), "v_mix"),
    (lambda c: c["layers"][2]["mixer"].update(vdim=20), "blended"),
    (lambda c: c["layers"][6]["mlp"]["router"].update(top=7), "kept groups"),
    (lambda c: c["layers"][6]["mlp"]["router"]["groups"].update(count=3), "divide"),
    (lambda c: c["layers"][6]["mlp"]["router"]["groups"].update(keep=6), "keep"),
    (lambda c: c["layers"][6]["mlp"].update(kind="serial"), "moe"),
    (lambda c: c["layers"][6]["mlp"]["expert"].pop("ff"), "ff"),
    (lambda c: c["layers"][7]["mlp"]["shared"].pop("ff"), "ff"),
    (lambda c: c["embedding"]["bigram"].update(buckets=0), "buckets"),
    (lambda c: c["embedding"]["bigram"].update(mul_prev=-3), "mul_prev"),
    (lambda c: c["embedding"]["bigram"].pop("mul_cur"), "mul_cur"),
    (lambda c: c.pop("norm"), "norm"),
])
def test_configuration_errors_name_the_key(change, text):
    cfg = json.loads(json.dumps(MIXED))
    change(cfg)
    with pytest.raises(ConfigError, match=text):
        config_from_dict(cfg)


def test_tensor_names_are_the_files(tmp_path):
    """The program's own description of a model folder lists the tensors that such a file holds, but for the shares that no
    layer uses."""
    w = random_weights(MIXED, 1)
    folder = write_model(tmp_path / "m", MIXED, w)
    program = str(build.ensure("engine", verbose=False))
    r = subprocess.run([program, "--kind", "describe", "--model-path", str(folder)], capture_output=True, text=True)
    assert r.returncode == 0, r.stderr
    got = json.loads(r.stdout)
    assert got["architecture"] == "Puvirax"
    assert got["tensor_names"] == sorted(set(w) - {"l1.mix.vmix"})


def test_the_banded_frequencies_are_the_plain_ones():
    from vosti_amd.cache.host import rotary_banded_frequencies
    for m in (rotated(1, 1, 64, 8, dims=48, base=10000.0, scaling=(8.0, 64, 1.0, 4.0)), rotated(1, 1, 32, 8, dims=32, base=77.0, scaling=(2.5, 300, 0.5, 8.0)),
              rotated(1, 1, 32, 8, dims=20, base=500.0, scaling=(3.0, 60, 2.0, 2.0))):
        rot = m[1]["rot"]
        got = rotary_banded_frequencies(rot["base"], rot["dims"], **rot["scaling"])
        assert np.allclose(got, plain.frequencies(rot).numpy(), rtol=1e-7, atol=0)


def test_the_distance_classes_are_the_plain_ones():
    from vosti_amd.cache.host import distance_class
    for rows, far in ((16, 150), (32, 128), (11, 300), (6, 25), (2, 20), (3, 9.5), (7, 4)):
        assert [distance_class(n, rows, far) for n in range(700)] == [plain.distance_class(n, rows, far) for n in range(700)]


def test_the_cache_manager_remembers_a_request_s_tokens():
    """What a step needs of the token before its first one: none at a request's start, the last committed one later, none of an
    abandoned step's, and those that a matched prefix brought along."""
    from vosti_amd.cache.manager import CacheManager, GroupSpec
    m = CacheManager(8, [GroupSpec(0, 8)], 2, prefix_cache=True)
    m.add_request(1)
    assert m.token(1, -1) == -1 and m.token(1, 0) == -1
    m.extend(1, [3, 4, 5])
    m.abort_step(1)
    assert m.token(1, 0) == -1
    m.extend(1, list(range(10, 18)))
    m.commit(1)
    m.extend(1, [30])
    assert [m.token(1, i) for i in (0, 7, 8, 9)] == [10, 17, 30, -1]
    assert m.add_request(2, list(range(10, 18)) + [9, 9]) == 8 and m.token(2, 7) == 17 and m.token(2, 8) == -1
    m.finish(1)
    assert m.token(1, 0) == -1


# ------------------------------------------------------------------------- the plain implementation's own pieces
def test_norms_against_torch():
    x = torch.randn(5, 12, dtype=F64, generator=torch.Generator().manual_seed(0))
    w = torch.randn(12, dtype=F64, generator=torch.Generator().manual_seed(1))
    assert torch.allclose(plain.norm(x, w, 1e-5), torch.nn.functional.rms_norm(x, (12,), eps=1e-5) * w, atol=1e-12)
    assert torch.allclose(plain.rms(x, 1e-5), torch.nn.functional.rms_norm(x, (12,), eps=1e-5), atol=1e-12)
    assert torch.equal(plain.squared_relu(torch.tensor([-2.0, 0.0, 3.0])), torch.tensor([0.0, 0.0, 9.0]))


def test_rows_of_pairs():
    b = {"buckets": 10, "mul_prev": 3, "mul_cur": 17}
    assert plain.bigram_rows(b, [4, 9, 9, 0]) == [10, (3 * 4 + 17 * 9) % 10, (3 * 9 + 17 * 9) % 10, (3 * 9) % 10]


def test_bands_written_out():
    """Three bands: a short wavelength, one between, a long one."""
    rot = {"base": 10000.0, "dims": 16, "scaling": {"factor": 4.0, "original": 200, "low": 1.0, "high": 4.0}}
    f = plain.frequencies(rot)
    whole = [10000.0 ** (-2 * i / 16) for i in range(8)]
    lengths = [2 * math.pi / x for x in whole]
    kinds = []
    for i in range(8):
        if lengths[i] < 50:
            want, kind = whole[i], "kept"
        elif lengths[i] > 200:
            want, kind = whole[i] / 4, "divided"
        else:
            s = (200 / lengths[i] - 1) / 3
            want, kind = (1 - s) * whole[i] / 4 + s * whole[i], "between"
        kinds.append(kind)
        assert math.isclose(float(f[i]), want, rel_tol=1e-12)
    assert kinds[:3] == ["kept", "kept", "between"] and set(kinds) == {"kept", "between", "divided"}
    x = torch.randn(5, 2, 20, dtype=F64, generator=torch.Generator().manual_seed(0))
    y = plain.rotate(x, rot)
    a = 3 * float(f[2])
    assert torch.allclose(y[3, :, 2], x[3, :, 2] * math.cos(a) - x[3, :, 10] * math.sin(a))
    assert torch.allclose(y[3, :, 10], x[3, :, 10] * math.cos(a) + x[3, :, 2] * math.sin(a))
    assert torch.equal(y[..., 16:], x[..., 16:]) and torch.equal(y[0], x[0])


def test_distance_classes_written_out():
    """Eight classes up to 32: four of one distance each, then four whose borders are 4, 4 * 8^(1/4), 4 * 8^(1/2), ..."""
    got = [plain.distance_class(n, 8, 32) for n in range(60)]
    assert got[:4] == [0, 1, 2, 3]
    borders = [4 * 8 ** (k / 4) for k in range(4)]
    for n in range(4, 60):
        assert got[n] == 4 + sum(n >= b for b in borders) - 1, n
    assert got[32:] == [7] * 28 and plain.distance_class(5, 3, 40) == 1 + math.floor(math.log(5) / math.log(40) * 2)


def test_a_window_is_the_last_keys():
    see = plain.visible(6, 3)
    assert [[j for j in range(6) if see[i, j]] for i in range(6)] == [[0], [0, 1], [0, 1, 2], [1, 2, 3], [2, 3, 4], [3, 4, 5]]
    assert torch.equal(plain.visible(4, 1), torch.eye(4, dtype=torch.bool)) and torch.equal(plain.visible(4), torch.ones(4, 4).tril().bool())


@pytest.mark.parametrize("kind", ["rotated", "windowed", "unrotated"])
def test_attention_written_out(kind):
    """Row by row and head by head, with values blended with another layer's."""
    mixer = {"rotated": rotated(4, 2, 6, 4, dims=4, base=50.0, scaling=(2.0, 16, 1.0, 4.0)), "windowed": windowed(4, 2, 6, 4, window=3, far=9),
             "unrotated": unrotated(4, 2, 6, 4, far=9)}[kind]
    cfg = config([layer(mixer)], width=8, vocab=10)
    w = {n: t.double() for n, t in random_weights(cfg, 2, classes=6).items()}
    w["l0.mix.vmix"] = torch.tensor(0.375, dtype=F64)
    m, p, eps = mixer[1], "l0.mix.", 1e-3
    h, v0 = torch.randn(7, 8, dtype=F64, generator=torch.Generator().manual_seed(1)), torch.randn(7, 8, dtype=F64, generator=torch.Generator().manual_seed(2))
    got = plain.attention(mixer[0], m, w, p, h, eps, {"v": v0})
    q, k, v = ((h @ w[p + n].T) for n in ("q", "k", "v"))
    v = 0.625 * v + 0.375 * v0
    length = lambda x: math.sqrt(float((x * x).mean()) + eps)
    qs, ks = torch.zeros(7, 4, 6, dtype=F64), torch.zeros(7, 2, 6, dtype=F64)
    for src, dst, name in ((q, qs, "q"), (k, ks, "k")):
        for i in range(7):
            for head in range(dst.shape[1]):
                x = src[i, head * 6:head * 6 + 6].clone()
                if kind == "windowed":
                    x = x / length(x) * w[p + name + ".norm"]
                elif kind == "unrotated":
                    x = x / length(src[i]) * w[p + name + ".norm"][head * 6:head * 6 + 6]
                else:
                    f = plain.frequencies(m["rot"])
                    for c in range(2):
                        a, b, t = x[c].item(), x[c + 2].item(), i * float(f[c])
                        x[c], x[c + 2] = a * math.cos(t) - b * math.sin(t), b * math.cos(t) + a * math.sin(t)
                    x = x / length(x)
                dst[i, head] = x
    out = torch.zeros(7, 4, 4, dtype=F64)
    for head in range(4):
        for i in range(7):
            js = list(range(max(0, i - 2) if kind == "windowed" else 0, i + 1))
            s = torch.tensor([float(qs[i, head] @ ks[j, head // 2]) * m["scale"] +
                              (0.0 if kind == "rotated" else float(w[p + "rel"][plain.distance_class(i - j, 6, 9), head])) for j in js], dtype=F64)
            e = torch.exp(s)
            out[i, head] = (e / e.sum()) @ v[js][:, head // 2 * 4:head // 2 * 4 + 4]
            if kind == "rotated":
                out[i, head] /= 1 + math.exp(-float(w[p + "g"][head] @ h[i]))
    assert torch.allclose(got, out.reshape(7, 16) @ w[p + "o"].T, atol=1e-12)


def test_the_first_layer_that_mixes_keeps_its_values():
    """Three layers of which the second and third mix: the third blends with the second's, and the second's own share is not used."""
    cfg = config([layer(windowed(2, 1, 8, 8, 4, 9, mix=False)), layer(rotated(2, 2, 8, 4, dims=4)), layer(unrotated(1, 1, 8, 8, 9))], width=16, vocab=10)
    w = random_weights(cfg, 2)
    tokens = [1, 5, 2, 2, 7]
    want = plain.forward(cfg, w, tokens)
    assert torch.equal(plain.forward(cfg, dict(w, **{"l1.mix.vmix": torch.tensor(0.0)}), tokens), want)
    assert not torch.allclose(plain.forward(cfg, dict(w, **{"l2.mix.vmix": torch.tensor(0.0)}), tokens), want, atol=1e-3)
    assert "l0.mix.vmix" not in w


def test_routing_by_groups_with_corrected_scores():
    mlp, p = moe(8, 3, 6, groups=(4, 2), shared=10), "l0.mlp."
    cfg = config([layer(windowed(1, 1, 4, 4, 4, 9), mlp)], width=8, vocab=10)
    w = {n: t.double() for n, t in random_weights(cfg, 2).items()}
    w[p + "correction"] = torch.tensor([-1.0, 0.3, -0.2, -0.9, 0.1, -1.2, 0.4, -0.5], dtype=F64)
    h = torch.randn(40, 8, dtype=F64, generator=torch.Generator().manual_seed(3)) * 2
    idx, wt = plain.route(mlp["router"], w, p, h)
    got = plain.experts(mlp, w, p, h)
    other_groups = uncorrected = negative = 0
    for t in range(40):
        s = 1 / (1 + torch.exp(-(w[p + "router"] @ h[t])))
        c = s + w[p + "correction"]
        kept = sorted(range(4), key=lambda g: -float(c[2 * g] + c[2 * g + 1]))[:2]
        order = sorted([e for g in kept for e in (2 * g, 2 * g + 1)], key=lambda e: -float(c[e]))[:3]
        assert idx[t].tolist() == order and torch.allclose(wt[t], s[order])
        other_groups += set(kept) != set(sorted(range(4), key=lambda g: -float(max(c[2 * g], c[2 * g + 1])))[:2])
        uncorrected += set(order) != set(torch.argsort(s, descending=True)[:3].tolist())
        negative += float(c[order].min()) < 0
        ff = lambda name: w[p + name + ".down"] @ torch.relu(w[p + name + ".up"] @ h[t]) ** 2
        want = ff("shared")
        for e in order:
            want = want + s[e] * ff(f"e{e}")
        assert torch.allclose(got[t], want, atol=1e-12)
    assert other_groups > 3 and uncorrected > 3 and negative > 3


def test_the_order_of_a_layer_and_the_end():
    cfg = config([layer(windowed(2, 1, 8, 8, 4, 9), dense(12)), layer(rotated(2, 2, 8, 4, dims=4))], width=16, vocab=10, logit_scale=2.5)
    w = {n: t.double() for n, t in random_weights(cfg, 2).items()}
    tokens = [1, 2, 3, 1]
    sums = []
    logits = plain.forward(cfg, w, tokens, sums)
    x = torch.stack([w["embed"][t] + w["bigram"][r] for t, r in zip(tokens, plain.bigram_rows(cfg["embedding"]["bigram"], tokens))])
    first = {}
    x = x + plain.attention("attention_2", cfg["layers"][0]["mixer"], w, "l0.mix.", plain.norm(x, w["l0.norm1"], 1e-5), 1e-5, first)
    x = x + torch.relu(plain.norm(x, w["l0.norm2"], 1e-5) @ w["l0.mlp.up"].T) ** 2 @ w["l0.mlp.down"].T
    assert torch.allclose(sums[0], x, atol=1e-12) and len(sums) == 2
    x = x + plain.attention("attention", cfg["layers"][1]["mixer"], w, "l1.mix.", plain.norm(x, w["l1.norm1"], 1e-5), 1e-5, first)
    assert torch.allclose(logits, 2.5 * plain.norm(x, w["final.norm"], 1e-5) @ w["embed"].T, atol=1e-12)
