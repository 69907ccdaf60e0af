"""The Puvirax decoder through the native engine against the plain implementation (tests/plain_puvirax.py).

Every test builds its own small model.  The engine is driven through its step function (given tokens in, logits out:
what bin/trace_run drives) and through its scheduler (``generate``).  In float32 the engine must agree with the plain
float64 implementation to a few units of 32-bit rounding; in bfloat16 to what rounding the matrix products to 16 bits
costs.  Two cuttings of the same tokens through the engine must agree far closer than either does with the plain
implementation: nothing may depend on portions, batches, pages or slots."""
import copy
import json

import numpy as np
import pytest
import torch

import plain_puvirax as plain
from puvirax_models import CONFIGS, config, dense, layer, moe, random_weights, rotated, unrotated, windowed, write_model

pytestmark = pytest.mark.gpu

TOLERANCE = {"float32": 2e-4, "bfloat16": 6e-2}      # of the logits' root mean square
SAME = {"float32": 2e-5, "bfloat16": 2e-5}           # two cuttings of the same tokens through the engine
DTYPES = pytest.mark.parametrize("dtype", ["float32", "bfloat16"])


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    out = {}
    for seed, (name, cfg) in enumerate(CONFIGS.items()):
        w = random_weights(cfg, 20 + seed)
        out[name] = (write_model(tmp_path_factory.mktemp(name), cfg, w), cfg, w)
    return out


def engine(folder, dtype, num_pages=24, page_size=16, max_num_seqs=4, **kw):
    from vosti_amd.engine.native import NativeEngine
    return NativeEngine(folder, dtype=dtype, num_pages=num_pages, page_size=page_size, max_num_seqs=max_num_seqs,
                        enable_prefix_cache=False, graphs=kw.pop("graphs", False), **kw)


def tokens_for(cfg, n, seed):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def run_cut(eng, rid, tokens, cuts, finish=True):
    """All logits of one request fed in portions of the given sizes."""
    rows, at = [], 0
    for c in cuts:
        rows.append(eng.trace_step([(rid, tokens[at:at + c], list(range(c)))]))
        at += c
    assert at == len(tokens)
    if finish:
        eng.trace_finish(rid)
    return np.concatenate(rows, 0)


def deviation(got, want):
    """Largest row deviation as a fraction of the logits' root mean square."""
    want = np.asarray(want, dtype=np.float64)
    return float(np.sqrt(((got - want) ** 2).mean(-1)).max() / np.sqrt((want ** 2).mean()))


def close(got, want, dtype):
    """Whether the engine's rows are the plain implementation's.  In float32 every row, to a few units of rounding.  In
    bfloat16 the router sees a rounded input, and where two experts' logits all but tie it may choose the other one: nine
    rows in ten must lie within what rounding costs, and none may be far off."""
    want = np.asarray(want, dtype=np.float64)
    rows = np.sqrt(((got - want) ** 2).mean(-1)) / np.sqrt((want ** 2).mean())
    if dtype == "float32":
        return bool(rows.max() < TOLERANCE[dtype])
    return bool(np.quantile(rows, 0.9) < TOLERANCE[dtype] and rows.max() < 0.5)


def plain_logits(cfg, w, tokens):
    return plain.forward(cfg, w, tokens).numpy()


# ------------------------------------------------------------------------------------------ each mechanism alone
SMALL = windowed(1, 1, 8, 8, window=6, far=9)        # a small mixer under what is tested
KW = dict(width=32, vocab=50)


def two(mixer, mlp=None, **kw):
    """The layer twice, so that the second's keys depend on the first's outputs (and, where it mixes, its values on them)."""
    return config([layer(mixer, mlp), layer(mixer, mlp)], **{**KW, **kw})


ALONE = {
    "rotated": two(rotated(4, 2, 16, 16, dims=16)),
    "rotated_partly_banded": two(rotated(4, 2, 20, 12, dims=12, base=300.0, scaling=(4.0, 30, 1.0, 4.0))),
    "rotated_band_without_a_middle": two(rotated(2, 1, 24, 8, dims=24, base=90.0, scaling=(2.5, 30, 2.0, 2.0))),
    "rotated_two_entries": two(rotated(3, 3, 10, 10, dims=2, base=7.0, mix=False)),
    "rotated_one_head_wide": two(rotated(1, 1, 256, 40, dims=200, scale=0.03)),
    "rotated_twenty_heads_on_one": two(rotated(20, 1, 8, 16, dims=4)),
    "rotated_of_64": two(rotated(4, 2, 64, 64, dims=64, mix=False)),
    "rotated_of_128": two(rotated(4, 1, 128, 128, dims=32)),
    "windowed": two(windowed(4, 2, 16, 16, window=9, far=20)),
    "windowed_odd_sizes": two(windowed(5, 5, 10, 12, window=7, far=11)),
    "windowed_values_wider": two(windowed(6, 3, 8, 40, window=25, far=12)),
    "windowed_of_64_without_mixing": two(windowed(4, 2, 64, 64, window=21, far=10, mix=False)),
    "windowed_of_128": two(windowed(4, 4, 128, 96, window=30, far=1000)),
    "windowed_of_256": two(windowed(2, 1, 256, 256, window=30, far=18)),
    "windowed_of_200": two(windowed(2, 1, 200, 8, window=33, far=18)),
    "window_of_one": two(windowed(2, 1, 8, 8, window=1, far=9)),
    "window_of_two": two(windowed(2, 1, 8, 8, window=2, far=9)),
    "window_of_a_page": two(windowed(2, 1, 8, 8, window=16, far=9)),
    "window_longer_than_the_sequence": two(windowed(2, 1, 8, 8, window=1000, far=17)),
    "unrotated": two(unrotated(4, 2, 16, 16, far=20)),
    "unrotated_odd_sizes": two(unrotated(3, 1, 14, 6, far=300)),
    "unrotated_one_head": two(unrotated(1, 1, 8, 24, far=9)),
    "unrotated_many_heads": two(unrotated(36, 2, 4, 4, far=15)),
    "unrotated_of_64_without_mixing": two(unrotated(4, 2, 64, 64, far=9, mix=False)),
    "unrotated_of_128": two(unrotated(4, 2, 128, 128, far=40)),
    "values_cut_into_other_heads": config([layer(unrotated(2, 2, 8, 12, far=9)), layer(rotated(3, 3, 8, 8, dims=4)), layer(windowed(4, 1, 16, 24, window=9, far=9)),
                                           layer(rotated(4, 4, 16, 6, dims=16))], **KW),
    "values_of_a_later_first_layer": config([layer(unrotated(2, 2, 8, 12, far=9, mix=False)), layer(rotated(2, 1, 16, 16, dims=4), dense(24)),
                                             layer(windowed(2, 2, 8, 12, window=9, far=9, mix=False)), layer(rotated(2, 1, 16, 16, dims=4))], **KW),
    "dense": two(SMALL, dense(24)),
    "dense_odd": two(SMALL, dense(13)),
    "experts": two(SMALL, moe(7, 2, 20)),
    "experts_with_a_shared_one": two(SMALL, moe(4, 3, 24, shared=9)),
    "experts_all_chosen": two(SMALL, moe(4, 4, 56, shared=64)),
    "experts_one": two(SMALL, moe(1, 1, 8, groups=(1, 1))),
    "experts_in_groups": two(SMALL, moe(12, 3, 16, groups=(6, 2), shared=24)),
    "experts_groups_of_one": two(SMALL, moe(9, 2, 16, groups=(9, 4))),
    "experts_many": two(SMALL, moe(160, 6, 8, groups=(8, 5))),
    "experts_whole_groups": two(SMALL, moe(6, 4, 16, groups=(3, 2))),
    "no_layers": config([], **KW, logit_scale=0.3),
    "one_bucket": config([layer(SMALL)], **KW, buckets=1, logit_scale=5.0),
    "large_multipliers": config([layer(SMALL)], **KW, buckets=991, mul_prev=2147483647, mul_cur=2147483629),
    "wide_and_uneven": config([layer(SMALL, moe(3, 2, 24)), layer(rotated(2, 1, 8, 8, dims=8), dense(16))], width=1048, vocab=50),
}


@DTYPES
@pytest.mark.parametrize("name", sorted(ALONE))
def test_each_mechanism_alone(tmp_path, name, dtype):
    cfg = copy.deepcopy(ALONE[name])
    w = random_weights(cfg, 3)
    folder = write_model(tmp_path / name, cfg, w)
    tokens = tokens_for(cfg, 45, 1)
    want = plain_logits(cfg, w, tokens)
    eng = engine(folder, dtype, page_size=16 if len(name) % 2 else 64)
    whole = run_cut(eng, 0, tokens, [45])
    assert close(whole, want, dtype)
    assert deviation(run_cut(eng, 1, tokens, [9, 2, 17] + [1] * 17), whole) < SAME[dtype]


@DTYPES
def test_many_rows_an_expert_take_the_tile_product(tmp_path, dtype):
    """A prompt long enough that the experts' rows go through the grouped tile product, its tokens one by one through the
    other route: the same logits."""
    cfg = config([layer(SMALL, moe(2, 1, 64, groups=(2, 1), shared=32))], width=64, vocab=50)
    w = random_weights(cfg, 4)
    folder = write_model(tmp_path / "tiles", cfg, w)
    tokens = tokens_for(cfg, 160, 2)
    eng = engine(folder, dtype)
    whole = run_cut(eng, 0, tokens, [160])
    assert close(whole, plain_logits(cfg, w, tokens), dtype)
    assert deviation(run_cut(eng, 1, tokens, [100] + [1] * 60), whole) < SAME[dtype]


def routed_otherwise(monkeypatch, mistake, cfg, w, tokens):
    """The plain implementation with a mistake in its router."""
    def route(router, w, p, h):
        E, top = router["experts"], router["top"]
        groups = router.get("groups") or {"count": 1, "keep": 1}
        size = E // groups["count"]
        s = torch.sigmoid(h @ w[p + "router"].double().T)
        c = s + (0.0 if mistake == "no correction" else w[p + "correction"].double())
        idx = torch.zeros(h.shape[0], top, dtype=torch.long)
        for t in range(h.shape[0]):
            def worth(g):
                of = c if mistake != "groups without correction" else s
                v = sorted(of[t, g * size:(g + 1) * size].tolist(), reverse=True)
                return v[0] if mistake == "groups by their largest" else sum(v[:2])
            best = sorted(range(groups["count"]), key=lambda g: -worth(g))[:groups["keep"]]
            value = lambda e: float(c[t, e]) if e // size in best else (0.0 if mistake == "others count as zero" else -1e30)
            idx[t] = torch.tensor(sorted(range(E), key=lambda e: -value(e))[:top])
        wts = torch.gather(c if mistake == "corrected weights" else s, 1, idx)
        return idx, wts / wts.sum(1, keepdim=True) if mistake == "weights of sum one" else wts
    with monkeypatch.context() as mp:
        mp.setattr(plain, "route", route)
        return plain_logits(cfg, w, tokens)


@DTYPES
def test_the_correction_decides_the_choice_and_not_the_weights(tmp_path, monkeypatch, dtype):
    """Fixed logits (a constant channel alone reaches the router) whose choice depends on the correction, on groups that are worth
    the sum of their two largest corrected scores, and on scores below zero that are still above those of groups left out."""
    cfg = config([layer(SMALL, moe(9, 3, 32, groups=(3, 1)))], width=32, vocab=50)
    w = random_weights(cfg, 6)
    bf = torch.bfloat16
    z = torch.tensor([2.0, -3.0, -3.0, 1.0, 0.9, 1.1, 0.5, 1.5, 1.2])
    base = torch.zeros(9, 32)
    base[:, 0] = z
    w["l0.mlp.router"] = base.to(bf)
    # Corrected: (0.3 -0.5 -0.6) (-0.2 -0.1 -0.9) (0.0 -0.8 -0.7): the second group's two best are worth most.
    target = torch.tensor([0.3, -0.9, -1.0, -0.2, -0.1, -0.9, 0.05, -0.8, -0.7])
    w["l0.mlp.correction"] = (target - torch.sigmoid(z)).to(bf)
    w["embed"][:, 0] = 3.0
    w["bigram"][:, 0] = 0.0
    w["l0.mix.o"][0] = 0.0                                               # the first channel stays what the embedding made it
    w["l0.norm2"][0] = 0.5
    for e in range(9):
        w[f"l0.mlp.e{e}.down"] = (w[f"l0.mlp.e{e}.down"].float() * 4).to(bf)
    # The router's input is a norm's output: near, not exactly, one.  The choice has room for that.
    tokens = tokens_for(cfg, 40, 3)
    want = plain_logits(cfg, w, tokens)
    for mistake in ("no correction", "groups without correction", "groups by their largest", "others count as zero", "corrected weights", "weights of sum one"):
        assert deviation(routed_otherwise(monkeypatch, mistake, cfg, w, tokens), want) > 0.1, mistake
    assert deviation(routed_otherwise(monkeypatch, "", cfg, w, tokens), want) < 1e-12
    folder = write_model(tmp_path / "groups", cfg, w)
    got = run_cut(engine(folder, dtype), 0, tokens, [17, 2] + [1] * 21)
    assert deviation(got, want) < TOLERANCE[dtype]


def test_the_residual_stream_is_32_bit(tmp_path):
    """Sixteen equal layers add small updates to a large stream; each is below half a step of a 16-bit stream of that size, so a
    stream that is rounded to 16 bits between sublayers loses them all.  The plain implementation with such a stream is checked
    to be far off first; the engine must be near the true one."""
    L = 16
    cfg = config([layer(windowed(2, 1, 8, 8, window=6, far=9, mix=False), dense(16)) for _ in range(L)], width=32, vocab=40, eps=1e-5)
    w = random_weights(cfg, 5)
    bf = torch.bfloat16
    w["embed"] = (torch.sign(w["embed"].float()) * 96.0).to(bf)
    w["bigram"] = torch.zeros_like(w["bigram"])
    w["l0.mix.o"] = (w["l0.mix.o"].float() * 0.15).to(bf)
    w["l0.mlp.down"] = (w["l0.mlp.down"].float() * 0.15).to(bf)
    for n in [n for n in w if n.startswith("l0.")]:
        for i in range(1, L):
            w[n.replace("l0.", f"l{i}.", 1)] = w[n].clone()
    tokens = tokens_for(cfg, 20, 2)
    want = plain_logits(cfg, w, tokens)
    eps = cfg["norm"]["eps"]
    x = plain.embed(cfg, w, tokens)
    base = (plain.norm(x, w["final.norm"], eps) @ w["embed"].double().T).numpy()
    for i in range(L):
        p = f"l{i}."
        x = (x + plain.attention("attention_2", cfg["layers"][i]["mixer"], w, p + "mix.", plain.norm(x, w[p + "norm1"], eps), eps, {})).to(bf).double()
        x = (x + plain.dense(w, p + "mlp.", plain.norm(x, w[p + "norm2"], eps))).to(bf).double()
    lossy = (plain.norm(x, w["final.norm"], eps) @ w["embed"].double().T).numpy()
    rms = np.sqrt(((want - base) ** 2).mean())
    assert np.sqrt((((lossy - base) - (want - base)) ** 2).mean()) > 0.5 * rms        # a 16-bit stream loses most of what the layers add
    folder = write_model(tmp_path / "deep", cfg, w)
    got = run_cut(engine(folder, "bfloat16"), 0, tokens, [20])
    # What the 16-bit products of the end cost moves every row alike; the layers' updates are what is compared: the
    # difference from the same engine without layers.
    bare = dict(cfg, layers=[])
    folder0 = write_model(tmp_path / "bare", bare, {n: t for n, t in w.items() if not n.startswith("l")})
    got0 = run_cut(engine(folder0, "bfloat16"), 0, tokens, [20])
    assert np.sqrt((((got - got0) - (want - base)) ** 2).mean()) < 0.35 * rms
    exact = run_cut(engine(folder, "float32"), 0, tokens, [20])
    assert np.sqrt(((exact - want) ** 2).mean()) < 0.02 * rms


@DTYPES
def test_the_token_before_wherever_a_request_is_cut(tmp_path, dtype):
    """No layers: the logits are the two embeddings'.  Every cut between two tokens, a request that starts where another ended
    (in its slot, its pages and its row of the batch), and one whose first token follows another request's last in a step."""
    cfg = config([], width=32, vocab=30, buckets=61, mul_prev=17, mul_cur=29, logit_scale=1.5)
    w = random_weights(cfg, 8)
    folder = write_model(tmp_path / "pairs", cfg, w)
    tokens = tokens_for(cfg, 12, 4)
    want = plain_logits(cfg, w, tokens)
    swapped = copy.deepcopy(cfg)
    swapped["embedding"]["bigram"].update(mul_prev=29, mul_cur=17)
    assert deviation(plain_logits(swapped, w, tokens), want) > 0.1
    eng = engine(folder, dtype, num_pages=2, page_size=16, max_num_seqs=2)
    for i in range(1, 12):
        assert close(run_cut(eng, i, tokens, [i, 12 - i]), want, dtype), i
    assert close(run_cut(eng, 20, tokens, [1] * 12), want, dtype)
    other = tokens_for(cfg, 7, 5)
    both = eng.trace_step([(30, other, [6]), (31, tokens[:3], [0, 2])])
    assert close(both, np.stack([plain_logits(cfg, w, other)[6], want[0], want[2]]), dtype)


# ----------------------------------------------------------------------------- cuttings, batches, pages and slots
@DTYPES
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_whole_prompt_portions_and_decoding_agree(models, name, dtype):
    folder, cfg, w = models[name]
    n = 150
    tokens = tokens_for(cfg, n, 7)
    want = plain_logits(cfg, w, tokens)
    eng = engine(folder, dtype, page_size=16 if name == "MIXED" else 64)
    whole = run_cut(eng, 0, tokens, [n])
    assert close(whole, want, dtype)
    # The first tokens of a sequence on their own rows (in bfloat16 a router may choose another expert for one of them).
    assert deviation(whole[:4], want[:4]) < (TOLERANCE[dtype] if dtype == "float32" else 0.5)
    cuttings = {
        "token by token": [1] * n,
        "portions down to two tokens": [2, 3, 16, 2, 1, 31, 2, 33, 5, 1, 1, 2, 17, 32, 2],
        "a prompt and then decoding": [n - 60] + [1] * 60,
        "portions that end on page borders": [16, 48, 64, 22],
    }
    for what, cuts in cuttings.items():
        got = run_cut(eng, 1, tokens, cuts)
        assert deviation(got, whole) < SAME[dtype], what


@DTYPES
def test_unequal_requests_in_one_batch(models, dtype):
    """Portions of some requests beside single tokens of others, a request left out of a step, against each alone."""
    folder, cfg, w = models["MIXED"]
    lengths = [70, 23, 41, 5]
    seqs = [tokens_for(cfg, n, 30 + i) for i, n in enumerate(lengths)]
    eng = engine(folder, dtype)
    alone = [run_cut(eng, 10 + i, s, [len(s)]) for i, s in enumerate(seqs)]
    at = [0] * 4
    got = [[] for _ in seqs]
    step = 0
    while any(a < n for a, n in zip(at, lengths)):
        entries, who = [], []
        for i, s in enumerate(seqs):
            if at[i] >= lengths[i] or (step + i) % 5 == 4:        # finished, or left out of this step
                continue
            c = min([7, 1, 2, 1][(step + i) % 4], lengths[i] - at[i])
            entries.append((i, s[at[i]:at[i] + c], list(range(c))))
            who.append((i, c))
            at[i] += c
        step += 1
        if not entries:
            continue
        rows = eng.trace_step(entries)
        r = 0
        for i, c in who:
            got[i].append(rows[r:r + c])
            r += c
    for i in range(4):
        assert deviation(np.concatenate(got[i], 0), alone[i]) < SAME[dtype], i


@DTYPES
def test_pages_are_used_again(models, dtype):
    """A pool of one request's pages: every request starts in what the one before left."""
    folder, cfg, w = models["MIXED"]
    eng = engine(folder, dtype, num_pages=4, page_size=16, max_num_seqs=1)
    for i, n in enumerate([60, 17, 64, 33]):
        tokens = tokens_for(cfg, n, 50 + i)
        got = run_cut(eng, i, tokens, [n // 2, n - n // 2 - 3, 1, 1, 1])
        assert close(got, plain_logits(cfg, w, tokens), dtype), i


@DTYPES
def test_long_decoding(models, dtype):
    folder, cfg, w = models["MIXED"]
    n = 300
    tokens = tokens_for(cfg, n, 9)
    eng = engine(folder, dtype, num_pages=20)
    got = run_cut(eng, 0, tokens, [40] + [1] * (n - 40))
    assert close(got, plain_logits(cfg, w, tokens), dtype)


@DTYPES
def test_some_rows_of_a_step_are_asked_for(models, dtype):
    """Logits at chosen places of a portion, at none, and of several requests at once: the rows of the whole."""
    folder, cfg, w = models["MIXED"]
    a, b = tokens_for(cfg, 30, 1), tokens_for(cfg, 12, 2)
    eng = engine(folder, dtype)
    whole_a, whole_b = run_cut(eng, 0, a, [30]), run_cut(eng, 1, b, [12])
    assert eng.trace_step([(2, a[:10], []), (3, b[:5], [])]).shape[0] == 0
    got = eng.trace_step([(2, a[10:], [19, 0, 7]), (3, b[5:], [6])])
    assert deviation(got, np.stack([whole_a[29], whole_a[10], whole_a[17], whole_b[11]])) < SAME[dtype]


# ------------------------------------------------------------------------- a key that stands out, wherever it is put
def marked_model(kind, window=None, dim=16, far=9.0, classes=6):
    """One layer with one head whose query is a constant direction and whose key lies along it for one token alone, the mark
    (token 1), and along another for the rest, and whose value carries the mark into the logits: the logits at a position move
    if and only if the marked key is visible from that position.  No biases by distance yet."""
    mixer = {"rotated": lambda: rotated(1, 1, dim, dim, dims=dim // 2, base=1e4, scale=14.0 / dim, mix=False),
             "windowed": lambda: windowed(1, 1, dim, dim, window, far, scale=14.0 / dim, mix=False),
             "unrotated": lambda: unrotated(1, 1, dim, dim, far, scale=14.0 / dim, mix=False)}[kind]()
    cfg = config([layer(mixer)], width=32, vocab=12)
    w = random_weights(cfg, 77, classes=classes)
    W, bf, p = cfg["width"], torch.bfloat16, "l0.mix."
    embed = torch.zeros(12, W)
    embed[:, 0] = 2.0                      # every token: a constant channel that makes the query and the other keys
    embed[1, 1] = 6.0                      # the mark: a channel that makes the key and the value
    embed[2:, 2:] = torch.randn(10, W - 2, generator=torch.Generator().manual_seed(3)) * 0.5
    w["embed"], w["bigram"] = embed.to(bf), torch.zeros_like(w["bigram"])
    for n in ("l0.norm1", "final.norm"):
        w[n] = torch.ones(W).to(bf)
    q, k, v, o = torch.zeros(dim, W), torch.zeros(dim, W), torch.zeros(dim, W), torch.zeros(W, dim)
    q[dim - 1, 0] = 1.0                    # beyond the rotated entries
    k[dim - 1, 1] = 4.0
    k[dim - 2, 0] = 0.25
    v[3, 1] = 1.0
    o[5, 3], o[9, 3] = 6.0, -6.0
    w[p + "q"], w[p + "k"], w[p + "v"], w[p + "o"] = q.to(bf), k.to(bf), v.to(bf), o.to(bf)
    if kind == "rotated":
        w[p + "g"] = torch.zeros(1, W).to(bf)
    else:
        w[p + "q.norm"], w[p + "k.norm"] = torch.ones(dim).to(bf), torch.ones(dim).to(bf)
        w[p + "rel"] = torch.zeros(classes, 1).to(bf)
    return cfg, w


@DTYPES
@pytest.mark.parametrize("window, dim", [(1, 16), (2, 16), (16, 24), (33, 64), (64, 128), (65, 200), (96, 256)])
def test_a_marked_key_is_seen_inside_the_window_alone(tmp_path, dtype, window, dim):
    cfg, w = marked_model("windowed", window, dim)
    folder = write_model(tmp_path / "marked", cfg, w)
    eng = engine(folder, dtype, num_pages=60, page_size=64 if dim in (64, 256) else 16)
    n = 140
    rid = 0
    # (marked position, asking position): at the asking position and just after it; just inside and just outside the window;
    # at page borders; the first tokens.
    cases = {(0, 0), (1, 0), (0, 1), (0, 2), (95, 95), (96, 95)}
    for ask in (window - 1, window, window + 1, 63, 64, 79, 80, 127, 128, n - 1):
        for mark in (ask - window - 1, ask - window, ask - window + 1, ask - window + 2):
            if 0 <= mark < n and ask < n:
                cases.add((mark, ask))
    base = [2 + (i * 7) % 10 for i in range(n)]
    p_base = plain_logits(cfg, w, base)
    for mark, ask in sorted(cases):
        tokens = list(base)
        tokens[mark] = 1
        seen = 0 <= ask - mark < window
        p_marked = plain_logits(cfg, w, tokens[:ask + 1])[ask]
        moved = np.abs(p_marked - p_base[ask]).max()
        assert (moved > 0.05) == seen, (mark, ask, moved)           # the plain implementation itself, first
        for cuts in ([n], [ask] + [1] * (n - ask) if ask else [n], [3, 2] + [5] * 27):
            got = run_cut(eng, rid, tokens, cuts)[ask]
            rid += 1
            assert np.sqrt(((got - p_marked) ** 2).mean()) < TOLERANCE[dtype] * np.sqrt((p_marked ** 2).mean()) + 1e-3, (mark, ask, cuts[:3])


@DTYPES
@pytest.mark.parametrize("kind, dim", [("windowed", 16), ("windowed", 128), ("unrotated", 24), ("unrotated", 256), ("rotated", 64), ("rotated", 200)])
def test_a_marked_key_far_away_among_hundreds(tmp_path, dtype, kind, dim):
    """One key far back, over many pages and segments, in a prompt, in portions and in decoding; with a window of 700 just
    inside for the rows before, just outside for the rows after."""
    cfg, w = marked_model(kind, 700, dim)
    folder = write_model(tmp_path / "far", cfg, w)
    n = 790
    tokens = [2 + (i * 7) % 10 for i in range(n)]
    tokens[70] = 1                                            # in a window of 700 the last row that sees it is 769
    want = plain_logits(cfg, w, tokens)[-40:]
    base = list(tokens)
    base[70] = 5
    moved = np.abs(want - plain_logits(cfg, w, base)[-40:]).max(-1)
    assert (moved[:20] > 0.05).all() and ((moved[20:] < 1e-9).all() if kind == "windowed" else (moved[20:] > 0.05).all())
    eng = engine(folder, dtype, num_pages=70, page_size=16 if dim % 64 else 64)
    for rid, cuts in enumerate(([n], [n - 40] + [1] * 40, [333, 2, 400, 15] + [1] * 40)):
        got = run_cut(eng, rid, tokens, cuts)[-40:]
        assert deviation(got, want) < TOLERANCE[dtype] + 1e-3, cuts[:3]


@DTYPES
@pytest.mark.parametrize("kind, dim, classes, far", [("windowed", 16, 16, 100.0), ("windowed", 64, 7, 20.0), ("unrotated", 128, 12, 60.0), ("unrotated", 24, 32, 350.0),
                                                     ("unrotated", 256, 9, 300.0), ("unrotated", 64, 2, 40.0)])
def test_a_bias_by_distance_at_the_borders_of_its_classes(tmp_path, dtype, kind, dim, classes, far):
    """One class's bias stands out against the others', and one marked key crosses it: its share of a row tells the row's distance
    from it.  Rows on both sides of every border of that class; the last class far away.  The plain implementation with a border
    that is one token off is checked to differ first."""
    n = 330
    eng = None
    for rid, cls in enumerate(sorted({0, classes // 2 - 1, classes // 2, classes - 2, classes - 1} - {-1})):
        cfg, w = marked_model(kind, 300, dim, far, classes)
        w["l0.mix.rel"] = torch.full((classes, 1), -14.0).to(torch.bfloat16)
        w["l0.mix.rel"][cls, 0] = 0.0
        tokens = [2 + (i * 7) % 10 for i in range(n)]
        tokens[11] = tokens[200] = 1
        want = plain_logits(cfg, w, tokens)
        per = [plain.distance_class(i, classes, far) for i in range(n)]
        assert any(c == cls for c in per) and any(c != cls for c in per)
        real, one_off = plain.distance_class, lambda i, rows, f: real(i + 1, rows, f)
        plain.distance_class = one_off
        try:
            assert deviation(plain_logits(cfg, w, tokens), want) > 0.05
        finally:
            plain.distance_class = real
        folder = write_model(tmp_path / f"class{cls}", cfg, w)
        eng = engine(folder, dtype, num_pages=40, page_size=16 if dim % 64 else 64)
        assert close(run_cut(eng, 2 * rid, tokens, [n]), want, dtype), cls
        assert close(run_cut(eng, 2 * rid + 1, tokens, [100, 2, 60] + [1] * (n - 162)), want, dtype), cls


@DTYPES
def test_banded_rotation_far_from_the_start(tmp_path, dtype):
    """Scores of rotated entries alone, at positions where a wrong frequency, pairing or band turns the keys away."""
    cfg = config([layer(rotated(2, 1, 32, 16, dims=32, base=10000.0, scaling=(4.0, 128, 1.0, 4.0), scale=0.25, mix=False))], width=32, vocab=30)
    w = random_weights(cfg, 8)
    tokens = tokens_for(cfg, 400, 4)
    want = plain_logits(cfg, w, tokens)
    for change in (lambda r: r.pop("scaling"), lambda r: r["scaling"].update(factor=3.5), lambda r: r["scaling"].update(low=2.0),
                   lambda r: r["scaling"].update(high=8.0), lambda r: r["scaling"].update(original=150), lambda r: r.update(base=9000.0), lambda r: r.update(dims=30)):
        other = copy.deepcopy(cfg)
        change(other["layers"][0]["mixer"]["rot"])
        assert deviation(plain_logits(other, w, tokens[:200]), want[:200]) > 2e-3
    folder = write_model(tmp_path / "bands", cfg, w)
    eng = engine(folder, dtype, num_pages=40)
    assert close(run_cut(eng, 0, tokens, [400]), want, dtype)
    assert close(run_cut(eng, 1, tokens, [350] + [1] * 50), want, dtype)


@DTYPES
def test_the_norm_stands_behind_the_rotation_and_the_gate_on_a_head(tmp_path, monkeypatch, dtype):
    """Queries and keys so small that eps counts in their norm, and gates that open one head and close another; the plain
    implementation with the gates exchanged, or without the norms, is checked to be far off first."""
    cfg = config([layer(rotated(2, 1, 8, 16, dims=4, scale=1.0, mix=False))], width=32, vocab=30, eps=1e-2)
    w = random_weights(cfg, 9)
    bf = torch.bfloat16
    for n in ("q", "k"):
        w[f"l0.mix.{n}"] = (w[f"l0.mix.{n}"].float() * 0.1).to(bf)
    w["l0.mix.g"] = (w["l0.mix.g"].float() * 3).to(bf)
    tokens = tokens_for(cfg, 50, 6)
    want = plain_logits(cfg, w, tokens)
    assert deviation(plain_logits(cfg, dict(w, **{"l0.mix.g": w["l0.mix.g"].flip(0)}), tokens), want) > 0.1
    for mistake in (lambda m, w, p, q, k, eps: (plain.rotate(q, m["rot"]), plain.rotate(k, m["rot"])),
                    lambda m, w, p, q, k, eps: (plain.rms(plain.rotate(q, m["rot"]), 0.0), plain.rms(plain.rotate(k, m["rot"]), 0.0))):
        with monkeypatch.context() as mp:
            mp.setitem(plain.QK, "attention", mistake)
            assert deviation(plain_logits(cfg, w, tokens), want) > 0.01
    folder = write_model(tmp_path / "gates", cfg, w)
    eng = engine(folder, dtype)
    assert close(run_cut(eng, 0, tokens, [50]), want, dtype)
    assert close(run_cut(eng, 1, tokens, [20, 2] + [1] * 28), want, dtype)


@DTYPES
def test_blended_values_are_what_is_cached(tmp_path, dtype):
    """Shares that all but replace a layer's own values: a row's output then hangs on the first layer's values of tokens that
    were computed many steps ago.  Another share, or the first layer's own share in use, is checked to be far off first."""
    cfg = config([layer(rotated(2, 2, 16, 16, dims=8)), layer(unrotated(4, 2, 8, 16, far=9)), layer(windowed(4, 1, 16, 32, window=20, far=9))], width=32, vocab=40)
    w = random_weights(cfg, 10)
    bf = torch.bfloat16
    w["l1.mix.vmix"], w["l2.mix.vmix"] = torch.tensor(0.9).to(bf), torch.tensor(1.25).to(bf)
    tokens = tokens_for(cfg, 60, 7)
    want = plain_logits(cfg, w, tokens)
    for n in ("l1.mix.vmix", "l2.mix.vmix"):
        assert deviation(plain_logits(cfg, dict(w, **{n: torch.tensor(0.0).to(bf)}), tokens), want) > 0.1
    folder = write_model(tmp_path / "blend", cfg, w)
    eng = engine(folder, dtype)
    whole = run_cut(eng, 0, tokens, [60])
    assert close(whole, want, dtype)
    assert deviation(run_cut(eng, 1, tokens, [13, 2, 5] + [1] * 40), whole) < SAME[dtype]


# ------------------------------------------------------------------------------------------------- generation
@pytest.mark.parametrize("graphs", [False, True])
def test_greedy_generation_through_the_scheduler(models, graphs):
    """create_engine -> the scheduler, the step function, the sampler: the tokens are the plain implementation's."""
    from vosti_amd.engine import create_engine
    from vosti_amd.sampling.params import SamplingParams
    folder, cfg, w = models["MIXED"]
    prompts = [tokens_for(cfg, n, 60 + i) for i, n in enumerate([19, 3, 40])]
    eng = create_engine(folder, dtype="float32", num_pages=24, page_size=16, max_num_seqs=4, graphs=graphs)
    for _ in range(2):                                         # the second time the recorded steps are replayed from the start
        out = eng.generate(prompts, SamplingParams(max_tokens=12, ignore_eos=True))
        for prompt, got in zip(prompts, out):
            assert list(got) == plain.generate_greedy(cfg, w, prompt, 12)


def test_a_shared_prefix_is_found_and_its_last_token_remembered(tmp_path):
    """Without windows pages are kept for later requests: a prompt that starts like an earlier one goes on behind the matched
    pages, where the embedding needs the token before."""
    from vosti_amd.engine import create_engine
    from vosti_amd.sampling.params import SamplingParams
    cfg = config([layer(rotated(2, 1, 16, 16, dims=8), dense(24)), layer(unrotated(4, 2, 8, 8, far=30))], width=32, vocab=60)
    w = random_weights(cfg, 12)
    folder = write_model(tmp_path / "prefix", cfg, w)
    eng = create_engine(folder, dtype="float32", num_pages=24, page_size=16, max_num_seqs=2, enable_prefix_cache=True)
    shared = tokens_for(cfg, 48, 90)
    for tail in (5, 9, 16):
        prompt = shared + tokens_for(cfg, tail, 91 + tail)
        assert list(eng.generate([prompt], SamplingParams(max_tokens=6, ignore_eos=True))[0]) == plain.generate_greedy(cfg, w, prompt, 6)
    assert eng.stats()["prefix_hits"] >= 6


def test_the_command_line_generates_the_plain_tokens(models):
    """The engine's program, started as a user starts it with --family puvirax: greedy tokens of the plain implementation."""
    import subprocess
    from vosti_amd.kernels import build
    folder, cfg, w = models["MIXED"]
    program = str(build.ensure("engine", verbose=False))
    lib = build.ensure("f32", verbose=False)
    prompt = tokens_for(cfg, 21, 70)
    r = subprocess.run([program, "--family", "puvirax", "--dtype", "float32", "--lib-dir", str(lib.parent), "--model-path", str(folder),
                        "--prompt-ids", ",".join(map(str, prompt)), "--max-tokens", "8", "--page-size", "16"], capture_output=True, text=True, timeout=110, env={})
    assert r.returncode == 0, r.stderr[-2000:]
    out = json.loads([l for l in r.stdout.splitlines() if l.startswith("MODEL_OUTPUT_TOKEN_IDS=")][0].split("=", 1)[1])
    assert out == plain.generate_greedy(cfg, w, prompt, 8)


# --------------------------------------------------------------------------------------------- the replay program
@DTYPES
def test_the_replay_program_with_four_slots_and_a_pool_for_the_live_requests(models, tmp_path, dtype):
    """bin/trace_run as a user starts it: seven requests of which at most four are live, portions of prompts beside single
    tokens, requests left out of steps, a pool sized for the live requests alone (so that pages are used again), a name that
    comes back after its request ended.  Every row against the plain implementation."""
    import random
    import subprocess
    import sys
    from pathlib import Path
    folder, cfg, w = models["MIXED"]
    lengths = {"a": 70, "b": 33, "c": 150, "d": 9, "e": 64, "f": 101, "a again": 41}
    tokens = {name: tokens_for(cfg, n, 80 + i) for i, (name, n) in enumerate(lengths.items())}
    rng = random.Random(5)
    waiting, live, fed, steps, most = list(lengths), [], {}, [], 0
    while waiting or live:
        while waiting and len(live) < 4 and not (waiting[0] == "a again" and "a" in live):
            live.append(waiting.pop(0))
            fed[live[-1]] = 0
        most = max(most, sum(-(-lengths[n] // 64) * 64 for n in live))
        entries, end = [], []
        for name in list(live):
            if rng.random() < 0.2 and len(live) > 1:
                continue                                            # left out of this step
            left = lengths[name] - fed[name]
            size = min(left, 1 if left <= 6 else rng.choice([1, 2, 3, 7, 16, 40]))
            entries.append({"id": name.split()[0], "name": name, "tokens": tokens[name][fed[name]:fed[name] + size], "want": list(range(size))})
            fed[name] += size
            if fed[name] == lengths[name]:
                end.append(name.split()[0])
                live.remove(name)
        steps.append({"step": len(steps), "entries": entries, "end": end})
    cmd = [sys.executable, str(Path(__file__).resolve().parent.parent / "bin" / "trace_run"), "--model", str(folder), "--dtype", dtype,
           "--out", str(tmp_path), "--max-tokens", str(most)]
    proc = subprocess.Popen(cmd, stdin=subprocess.PIPE, stdout=subprocess.PIPE, text=True)
    for rec in steps:
        proc.stdin.write(json.dumps(rec) + "\n")
        proc.stdin.flush()
        assert proc.stdout.readline().strip() == f"done {rec['step']}"
    proc.stdin.close()
    assert proc.wait(timeout=60) == 0
    rows = {name: [] for name in lengths}
    for rec in steps:
        if not any(e["want"] for e in rec["entries"]):
            continue
        got = np.fromfile(tmp_path / f"{rec['step']}.f32", dtype="<f4").reshape(-1, cfg["vocab"])
        at = 0
        for e in rec["entries"]:
            rows[e["name"]].append(got[at:at + len(e["want"])])
            at += len(e["want"])
        assert at == got.shape[0]
    for name in lengths:
        assert close(np.concatenate(rows[name], 0), plain_logits(cfg, w, tokens[name]), dtype), name
