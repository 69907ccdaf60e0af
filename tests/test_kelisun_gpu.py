"""The Kelisun decoder through the native engine against the plain implementation (tests/plain_kelisun.py).

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

import plain_kelisun as plain
from kelisun_models import CONFIGS, again, config, latent, layer, moe, random_weights, write_model

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
SMALL = latent(1, 8, 4, 8, kv_rank=8, window=6)      # a small mixer under what is tested
PLAIN32 = dict(width=32, vocab=50)


def two(mixer, **kw):
    """The layer twice, so that the second run's keys depend on the first's outputs."""
    layers = [layer(mixer)]
    return config(layers + [again(layers, 0)], **PLAIN32, **kw)


ALONE = {
    "latent": two(latent(3, 16, 8, 16, kv_rank=24, window=9)),
    "latent_twenty_heads": two(latent(20, 8, 4, 8, kv_rank=16, window=17)),
    "latent_many_heads_of_one_entry": two(latent(33, 1, 2, 1, kv_rank=16, window=12)),
    "latent_odd_sizes": two(latent(5, 10, 6, 12, kv_rank=13, window=7, base=300.0, scaling=(2.5, 30, 8.0, 1.0))),
    "latent_one_head_wide": two(latent(1, 64, 32, 80, kv_rank=96, window=40)),
    "latent_values_wider_than_the_latent": two(latent(2, 8, 2, 40, kv_rank=8, window=16)),
    "latent_row_of_64": two(latent(4, 16, 16, 16, kv_rank=48, window=20)),
    "latent_row_of_256": two(latent(3, 32, 64, 24, kv_rank=192, window=30)),
    "latent_row_wider_than_the_tiles": two(latent(3, 24, 32, 40, kv_rank=288, window=19, scaling=(4.0, 64, 8.0, 1.0))),
    "latent_row_of_all_columns": two(latent(2, 16, 64, 16, kv_rank=960, window=41)),
    "window_of_one": two(latent(2, 8, 4, 8, kv_rank=8, window=1)),
    "window_of_two": two(latent(2, 8, 4, 8, kv_rank=8, window=2)),
    "window_of_a_page": two(latent(2, 8, 4, 8, kv_rank=8, window=16)),
    "window_longer_than_the_sequence": two(latent(2, 8, 4, 8, kv_rank=8, window=1000)),
    "one_stream": two(SMALL, streams=1),
    "three_streams": two(SMALL, streams=3),
    "four_streams": two(SMALL, streams=4),
    "seven_streams": two(SMALL, streams=7),
    "experts": config([layer(SMALL, moe(7, 2, 20))], **PLAIN32),
    "experts_scaled": config([layer(SMALL, moe(4, 3, 24, scale=3.5))], **PLAIN32),
    "experts_all_chosen": config([layer(SMALL, moe(4, 4, 56))], **PLAIN32),
    "experts_one": config([layer(SMALL, moe(1, 1, 8, groups=(1, 1)))], **PLAIN32),
    "experts_in_groups": config([layer(SMALL, moe(12, 3, 16, groups=(6, 2)))], **PLAIN32),
    "experts_groups_of_one": config([layer(SMALL, moe(9, 2, 16, groups=(9, 4)))], **PLAIN32),
    "experts_many": config([layer(SMALL, moe(160, 6, 8, groups=(80, 5)))], **PLAIN32),
    "experts_whole_groups": config([layer(SMALL, moe(6, 4, 16, groups=(3, 2)))], **PLAIN32),
    "no_layers": config([], **PLAIN32),
    "wide_and_uneven": config([layer(latent(2, 8, 4, 8, kv_rank=8, window=8), moe(3, 2, 24))], width=1048, vocab=50, streams=2),
}


@DTYPES
@pytest.mark.parametrize("name", sorted(ALONE))
def test_each_mechanism_alone(tmp_path, name, dtype):
    cfg = copy.deepcopy(ALONE[name])
    w = random_weights(cfg, 3)
    folder = write_model(tmp_path / name, cfg, w)
    tokens = tokens_for(cfg, 45, 1)
    want = plain_logits(cfg, w, tokens)
    eng = engine(folder, dtype)
    assert close(run_cut(eng, 0, tokens, [45]), want, dtype)
    assert close(run_cut(eng, 1, tokens, [9, 2, 17] + [1] * 17), want, dtype)


@DTYPES
def test_many_rows_an_expert_take_the_tile_product(tmp_path, dtype):
    """A prompt long enough that the experts' rows go through the grouped tile product, its tokens one by one through the
    other route: the same logits."""
    cfg = config([layer(SMALL, moe(2, 1, 64, groups=(2, 1), scale=1.5))], width=64, vocab=50)
    w = random_weights(cfg, 4)
    folder = write_model(tmp_path / "tiles", cfg, w)
    tokens = tokens_for(cfg, 160, 2)
    eng = engine(folder, dtype)
    whole = run_cut(eng, 0, tokens, [160])
    assert close(whole, plain_logits(cfg, w, tokens), dtype)
    assert deviation(run_cut(eng, 1, tokens, [100] + [1] * 60), whole) < SAME[dtype]


@DTYPES
def test_groups_decide_which_experts_are_chosen(tmp_path, dtype):
    """Router weights of which one group holds the best expert and the two next best lie in another: with one kept group the
    second choice is a bad expert of the first group.  The plain implementation without groups is checked to be far off."""
    cfg = config([layer(SMALL, moe(6, 2, 32, groups=(2, 1), scale=4.0))], width=32, vocab=50)
    w = random_weights(cfg, 6)
    base = torch.zeros(6, 32)
    base[:, 0] = torch.tensor([3.0, -1.0, -2.0, 2.0, 2.5, 2.2])          # group 0: 3, -1, -2; group 1: 2, 2.5, 2.2
    w["l0.mlp.router"] = base.to(torch.bfloat16)
    w["embed"][:, 0] = 2.0
    w["l0.norm2"][0] = 1.0
    w["embed.norm"][0] = 1.5
    w["l0.mix.o"][0] = 0.0                                               # the first channel stays what the embedding made it
    tokens = tokens_for(cfg, 40, 3)
    want = plain_logits(cfg, w, tokens)
    free = copy.deepcopy(cfg)
    del free["layers"][0]["mlp"]["router"]["groups"]
    assert deviation(plain_logits(free, w, tokens), want) > 0.1
    normed = copy.deepcopy(cfg)
    normed["layers"][0]["mlp"]["router"]["scale"] = 1.0
    assert deviation(plain_logits(normed, w, tokens), want) > 0.1
    folder = write_model(tmp_path / "groups", cfg, w)
    assert close(run_cut(engine(folder, dtype), 0, tokens, [17, 2] + [1] * 21), want, dtype)


def test_the_residual_streams_are_32_bit(tmp_path):
    """Sixteen runs of one layer add small updates to large streams; each is below half a step of a 16-bit stream of that
    size, so streams that are rounded to 16 bits between sublayers lose them all.  The plain implementation with such
    streams is checked to be far off first; the engine must be near the true one."""
    layers = [layer(SMALL)]
    cfg = config(layers + [again(layers, 0) for _ in range(15)], width=32, vocab=40, streams=2)
    w = random_weights(cfg, 5)
    bf = torch.bfloat16
    w["l0.hc1.mix"], w["l0.hc1.out"], w["l0.hc1.in"] = torch.eye(2).to(bf), torch.full((2,), 0.125).to(bf), torch.full((2,), 0.5).to(bf)
    w["embed.norm"] = torch.full((32,), 64.0).to(bf)
    w["embed"] = torch.sign(w["embed"].float()).to(bf) * 1.5
    # Every token's value points the same way: the last channel of the latent is a constant.
    w["l0.mix.o"] = (w["l0.mix.o"].float() * 0.5).to(bf)
    tokens = tokens_for(cfg, 20, 2)
    want = plain_logits(cfg, w, tokens)
    eps = cfg["norm"]["eps"]
    x = plain.norm(w["embed"].double()[torch.tensor(tokens)], w["embed.norm"], eps)
    xs = x[None].repeat(2, 1, 1)
    for _ in range(16):
        xs = plain.hyper(xs, w, "l0.hc1.", lambda u: plain.latent_attention(SMALL, w, "l0.mix.", plain.norm(u, w["l0.norm1"], eps), eps))
        xs = xs.to(bf).double()
    lossy = (plain.norm(xs.sum(0), w["final.norm"], eps) @ w["head"].double().T).numpy()
    base = (plain.norm(x, w["final.norm"], eps) @ w["head"].double().T).numpy()
    moved = deviation(base, want)
    assert deviation(lossy, want) > 0.5 * moved and moved > 5e-3                # a 16-bit stream loses most of what the layers add
    folder = write_model(tmp_path / "deep", cfg, w)
    got = run_cut(engine(folder, "bfloat16"), 0, tokens, [20])
    # What the 16-bit products of the end cost moves every row alike; the layers' updates are what is compared: the
    # difference from the same engine without layers.
    bare = dict(cfg, layers=[])
    folder0 = write_model(tmp_path / "bare", bare, {n: t for n, t in w.items() if not n.startswith("l0.")})
    got0 = run_cut(engine(folder0, "bfloat16"), 0, tokens, [20])
    rms = np.sqrt(((want - base) ** 2).mean())
    assert np.sqrt((((got - got0) - (want - base)) ** 2).mean()) < 0.35 * rms
    assert np.sqrt((((lossy - base) - (want - base)) ** 2).mean()) > 0.5 * rms
    exact = run_cut(engine(folder, "float32"), 0, tokens, [20])
    assert deviation(exact, want) < 0.02 * moved


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
def marked_model(window, kv_rank=16, sink=0.0, head=16, page_rot=2):
    """One layer whose attention has one head whose query is a constant direction and whose key lies along it for one
    token alone, the mark (token 1), and whose value carries the mark into the logits: the logits at a position move if and
    only if the marked key is in the window of that position.  The second stream alone carries the attention's output."""
    cfg = config([layer(latent(1, head, page_rot, head, kv_rank=kv_rank, window=window, base=1e6, scale=1.0))], width=32, vocab=12)
    w = random_weights(cfg, 77)
    W, bf = cfg["width"], torch.bfloat16
    embed = torch.zeros(12, W)
    embed[:, 0] = 1.0                      # every token: a constant channel that makes the query
    embed[1, 1] = 6.0                      # the mark: a channel that makes the key and the value
    embed[2:, 2:] = torch.randn(10, W - 2, generator=torch.Generator().manual_seed(3)) * 0.2
    w["embed"] = embed.to(bf)
    for n in ("embed.norm", "l0.norm1"):
        w[n] = torch.ones(W).to(bf)
    q, dkv = torch.zeros(head + page_rot, W), torch.zeros(kv_rank + page_rot, W)
    q[0, 0] = 0.75
    dkv[0, 1] = 1.0                        # the latent's first entry: the mark
    dkv[1, 0] = 1.0                        # its second: the constant, so that its norm never divides by nothing
    uk, uv = torch.zeros(head, kv_rank), torch.zeros(head, kv_rank)
    uk[0, 0] = (16.0 / kv_rank) ** 0.5     # the key's first entry is the latent's first
    uv[:, 0] = 1.0
    p = "l0.mix."
    w[p + "q"], w[p + "dkv"], w[p + "uk"], w[p + "uv"] = q.to(bf), dkv.to(bf), uk.to(bf), uv.to(bf)
    w[p + "dkv.norm"] = torch.ones(kv_rank).to(bf)
    w[p + "sink"] = torch.tensor([sink]).to(bf)
    w["l0.hc1.in"], w["l0.hc1.out"], w["l0.hc1.mix"] = torch.tensor([1.0, 0.0]).to(bf), torch.tensor([0.0, 1.0]).to(bf), torch.eye(2).to(bf)
    return cfg, w


@DTYPES
@pytest.mark.parametrize("window, kv_rank", [(1, 16), (2, 16), (16, 16), (33, 62), (64, 16), (65, 126), (96, 300)])
def test_a_marked_key_is_seen_inside_the_window_alone(tmp_path, dtype, window, kv_rank):
    page = 16 if kv_rank != 126 else 64
    cfg, w = marked_model(window, kv_rank)
    folder = write_model(tmp_path / "marked", cfg, w)
    eng = engine(folder, dtype, num_pages=60, page_size=page)
    n = 140
    rid = 0
    # (marked position, asking position): at the asking position and just after it; just inside and just outside the window;
    # at page borders; the first tokens.
    cases = {(0, 0), (1, 0), (0, 1), (0, 2), (95, 95), (96, 95)}
    for ask in (window - 1, window, window + 1, 63, 64, 79, 80, 127, 128, n - 1):
        for mark in (ask - window - 1, ask - window, ask - window + 1, ask - window + 2):
            if 0 <= mark < n and ask < n:
                cases.add((mark, ask))
    for mark, ask in sorted(cases):
        tokens = [2 + (i * 7) % 10 for i in range(n)]
        base = list(tokens)
        tokens[mark] = 1
        seen = 0 <= ask - mark < window
        p_marked = plain_logits(cfg, w, tokens[:ask + 2])[ask]
        p_base = plain_logits(cfg, w, base[:ask + 2])[ask]
        moved = np.abs(p_marked - p_base).max()
        assert (moved > 0.05) == seen, (mark, ask, moved)           # the plain implementation itself, first
        for cuts in ([n], [ask] + [1] * (n - ask) if ask else [n], [3, 2] + [5] * 27):
            got = run_cut(eng, rid, tokens, cuts)[ask]
            rid += 1
            assert np.sqrt(((got - p_marked) ** 2).mean()) < TOLERANCE[dtype] * np.sqrt((p_marked ** 2).mean()) + 1e-3, (mark, ask, cuts[:3])


@DTYPES
@pytest.mark.parametrize("kv_rank", [16, 110, 270])
def test_a_marked_key_far_away_among_hundreds(tmp_path, dtype, kv_rank):
    """One key at the far end of a window of 700, over many pages and segments, in a prompt, in portions and in decoding: just
    inside for the rows before, just outside for the rows after."""
    cfg, w = marked_model(700, kv_rank)
    folder = write_model(tmp_path / "far", cfg, w)
    n = 790
    tokens = [2 + (i * 7) % 10 for i in range(n)]
    tokens[70] = 1                                            # the last row that sees it: 769
    want = plain_logits(cfg, w, tokens)[-40:]
    base = list(tokens)
    base[70] = 5
    moved = np.abs(want - plain_logits(cfg, w, base)[-40:]).max(-1)
    assert (moved[:20] > 0.05).all() and (moved[20:] < 1e-9).all()
    eng = engine(folder, dtype, num_pages=70, page_size=16)
    for rid, cuts in enumerate(([n], [n - 40] + [1] * 40, [333, 2, 400, 15] + [1] * 40)):
        got = run_cut(eng, rid, tokens, cuts)[-40:]
        assert deviation(got, want) < TOLERANCE[dtype] + 1e-3, cuts[:3]


@DTYPES
@pytest.mark.parametrize("kv_rank", [16, 270])
@pytest.mark.parametrize("sink", [-30.0, 4.0, 9.0, 40.0])
def test_a_sink_takes_its_share(tmp_path, dtype, sink, kv_rank):
    """A sink that is nothing, comparable to the marked key's score, or far beyond every score.  The plain implementation with
    another sink is checked to differ first, where it must."""
    cfg, w = marked_model(50, kv_rank, sink=sink)
    folder = write_model(tmp_path / "sink", cfg, w)
    tokens = [2 + (i * 7) % 10 for i in range(60)]
    tokens[3] = tokens[57] = 1
    want = plain_logits(cfg, w, tokens)
    other = dict(w)
    other["l0.mix.sink"] = torch.tensor([sink - 1.5]).to(torch.bfloat16)
    changed = np.abs(plain_logits(cfg, other, tokens) - want).max()
    assert (changed > 0.05) if 0 < sink < 30 else (changed < 1e-3)
    for cuts in ([60], [20, 2, 30] + [1] * 8):
        assert close(run_cut(engine(folder, dtype), 0, tokens, cuts), want, dtype)


@DTYPES
def test_stretched_rotation_far_from_the_start(tmp_path, dtype):
    """Scores of the rotated part alone, at positions where a wrong frequency, pairing or factor turns the keys away."""
    cfg = config([layer(latent(2, 8, 32, 16, kv_rank=16, window=60, base=10000.0, scaling=(4.0, 128, 8.0, 0.5), scale=0.5))], width=32, vocab=30)
    w = random_weights(cfg, 8)
    q = w["l0.mix.q"].float().view(2, 40, 32)
    q[:, :8] = 0
    w["l0.mix.q"] = q.view(80, 32).to(torch.bfloat16)
    tokens = tokens_for(cfg, 400, 4)
    want = plain_logits(cfg, w, tokens)
    for change in (lambda r: r.pop("scaling"), lambda r: r["scaling"].update(factor=3.5), lambda r: r["scaling"].update(slow=2.0),
                   lambda r: r["scaling"].update(fast=32.0), lambda r: r.update(base=9000.0)):
        other = copy.deepcopy(cfg)
        change(other["layers"][0]["mixer"]["rot"])
        assert deviation(plain_logits(other, w, tokens[:200]), want[:200]) > 2e-3
    folder = write_model(tmp_path / "yarn", cfg, w)
    eng = engine(folder, dtype, num_pages=40)
    assert close(run_cut(eng, 0, tokens, [400]), want, dtype)
    assert close(run_cut(eng, 1, tokens, [350] + [1] * 50), want, dtype)


@DTYPES
def test_layers_that_share_weights_keep_their_own_keys(tmp_path, dtype):
    """Four runs of one layer, the first tokens far from the later ones: a cache that the runs shared would show."""
    layers = [layer(latent(2, 8, 8, 16, kv_rank=24, window=25), moe(3, 3, 16))]
    layers += [again(layers, 0) for _ in range(3)]
    cfg = config(layers, width=32, vocab=40, streams=2)
    w = random_weights(cfg, 9)
    tokens = tokens_for(cfg, 90, 6)
    want = plain_logits(cfg, w, tokens)
    once = plain_logits(dict(cfg, layers=layers[:1]), w, tokens)
    assert deviation(once, want) > 0.1
    folder = write_model(tmp_path / "shared", cfg, w)
    eng = engine(folder, dtype)
    whole = run_cut(eng, 0, tokens, [90])
    assert close(whole, want, dtype)
    assert deviation(run_cut(eng, 1, tokens, [31, 2] + [1] * 57), whole) < SAME[dtype]


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


def test_the_command_line_generates_the_plain_tokens(models):
    """The engine's program, started as a user starts it with --family kelisun: greedy tokens of the plain implementation."""
    import subprocess
    from vosti_amd.kernels import build
    folder, cfg, w = models["MIXED"]
    program = str(build.ensure("engine", verbose=False))
    lib = build.ensure("f32", verbose=False)
    prompt = tokens_for(cfg, 21, 70)
    r = subprocess.run([program, "--family", "kelisun", "--dtype", "float32", "--lib-dir", str(lib.parent), "--model-path", str(folder),
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
