"""Fezuzen on the GPU against its plain implementation (``tests/plain/fezuzen_plain.py``): each mechanism alone, whole
prompts against portions and token-by-token decoding, unequal requests in one batch against each alone, pages and slots
that are used again, keys just inside and just outside windows and blocks in prompts and in decoding, one far key among
hundreds, the rows before a portion's first one (of the sublayers' inputs and of q, k and v), values turned by their
distance, a softmax whose denominator is mostly the one added to it, layers that read another layer's cache through a
wider window, groups that change the choice of experts, long decoding through recorded steps, sizes that are no
multiples of anything, greedy generation through the entry point and its scheduler, and the kernels alone."""
from types import SimpleNamespace

import numpy as np
import pytest
import torch

from tests.fezuzen_util import (ALL_SMALL, LONG, SMALL_A, SMALL_B, SMALL_C, attention, check_rows, config, expected, latent,
                                layer, make_folder, moe, plain_logits, plain_of, tokens_of)
from tests.plain import fezuzen_plain as P

pytestmark = pytest.mark.gpu
DTYPES = ["float32", "bfloat16"]


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    return {s["name"]: make_folder(s, tmp_path_factory.mktemp(f"fz{s['name']}")) for s in ALL_SMALL}


def entry(rid, tokens, want=None):
    from jax_vllm_amd.engine.entries import StepEntry

    return StepEntry(rid, tokens, range(len(tokens)) if want is None else want)


def make_core(folder, dtype, page_size, pages=64, seqs=4, graphs=False):
    from jax_vllm_amd.config import EngineConfig
    from jax_vllm_amd.engine.core import EngineCore
    from jax_vllm_amd.weights import load_model

    model, _ = load_model(folder, dtype, "cuda")
    cfg = EngineConfig(dtype=dtype, block_size=page_size, num_blocks=pages + 1, max_num_seqs=seqs,
                       max_model_len=pages * page_size, max_num_batched_tokens=4096, enable_prefix_cache=False,
                       use_hip_graphs=graphs)
    return EngineCore(model, cfg)


def run_cut(core, rid, tokens, cuts):
    """The request's logits at every position, its tokens fed in portions of the given sizes."""
    core.start_request(rid)
    out, at = [], 0
    for n in cuts:
        out.append(core.run([entry(rid, tokens[at:at + n])]).cpu().numpy())
        at += n
    assert at == len(tokens)
    core.finish_request(rid)
    return np.concatenate(out)


# ------------------------------------------------------------------ each mechanism alone
TINY = attention(1, 1, 4, conv=None)            # the smallest mixer, beside the feed-forward under test
ALONE = {
    "input_filters_of_six_taps": dict(layers=[layer(TINY)], taps=6),
    "input_filters_of_one_tap": dict(layers=[layer(TINY, moe(2, 1, 8))], taps=1),
    "filters_on_q_k_v": dict(layers=[layer(attention(2, 1, 8, conv=5))], taps=2),
    "filters_on_q_k_v_of_one_tap": dict(layers=[layer(attention(2, 1, 8, conv=1))], taps=3),
    "part_of_a_head_turned": dict(layers=[layer(attention(3, 3, 16, conv=None, rot=(6, 200.0)))]),
    "values_wider_than_keys": dict(layers=[layer(attention(4, 2, 8, 24, scale=0.7))]),
    "values_narrower_than_keys": dict(layers=[layer(attention(4, 1, 24, 6))]),
    "blocks": dict(layers=[layer(attention(2, 2, 8, size=12))]),
    "blocks_of_one": dict(layers=[layer(attention(2, 1, 8, size=1))]),
    "latent_attention": dict(layers=[layer(latent(3, 8, 4, 12, 10, 20, scale=0.5, rot=(4, 100.0)))]),
    "latent_window": dict(layers=[layer(latent(2, 8, 4, 12, 9, 20, size=7))]),
    "latent_rescaled_frequencies": dict(layers=[layer(latent(2, 6, 16, 5, 12, 11, rot=(16, 100.0), scaling=LONG))]),
    "latent_part_of_the_part_turned": dict(layers=[layer(latent(2, 6, 8, 5, 12, 11, rot=(2, 30.0)))]),
    "latent_cache_read_by_two_layers": dict(layers=[
        layer(latent(2, 8, 4, 6, 10, 16, size=5, rot=(4, 50.0))), layer(TINY),
        layer(latent(3, 4, 4, 10, 8, 16, scale=0.7, size=11, rot=(4, 50.0), kv_from=0)),
        layer(latent(1, 12, 4, 8, 6, 16, size=2, rot=(4, 50.0), kv_from=0))]),
    "experts": dict(layers=[layer(TINY, moe(7, 3, 24))]),
    "experts_one_chosen": dict(layers=[layer(TINY, moe(4, 1, 10))]),
    "experts_all_chosen": dict(layers=[layer(TINY, moe(3, 3, 16))]),
    "experts_in_groups": dict(layers=[layer(TINY, moe(12, 3, 16, groups=(4, 2)))]),
    "experts_in_groups_of_one": dict(layers=[layer(TINY, moe(5, 2, 8, groups=(5, 2)))]),
    "one_group_kept": dict(layers=[layer(TINY, moe(8, 4, 8, groups=(2, 1)))]),
    "shared_expert": dict(layers=[layer(TINY, moe(4, 2, 8, shared=20))]),
    "shared_expert_of_the_experts_size": dict(layers=[layer(TINY, moe(4, 2, 16, shared=16))]),
    "shared_expert_of_three_times_the_experts_size": dict(layers=[layer(TINY, moe(4, 2, 8, shared=24))]),
    "constant_on_the_logits": dict(layers=[layer(TINY)], logit_scale=0.3),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("which", sorted(ALONE))
def test_one_mechanism_at_a_time(tmp_path, dtype, which):
    """A model of one or a few layers with one mechanism beside the smallest mixer and nothing else optional: a prompt
    of 70 tokens whole, and again in portions down to two tokens and single ones."""
    small = dict(name=which, seed=11, std=0.3, norm_std=0.2, config=config(40, 61, **ALONE[which]))
    folder = make_folder(small, tmp_path)
    cfg, w = plain_of(folder)
    toks = tokens_of(cfg, 70, 1)
    want = expected(cfg, w, toks, dtype)
    core = make_core(folder, dtype, 8)
    check_rows(dtype, run_cut(core, "whole", toks, [70]), want, "whole")
    check_rows(dtype, run_cut(core, "cut", toks, [2, 3, 1, 17, 2, 31, 1, 1, 2, 10]), want, "portions")


# ------------------------------------------------------------------ portions, decoding, first tokens
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("small", ALL_SMALL, ids=[s["name"] for s in ALL_SMALL])
def test_whole_prompt_portions_and_decoding_agree(folders, dtype, small):
    cfg, w = plain_of(folders[small["name"]])
    toks = tokens_of(cfg, 75, 2)
    want = expected(cfg, w, toks, dtype)
    core = make_core(folders[small["name"]], dtype, small["page_size"])
    check_rows(dtype, run_cut(core, "whole", toks, [75]), want, "whole")
    check_rows(dtype, run_cut(core, "single", toks, [1] * 75), want, "token by token")
    check_rows(dtype, run_cut(core, "twos", toks, [2] * 37 + [1]), want, "portions of two")
    check_rows(dtype, run_cut(core, "mixed", toks, [7, 9, 16, 1, 1, 33, 8]), want, "portions of several sizes")
    check_rows(dtype, run_cut(core, "prompt+decode", toks, [40] + [1] * 35), want, "prompt, then decoding")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("small", ALL_SMALL, ids=[s["name"] for s in ALL_SMALL])
def test_first_tokens_of_a_sequence(folders, dtype, small):
    """The first tokens see filters whose further taps lie before the sequence and one key beside the one added to the
    denominator: prompts of one to nine tokens (as many as the longest filter has taps, and one more) in every cut."""
    cfg, w = plain_of(folders[small["name"]])
    toks = [5, 1, 9, 2, 7, 30, 8, 8, 4]
    want = expected(cfg, w, toks, dtype)
    core = make_core(folders[small["name"]], dtype, small["page_size"])
    for rid, cuts in (("one", [1] * 9), ("two", [1, 2, 2, 2, 2]), ("three", [3, 2, 4]), ("whole", [9]), ("late", [8, 1])):
        check_rows(dtype, run_cut(core, rid, toks, cuts), want, rid)
    check_rows(dtype, run_cut(core, "alone", toks[:1], [1]), expected(cfg, w, toks[:1], dtype), "a prompt of one token")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("where", ["sublayer inputs", "q, k and v"])
def test_the_rows_before_a_portion_decide_its_first_rows(tmp_path, dtype, where):
    """Filters whose furthest tap is the largest, and two requests with the same tokens but for one in the middle: the
    row three tokens behind it differs by much (checked on the plain implementation), so a row before that is lost at a
    portion's start, taken from the batch's neighbour or from the slot's last owner shows.  Both requests run cut at
    different places, alone and side by side, and a third in a slot that was used before.  Blocks of one token: no key
    carries the changed token on."""
    inputs = where == "sublayer inputs"
    small = dict(name="rows", seed=13, std=0.3, norm_std=0.1,
                 config=config(32, 50, [layer(attention(2, 1, 8, size=1, conv=None if inputs else 4))], taps=4 if inputs else 1))
    tap = lambda t: torch.cat([torch.full_like(t[:, :1], 2.0), t[:, 1:]], dim=1)      # noqa: E731
    patch = {"l0.canon1": tap} if inputs else {f"l0.mix.{s}.conv": tap for s in "qkv"}
    folder = make_folder(small, tmp_path, patch)
    cfg, w = plain_of(folder)
    a = tokens_of(cfg, 40, 3)
    b = list(a)
    b[19] = (a[19] + 7) % 50
    c = [(t + 3) % 50 for t in a]
    plain_a, plain_b = plain_logits(cfg, w, a), plain_logits(cfg, w, b)
    moved = np.abs(plain_a - plain_b).max(axis=-1)
    assert moved[22] > 0.05 * np.abs(plain_a).max() and moved[23:].max() == 0 and moved[:19].max() == 0
    core = make_core(folder, dtype, 8, seqs=2)
    for rid, toks in (("a", a), ("b", b)):
        for cuts in ([1, 1, 2, 5, 1, 1, 9, 2, 18], [20, 20], [21, 1, 18], [22, 18], [19] + [1] * 21):
            check_rows(dtype, run_cut(core, rid, toks, cuts), expected(cfg, w, toks, dtype), f"{rid} {cuts}")
    core.start_request("a")
    core.start_request("b")
    got = {"a": [], "b": []}
    at = {"a": 0, "b": 0}
    for na, nb in ((20, 1), (1, 19), (2, 1), (1, 1), (16, 18)):
        es = []
        for r, toks, n in (("a", a, na), ("b", b, nb)):
            es.append(entry(r, toks[at[r]:at[r] + n]))
            at[r] += n
        out = core.run(es).cpu().numpy()
        got["a"].append(out[:na])
        got["b"].append(out[na:])
    core.finish_request("a")
    core.finish_request("b")
    check_rows(dtype, np.concatenate(got["a"]), expected(cfg, w, a, dtype), "a beside b")
    check_rows(dtype, np.concatenate(got["b"]), expected(cfg, w, b, dtype), "b beside a")
    check_rows(dtype, run_cut(core, "c", c, [1] * 6 + [34]), expected(cfg, w, c, dtype), "a slot used again")


# ------------------------------------------------------------------ windows, blocks, far keys
def edge_model(tmp_path, kind, size, scale=0.15):
    """One layer with scores sharp enough that single keys count in many rows (filters that hardly reach back)."""
    mix = attention(4, 2, 16, scale=scale, size=size, conv=None) if kind == "blocks" else latent(4, 16, 16, 8, 24, 32, scale=scale, size=size)
    small = dict(name="edge", seed=23, std=0.35, norm_std=0.1, config=config(32, 50, [layer(mix)], taps=2))
    folder = make_folder(small, tmp_path, {"l0.canon1": lambda t: t * 0.1})
    return folder, *plain_of(folder)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind,size", [("window", 16), ("window", 37), ("window", 64), ("blocks", 16), ("blocks", 37), ("blocks", 64)])
def test_keys_just_inside_and_just_outside_a_window_or_block(tmp_path, dtype, kind, size):
    """One key more or less at the edge moves many rows by much on the plain implementation.  Whole prompts, portions that
    end at, one before and one behind edges of blocks and pages, and decoding across them."""
    folder, cfg, w = edge_model(tmp_path, kind, size)
    n = 150
    toks = tokens_of(cfg, n, 12)
    plain = plain_logits(cfg, w, toks)
    i, j = torch.arange(n).view(n, 1), torch.arange(n).view(1, n)
    seen = P.chunk_mask(n, size) if kind == "blocks" else P.window_mask(n, size)
    first = (i - i % size) if kind == "blocks" else torch.clamp(i - size + 1, min=0)
    inside = seen & ~((j == first) & (j < i))                               # the first key in sight is lost
    outside = seen | ((j == first - 1) & (first > 0))                       # the last key out of sight is seen
    for mask in (inside, outside):
        moved = np.abs(plain_logits(cfg, w, toks, masks={0: mask}) - plain).max(axis=-1)
        assert (moved > 0.005 * np.abs(plain).max()).mean() > 0.3
    want = expected(cfg, w, toks, dtype)
    core = make_core(folder, dtype, 16, pages=12)
    check_rows(dtype, run_cut(core, "whole", toks, [n]), want, "whole")
    check_rows(dtype, run_cut(core, "decoded", toks, [size - 1] + [1] * (n - size + 1)), want, "decoded across every edge")
    check_rows(dtype, run_cut(core, "cut", toks, [15, 1, 1, 15, 4, 2, 26, 1, 64, 21]), want, "portions")
    assert core.cache.num_free_pages(0) == 12       # every page came back


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["blocks", "window"])
def test_one_far_key_among_hundreds_and_page_borders(tmp_path, dtype, kind):
    """Blocks and windows of 400: rows beyond position 200 change by much when the plain implementation is kept from
    seeing keys more than 150 back.  500 tokens over 32 pages: whole, in portions that end at, one before and one after
    page borders, with the last 60 decoded; the pages of the first block go back when the second one begins."""
    folder, cfg, w = edge_model(tmp_path, kind, 400, scale=0.3)
    n = 500
    toks = tokens_of(cfg, n, 13)
    want = expected(cfg, w, toks, dtype)
    plain = plain_logits(cfg, w, toks)
    seen = P.chunk_mask(n, 400) if kind == "blocks" else P.window_mask(n, 400)
    near = plain_logits(cfg, w, toks, masks={0: seen & P.window_mask(n, 150)})
    assert np.median(np.abs(near[200:400] - plain[200:400]).max(axis=-1)) > 0.01 * np.abs(plain).max()
    core = make_core(folder, dtype, 16, pages=32)
    check_rows(dtype, run_cut(core, "whole", toks, [n]), want, "whole")
    core.start_request("again")
    got, at = [], 0
    for m in [64, 63, 1, 17, 47, 2, 66, 139, 1, 40] + [1] * 60:
        got.append(core.run([entry("again", toks[at:at + m])]).cpu().numpy())
        at += m
        if kind == "blocks" and at >= 400:
            assert sum(1 for t in core.cache.block_table("again", 0) if t) <= -(-at // 16) - 25
    assert at == n
    core.finish_request("again")
    check_rows(dtype, np.concatenate(got), want, "portions and decoding")
    assert core.cache.num_free_pages(0) == 32


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_reader_with_a_wider_window_finds_its_keys(tmp_path, dtype):
    """A layer with a window of 6 and one with a window of 90 on its cache: the pages stay for the wider one (on the plain
    implementation the narrower window moves many rows by much), and go back behind it."""
    layers = [layer(latent(2, 16, 8, 8, 16, 24, scale=2.0, size=6, rot=(8, 1e3))),
              layer(latent(4, 16, 8, 8, 16, 24, scale=3.0, size=90, rot=(8, 1e3), kv_from=0))]
    small = dict(name="reader", seed=29, std=0.35, norm_std=0.1, config=config(32, 50, layers, taps=2))
    folder = make_folder(small, tmp_path)
    cfg, w = plain_of(folder)
    toks = tokens_of(cfg, 200, 5)
    plain = plain_logits(cfg, w, toks)
    moved = np.abs(plain_logits(cfg, w, toks, masks={1: P.window_mask(200, 6)}) - plain).max(axis=-1)
    assert np.median(moved[60:]) > 0.02 * np.abs(plain).max()
    want = expected(cfg, w, toks, dtype)
    core = make_core(folder, dtype, 8, pages=27)
    assert core.group_keys == [("window", 90)]
    check_rows(dtype, run_cut(core, "whole", toks, [200]), want, "whole")
    check_rows(dtype, run_cut(core, "cut", toks, [50, 3, 70, 2] + [1] * 75), want, "portions and decoding")
    assert core.cache.num_free_pages(0) == 27


@pytest.mark.parametrize("dtype", DTYPES)
def test_values_turn_by_their_distance(tmp_path, dtype):
    """Flat scores (every key weighs alike) over values that turn fast: without the turn, or without turning the result
    back, the plain logits move by much, also at positions in the thousands."""
    small = dict(name="turn", seed=31, std=0.3, norm_std=0.1, config=config(32, 50, [layer(attention(2, 1, 8, 12, scale=0.01, size=24, conv=2, rot=(2, 10.0)))], taps=1))
    folder = make_folder(small, tmp_path)
    cfg, w = plain_of(folder)
    toks = tokens_of(cfg, 3000, 6)
    plain = plain_logits(cfg, w, toks[:100])
    turn = P.turn_values
    try:
        for fake in (lambda x, base, sign=1.0: x, lambda x, base, sign=1.0: turn(x, base) if sign > 0 else x):
            P.turn_values = fake
            assert np.median(np.abs(plain_logits(cfg, w, toks[:100]) - plain).max(axis=-1)) > 0.05 * np.abs(plain).max()
    finally:
        P.turn_values = turn
    # a sequence's last blocks far from its start: the plain implementation over all 3,000 positions, filters included
    want = expected(cfg, w, toks, dtype)
    core = make_core(folder, dtype, 16, pages=190)
    got = run_cut(core, "long", toks, [1000, 1, 999, 960] + [1] * 40)
    if dtype == "float32":      # angles in the thousands of radians are rounded to float: a few 1e-4
        err = np.abs(got - want).max(axis=-1)
        scale = np.abs(want).max()
        assert err.max() <= 1e-3 * scale and err[:200].max() <= 5e-5 * scale, (err.max(), err[:200].max(), scale)
    else:
        check_rows(dtype, got, want, "long")


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_one_in_the_denominator_counts(tmp_path, dtype):
    """Small scores in short blocks: the one added to the denominator takes much of every row's weight (an ordinary softmax
    moves the plain logits by much); the split of a decoded token's keys over several blocks counts it once."""
    small = dict(name="one", seed=37, std=0.3, norm_std=0.1, config=config(32, 50, [layer(attention(4, 1, 16, scale=0.02, size=300))], taps=3))
    folder = make_folder(small, tmp_path)
    cfg, w = plain_of(folder)
    toks = tokens_of(cfg, 280, 4)
    plain = plain_logits(cfg, w, toks)
    plus_one = P.softmax_plus_one
    try:
        P.softmax_plus_one = lambda s, seen: torch.softmax(s.masked_fill(~seen, float("-inf")), dim=-1)
        off = plain_logits(cfg, w, toks)
    finally:
        P.softmax_plus_one = plus_one
    moved = np.abs(off - plain).max(axis=-1)
    assert moved[:8].max() > 0.03 * np.abs(plain).max() and (moved[:40] > 0.001 * np.abs(plain).max()).mean() > 0.5
    want = expected(cfg, w, toks, dtype)
    core = make_core(folder, dtype, 16)
    check_rows(dtype, run_cut(core, "whole", toks, [280]), want, "whole")
    check_rows(dtype, run_cut(core, "cut", toks, [1, 1, 2, 226, 10] + [1] * 40), want, "portions and decoding")


def test_groups_change_the_choice_of_experts(tmp_path):
    """One of four groups kept: most tokens choose other experts than their largest scores, the weights still are the
    softmax over all experts, and the engine follows."""
    small = dict(name="groups", seed=19, std=0.3, norm_std=0.2, config=config(40, 61, [layer(TINY, moe(16, 3, 12, shared=8, groups=(4, 1)))]))
    folder = make_folder(small, tmp_path)
    cfg, w = plain_of(folder)
    u = torch.randn(60, 40, dtype=torch.float64)
    f = cfg["layers"][0]["mlp"]
    choice, _ = P.router(w, "l0.mlp.", f, u)
    free = torch.topk(u @ w["l0.mlp.router"].T, 3, dim=-1).indices
    assert (choice.sort(-1).values != free.sort(-1).values).any(-1).float().mean() > 0.7
    toks = tokens_of(cfg, 60, 2)
    want = expected(cfg, w, toks, "float32")
    core = make_core(folder, "float32", 8)
    check_rows("float32", run_cut(core, "whole", toks, [60]), want, "whole")
    check_rows("float32", run_cut(core, "cut", toks, [1, 2, 30, 27]), want, "portions")


# ------------------------------------------------------------------ batches, pages and slots used again
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("small", [SMALL_A, SMALL_C], ids=["A", "C"])
def test_unequal_requests_in_one_batch_with_pages_and_slots_used_again(folders, dtype, small):
    """Seven requests of 1 to 90 tokens through two slots and a small pool of pages, portions of some beside single
    tokens of others; each request's logits equal the plain implementation's of it alone."""
    cfg, w = plain_of(folders[small["name"]])
    ps = small["page_size"]
    lengths = [33, 1, 90, 17, 64, 5, 48]
    reqs = {f"r{i}": tokens_of(cfg, n, 10 + i) for i, n in enumerate(lengths)}
    want = {r: expected(cfg, w, t, dtype) for r, t in reqs.items()}
    pages = max(14, 2 * (-(-90 // ps)) + 2)
    core = make_core(folders[small["name"]], dtype, ps, pages=pages, seqs=2)
    got = {r: [] for r in reqs}
    at = {r: 0 for r in reqs}
    waiting, live = list(reqs), []
    rng = np.random.default_rng(5)
    slots_seen = []
    while waiting or live:
        while waiting and len(live) < 2:
            r = waiting.pop(0)
            core.start_request(r)
            slots_seen.append(core.cache.slot(r))
            live.append(r)
        entries = []
        for r in live:
            left = len(reqs[r]) - at[r]
            n = 1 if (at[r] > 0 and rng.integers(2)) else int(min(left, rng.choice([1, 2, 3, 8, 21])))
            entries.append(entry(r, reqs[r][at[r]:at[r] + n]))
            at[r] += n
        logits = core.run(entries).cpu().numpy()
        k = 0
        for e in entries:
            got[e.request_id].append(logits[k:k + len(e.tokens)])
            k += len(e.tokens)
        for r in list(live):
            if at[r] == len(reqs[r]):
                core.finish_request(r)
                live.remove(r)
        core.cache.check_invariants()
    assert sorted(set(slots_seen)) == [0, 1] and len(slots_seen) == 7         # slots were used again
    assert all(core.cache.num_free_pages(g) == pages for g in range(len(core.group_keys)))
    if dtype == "float32":
        for r in reqs:
            check_rows(dtype, np.concatenate(got[r]), want[r], r)
    else:       # few rows a request: the shares of rows that rounding moves far are judged over all of them
        check_rows(dtype, np.concatenate([x for r in reqs for x in got[r]]),
                   tuple(np.concatenate([want[r][k] for r in reqs]) for k in (0, 1)), "all requests")


# ------------------------------------------------------------------ long decoding, recorded steps
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("graphs", [False, True], ids=["eager", "recorded"])
def test_long_decoding(folders, dtype, graphs):
    """260 decoded tokens behind a prompt of 9, over many pages, windows and blocks; with recorded steps two requests
    decode side by side (the shorter one leaves a padded row, whose state goes to the spare slot)."""
    cfg, w = plain_of(folders["A"])
    a, b = tokens_of(cfg, 269, 6), tokens_of(cfg, 150, 7)
    want_a, want_b = expected(cfg, w, a, dtype), expected(cfg, w, b, dtype)
    core = make_core(folders["A"], dtype, SMALL_A["page_size"], pages=60, graphs=graphs)
    core.start_request("a")
    core.start_request("b")
    got_a = [core.run([entry("a", a[:9])]).cpu().numpy()]
    got_b = [core.run([entry("b", b[:30])]).cpu().numpy()]
    for i in range(9, 269):
        es = [entry("a", a[i:i + 1])]
        j = 30 + i - 9
        if j < 150:
            es.append(entry("b", b[j:j + 1]))
        out = core.run(es).cpu().numpy()
        got_a.append(out[:1])
        if j < 150:
            got_b.append(out[1:2])
    check_rows(dtype, np.concatenate(got_a), want_a, "a")
    check_rows(dtype, np.concatenate(got_b), want_b, "b")
    if graphs:
        assert core.graph_replays > 200


# ------------------------------------------------------------------ the entry point
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("which", ["A", "C"])
def test_greedy_generation_through_the_entry_point(folders, dtype, which):
    """Four prompts through ``LLM.generate`` with two slots, a small token budget (prompts are cut) and few pages, decode
    steps recorded and following each other without the host in between: in float32 every token is the plain
    implementation's argmax; in bfloat16 each token is within a margin of the plain maximum given what came before."""
    from jax_vllm_amd import LLM, SamplingParams

    small = {"A": SMALL_A, "C": SMALL_C}[which]
    cfg, w = plain_of(folders[which])
    prompts = [tokens_of(cfg, n, 30 + n) for n in (3, 41, 18, 70)]
    llm = LLM(folders[which], dtype=dtype, block_size=small["page_size"], max_num_seqs=2, max_model_len=128,
              max_num_batched_tokens=24, num_blocks=max(9, 256 // small["page_size"] + 1))
    assert llm.prewarm() > 0.0
    got = llm.generate(prompts, SamplingParams(max_new_tokens=12))
    assert [len(g) for g in got] == [12] * 4
    for p, g in zip(prompts, got):
        seq = list(p)
        for i, t in enumerate(g):
            logits = P.forward(w, cfg, seq)[-1]
            if dtype == "float32":
                assert int(torch.argmax(logits)) == t, f"token {i}: engine {t}, plain {int(torch.argmax(logits))}"
            else:
                assert float(logits.max() - logits[t]) <= 0.06 * float(logits.abs().max()), f"token {i} is far below the maximum"
            seq.append(t)


def test_command_line_runs_the_design(folders, capsys):
    from jax_vllm_amd.engine.cli import main

    cfg, w = plain_of(folders["B"])
    prompt = tokens_of(cfg, 12, 40)
    code = main(["--model-path", str(folders["B"]), "--dtype", "fp32", "--block-size", "16", "--max-model-len", "64",
                 "--max-prefill-len", "32", "--max-new-tokens", "5", "--no-prewarm", "--prompt-ids",
                 " ".join(map(str, prompt))])
    assert code == 0
    got = [int(t) for t in capsys.readouterr().out.split()]
    seq = list(prompt)
    for t in got:
        assert int(torch.argmax(P.forward(w, cfg, seq)[-1])) == t
        seq.append(t)
    assert len(got) == 5


class _Both:
    """(plain logits, plain logits with rounded products) of a request, indexed by position as one."""

    def __init__(self, pair):
        self.pair = pair

    def __getitem__(self, pos):
        return self.pair


@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_replay_with_four_slots_and_a_pool_for_the_live_requests_only(folders, dtype, tmp_path):
    """``bin/trace_run`` on a mixed schedule: nine requests of 20 to 150 tokens, at most four live, portions of some
    beside single tokens of others, some sitting a step out; the pool holds what the live requests hold at the peak, so
    pages and slots are used again; then one request whole, one with its tail decoded, one in portions down to two."""
    from tests.replay_util import Trace, compare, mixed, portions, run_trace, tail_one_by_one, whole

    cfg, w = plain_of(folders["A"])
    rng = np.random.default_rng(17)
    reqs = {f"q{i}": tokens_of(cfg, n, 50 + i) for i, n in enumerate((150, 20, 77, 64, 33, 129, 48, 90, 65))}
    trace = Trace()
    peak = mixed(trace, reqs, rng)
    whole(trace, "q0#w", reqs["q0"])
    tail_one_by_one(trace, "q2#t", reqs["q2"], tail=40)
    portions(trace, "q5#p", reqs["q5"], (2, 31, 3, 17))
    got = run_trace(folders["A"], dtype, trace, max(peak, 192), tmp_path / "out", block_size=SMALL_A["page_size"])
    want = {r: expected(cfg, w, t, dtype) for r, t in reqs.items()}
    rows_got, rows_plain, rows_rounded = [], [], []

    def collect(name, pos, got_row, want_row):
        rows_got.append(got_row)
        if dtype == "float32":
            rows_plain.append(want_row)
        else:
            rows_plain.append(want_row[0][pos])
            rows_rounded.append(want_row[1][pos])

    if dtype == "float32":
        n = compare(trace, got, want, collect)
        check_rows(dtype, np.stack(rows_got), np.stack(rows_plain), "trace")
    else:
        n = compare(trace, got, {r: _Both(v) for r, v in want.items()}, collect)
        check_rows(dtype, np.stack(rows_got), (np.stack(rows_plain), np.stack(rows_rounded)), "trace")
    assert n == sum(len(t) for t in reqs.values()) + 150 + 41 + 129


# ------------------------------------------------------------------ other sizes
@pytest.mark.parametrize("dtype", DTYPES)
def test_odd_sizes_and_heads_beyond_the_matrix_core_kernels(tmp_path, dtype):
    """A width that is no multiple of 4, a cached latent vector of 263 elements (above the matrix-core attention
    kernels: the float kernel runs in bfloat16 too), heads of 6, 10 and 18, seven q heads on one kv head, experts of odd
    sizes in three groups, pages of 24 tokens."""
    small = dict(name="odd", seed=31, std=0.25, norm_std=0.2, config=config(50, 61, [
        layer(latent(2, 10, 6, 7, 11, 257, size=23, rot=(6, 77.0)), moe(9, 2, 13, shared=9, groups=(3, 1))),
        layer(attention(7, 1, 18, 10, size=29, conv=3, rot=(10, 300.0)), None),
        layer(latent(3, 5, 6, 3, 5, 257, size=31, rot=(6, 77.0), kv_from=0), moe(3, 1, 5)),
        layer(attention(3, 3, 6, 270, conv=6), moe(5, 5, 21, shared=63)),
    ], taps=5, logit_scale=1.7))
    folder = make_folder(small, tmp_path)
    cfg, w = plain_of(folder)
    toks = tokens_of(cfg, 90, 8)
    want = expected(cfg, w, toks, dtype)
    core = make_core(folder, dtype, 24)
    check_rows(dtype, run_cut(core, "whole", toks, [90]), want, "whole")
    check_rows(dtype, run_cut(core, "cut", toks, [33, 2, 1, 17, 1, 1, 15, 20]), want, "portions")


@pytest.mark.parametrize("dtype", DTYPES)
def test_wider_layers_and_a_long_prompt(tmp_path, dtype):
    """Six layers at a width of 288 with heads of 32 to 128 and cached vectors of 96 and 192 (the sizes at which the
    matrix-core attention kernels, the matrix-core expert products and the streaming products all run), a prompt of
    420 tokens: whole, in portions that end inside pages, and with a decoded tail."""
    small = dict(name="wide", seed=41, std=0.08, norm_std=0.1, config=config(288, 500, [
        layer(latent(8, 32, 32, 64, 96, 160, scale=0.2, size=100, rot=(32, 5e4), scaling=dict(LONG, original=512)), moe(8, 2, 64, shared=64, groups=(4, 2))),
        layer(attention(8, 2, 64, scale=0.15, size=128), moe(8, 2, 96, shared=192)),
        layer(attention(4, 4, 128, 96, scale=0.1, size=90, conv=2, rot=(64, 1e5)), None),
        layer(latent(4, 64, 32, 32, 64, 160, size=220, rot=(32, 5e4), scaling=dict(LONG, original=512), kv_from=0), moe(16, 4, 64, groups=(8, 2))),
        layer(latent(2, 16, 16, 128, 48, 80, size=64, rot=(8, 1e4)), moe(4, 1, 192)),
        layer(attention(6, 2, 32, 64, conv=4), moe(12, 3, 32, shared=32, groups=(3, 2))),
    ], taps=4, logit_scale=0.7))
    folder = make_folder(small, tmp_path)
    cfg, w = plain_of(folder)
    toks = tokens_of(cfg, 420, 9)
    want = expected(cfg, w, toks, dtype)
    core = make_core(folder, dtype, 16, pages=40)
    whole, cut = run_cut(core, "whole", toks, [420]), run_cut(core, "cut", toks, [100, 31, 2, 64, 33, 7, 129, 14] + [1] * 40)
    if dtype == "bfloat16":
        check_rows(dtype, whole, want, "whole")
        check_rows(dtype, cut, want, "portions and decoding")
        return
    # a few positions are badly conditioned (a close choice between experts, a small output in front of a norm): the
    # plain implementation in float32 is itself off there, so a row may be off by three times that on top of the bound
    own = np.abs(P.forward(P.read_weights(folder, torch.float32), cfg, toks).numpy().astype(np.float64) - want).max(axis=-1)
    scale = float(np.abs(want).max())
    for what, got in (("whole", whole), ("portions and decoding", cut)):
        err = np.abs(got.astype(np.float64) - want).max(axis=-1)
        worst = int((err - 3 * own).argmax())
        assert (err <= 3e-5 * scale + 1e-5 + 3 * own).all(), f"{what}: row {worst} is off by {err[worst]}, plain float32 by {own[worst]}"
        assert np.median(err) <= 1e-5 * scale, f"{what}: median error {np.median(err)}"


# ------------------------------------------------------------------ the kernels alone
def _dev(x, dtype=None):
    return x.to("cuda").to(dtype) if dtype is not None else x.to("cuda")


def _i32(a):
    return _dev(torch.tensor(a, dtype=torch.int32))


BOTH = pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["f32", "bf16"])


def filtered_rows(x, weight, state, lens, slots):
    """(filter of every row in double, the state it leaves): request r's rows continue slots[r]'s state rows."""
    taps = weight.shape[1]
    out, new = [], state.clone()
    at = 0
    for n, s in zip(lens, slots):
        full = torch.cat([state[s].double(), x[at:at + n].double()])
        out.append(sum(full[j:j + n] * weight[:, j].double() for j in range(taps)))
        if taps > 1:
            new[s] = full[full.shape[0] - (taps - 1):].float()
        at += n
    return torch.cat(out), new


@BOTH
@pytest.mark.parametrize("taps", [1, 2, 4, 8])
@pytest.mark.parametrize("channels", [50, 64, 1032])
def test_kernel_input_plus_its_filter(dtype, taps, channels):
    """Five requests of 5, 1, 12, 70 and 3 rows that continue states of their own; the states that the step leaves,
    other slots as they were."""
    from jax_vllm_amd.ops import kernels as K

    g = torch.Generator().manual_seed(1)
    lens, slots = [5, 1, 12, 70, 3], [2, 0, 3, 6, 5]
    x = torch.randn(sum(lens), channels, generator=g).to(dtype)
    weight = torch.randn(channels, taps, generator=g)
    state = torch.randn(8, taps - 1, channels, generator=g).to(dtype).float()
    want, want_state = filtered_rows(x, weight, state, lens, slots)
    st = _dev(state.clone())
    got = K.token_filter(_dev(x), _dev(weight.t().contiguous()), st, _i32(slots), _i32(np.cumsum([0] + lens).tolist()), max(lens))
    tol = 1e-5 if dtype == torch.float32 else 2e-2
    assert torch.allclose(got.double().cpu(), want + x.double(), atol=tol, rtol=tol)
    assert torch.equal(st.cpu(), want_state)


@BOTH
@pytest.mark.parametrize("taps", [1, 3, 4, 8])
@pytest.mark.parametrize("hidden,parts", [(48, 0), (64, 3), (2048, 5), (4096, 2)])
def test_kernel_norms_and_filter_in_one_launch(dtype, taps, hidden, parts):
    """One token a request: the residual step under the sublayer's own norm, the next norm, the filter and its state,
    against the three steps written out; and the first layer's form, where nothing joins the stream."""
    from jax_vllm_amd.ops import kernels as K

    g = torch.Generator().manual_seed(2)
    n, slots = 5, [3, 0, 5, 1, 4]
    h = torch.randn(n, hidden, generator=g)
    y = torch.randn(n, hidden, generator=g).to(dtype)
    stack = torch.randn(parts, n, hidden, generator=g) if parts else None
    wb, wn = torch.rand(hidden, generator=g) + 0.5, torch.rand(hidden, generator=g) + 0.5
    weight = torch.randn(hidden, taps, generator=g)
    state = torch.randn(7, taps - 1, hidden, generator=g).to(dtype).float()
    norm = lambda a, w, eps: a / torch.sqrt((a * a).mean(-1, keepdim=True) + eps) * w.double()      # noqa: E731
    tol = 2e-5 if dtype == torch.float32 else 4e-2
    for pending in (True, False):
        out = y.double() + (stack.double().sum(0) if parts else 0.0)
        new = h.double() + norm(out, wb, 1e-3) if pending else h.double()
        u = norm(new, wn, 1e-5)
        want, want_state = filtered_rows(u.to(dtype), weight, state, [1] * n, slots)
        hd, st = _dev(h.clone()), _dev(state.clone())
        delta = K.PendingNorm(_dev(y), _dev(stack) if parts else None, _dev(wb), 1e-3) if pending else None
        got = K.norm_filter(hd, delta, _dev(wn), 1e-5, _dev(weight.t().contiguous()), st, _i32(slots), dtype)
        assert torch.allclose(hd.double().cpu(), new, atol=1e-5, rtol=1e-5)
        assert torch.allclose(got.double().cpu(), want + u.to(dtype).double(), atol=tol, rtol=tol)
        assert torch.allclose(st.double().cpu(), want_state.double(), atol=tol, rtol=tol)
        assert torch.equal(st[2].cpu(), state[2]) and torch.equal(st[6].cpu(), state[6])


@BOTH
@pytest.mark.parametrize("taps", [None, 1, 4, 7])
@pytest.mark.parametrize("sizes", [(3, 1, 10, 6, 8), (4, 2, 16, 32, 16), (2, 2, 64, 48, 16), (1, 1, 8, 8, 24)])
def test_kernel_filtered_attention_input(dtype, taps, sizes):
    """Prompt portions that begin at any place of a page beside a decoded token: q rows (with their zeros), key pages,
    transposed value pages and the states, with part of the keys turned; one token of each request is not stored."""
    from jax_vllm_amd.ops import kernels as K

    nq, nkv, dk, dv, page = sizes
    g = torch.Generator().manual_seed(3)
    lens, slots, ctx = [37, 1, 6, 90], [2, 0, 3, 4], [5, 77, 16, 8]
    n, dims = sum(lens), dk - 2 if dk > 8 else dk
    dp = K.padded_head_dim(dk, dv)
    channels = (nq + nkv) * dk + nkv * dv
    rows = torch.randn(n, channels + 8 + (-channels) % 8, generator=g).to(dtype)
    weight = torch.randn(channels, taps, generator=g) if taps else None
    state = torch.randn(6, (taps or 1) - 1, channels, generator=g).to(dtype).float()
    x = rows[:, :channels]
    y, want_state = filtered_rows(x, weight, state, lens, slots) if taps else (x.double(), state)
    positions = torch.cat([torch.arange(c, c + m) for c, m in zip(ctx, lens)])
    table, nxt, slot_map = [], 1, []
    for c, m in zip(ctx, lens):
        pages = list(range(nxt, nxt + -(-(c + m) // page)))
        nxt += len(pages)
        slot_map += [pages[p // page] * page + p % page for p in range(c, c + m)]
    slot_map[3] = slot_map[60] = -1
    kf = 100.0 ** (-torch.arange(0, dims, 2).double() / dims)
    vf = 30.0 ** (-torch.arange(0, dv, 2).double() / dv)
    k_cs = K.rope_table(_i32(positions.tolist()), _dev(kf.float()))
    v_cs = K.rope_table(_i32(positions.tolist()), _dev(vf.float()))
    kp = torch.zeros(nxt, nkv, page, dp, dtype=dtype, device="cuda")
    vp = torch.zeros(nxt, nkv, dp, page, dtype=dtype, device="cuda")
    st = _dev(state.clone())
    q = K.attn_prepare_filtered(_dev(rows), _dev(weight.t().contiguous()) if taps else None, st, _i32(slots),
                                _i32(np.cumsum([0] + lens).tolist()), _i32(ctx), max(lens), k_cs, dims, v_cs, _i32(slot_map), kp, vp,
                                page, nq, nkv, dk, dv, dp)
    want_q = P.turn_pairs(y[:, :nq * dk].reshape(n, nq, dk), positions.double().view(-1, 1) * kf)
    want_k = P.turn_pairs(y[:, nq * dk:(nq + nkv) * dk].reshape(n, nkv, dk), positions.double().view(-1, 1) * kf)
    want_v = P.turn_pairs(y[:, (nq + nkv) * dk:].reshape(n, nkv, dv), positions.double().view(-1, 1) * vf)
    tol = 5e-5 if dtype == torch.float32 else 4e-2
    got_q = q.double().cpu().view(n, nq, dp)
    assert torch.allclose(got_q[..., :dk], want_q, atol=tol, rtol=tol) and not got_q[..., dk:].any()
    sm = torch.tensor(slot_map)
    keep = sm >= 0
    pg, off = (sm // page)[keep], (sm % page)[keep]
    kc, vc = kp.double().cpu(), vp.double().cpu()
    assert torch.allclose(kc[pg, :, off, :dk], want_k[keep], atol=tol, rtol=tol)
    assert torch.allclose(vc[pg, :, :dv, off], want_v[keep], atol=tol, rtol=tol)
    # nothing else was written: pads, other slots, the null page, other states
    kc[pg, :, off, :dk] = 0
    vc[pg, :, :dv, off] = 0
    assert not kc.any() and not vc.any()
    assert torch.equal(st.cpu(), want_state)


@BOTH
@pytest.mark.parametrize("heads,dv,dp", [(3, 6, 16), (2, 64, 64), (5, 40, 48)])
def test_kernel_results_turned_back_under_a_gate(dtype, heads, dv, dp):
    from jax_vllm_amd.ops import kernels as K

    g = torch.Generator().manual_seed(4)
    n = 23
    o = torch.randn(n, heads * dp, generator=g).to(dtype)
    gates = torch.randn(n, heads * dv + 16, generator=g).to(dtype)
    positions = torch.randint(0, 300, (n,), generator=g)
    f = 50.0 ** (-torch.arange(0, dv, 2).double() / dv)
    cs = K.rope_table(_i32(positions.tolist()), _dev(f.float()))
    back = P.turn_pairs(o.double().view(n, heads, dp)[..., :dv], -positions.double().view(-1, 1) * f)
    gate = torch.sigmoid(gates.double()[:, 8:8 + heads * dv]).view(n, heads, dv)
    tol = 2e-4 if dtype == torch.float32 else 3e-2
    for use_gate, use_turn in ((True, True), (False, True), (True, False)):
        got = _dev(o.clone())
        K.rotate_back_gate(got, _dev(gates)[:, 8:8 + heads * dv] if use_gate else None, cs if use_turn else None, heads, dv, dp)
        got = got.double().cpu().view(n, heads, dp)
        want = (back if use_turn else o.double().view(n, heads, dp)[..., :dv]) * (gate if use_gate else 1.0)
        assert torch.allclose(got[..., :dv], want, atol=tol, rtol=tol)
        assert torch.equal(got[..., dv:], o.double().view(n, heads, dp)[..., dv:])


@BOTH
@pytest.mark.parametrize("head_dim", [40, 64, 160])
@pytest.mark.parametrize("window,chunk", [(None, 33), (None, 64), (None, 500), (50, None), (1, None), (None, 1)])
def test_kernel_attention_in_blocks_and_windows(dtype, head_dim, window, chunk):
    """Prompt portions and single tokens of three requests over a paged cache (the page tables of keys that nobody sees
    hold the null page): the float kernel, and in bfloat16 the matrix-core kernels for prompts and for decoded tokens."""
    from jax_vllm_amd.parts import attention_backend
    from jax_vllm_amd.parts.spec import LayerMemory, StepContext

    g = torch.Generator().manual_seed(5)
    nq, nkv, page, D = 4, 2, 16, head_dim
    first_of = lambda p: p - p % chunk if chunk else max(0, p - window + 1)      # noqa: E731
    for q_lens, ctx_lens in (([150, 5, 1], [0, 120, 700]), ([1, 1, 1], [3, 900, 64])):
        R, n = len(q_lens), sum(q_lens)
        total = [c + q for c, q in zip(ctx_lens, q_lens)]
        width = max(-(-t // page) for t in total)
        tables = torch.zeros(R, width, dtype=torch.int32)
        nxt = 1
        for r, t in enumerate(total):
            for p in range(first_of(ctx_lens[r]) // page, -(-t // page)):
                tables[r, p] = nxt
                nxt += 1
        kp = (torch.randn(nxt, nkv, page, D, generator=g) * 0.5).to(dtype)
        vp = torch.randn(nxt, nkv, D, page, generator=g).to(dtype)
        kp[0] = vp[0] = 0
        q = (torch.randn(n, nq * D, generator=g) * 0.5).to(dtype)
        scale = 0.3
        want = torch.empty(n, nq, D, dtype=torch.float64)
        cu = np.cumsum([0] + q_lens)
        positions, token_req = [], []
        for r in range(R):
            kk = kp.double()[tables[r].long()].permute(0, 2, 1, 3).reshape(-1, nkv, D)
            vv = vp.double()[tables[r].long()].permute(0, 3, 1, 2).reshape(-1, nkv, D)
            for i in range(q_lens[r]):
                pos = ctx_lens[r] + i
                positions.append(pos)
                token_req.append(r)
                lo = first_of(pos)
                for h in range(nq):
                    s = (kk[lo:pos + 1, h // (nq // nkv)] @ q[cu[r] + i].double().view(nq, D)[h]) * scale
                    p = torch.exp(s) / (1 + torch.exp(s).sum())
                    want[cu[r] + i, h] = p @ vv[lo:pos + 1, h // (nq // nkv)]
        ctx = StepContext(num_tokens=n, num_requests=R, positions=_i32(positions), token_req=_i32(token_req), cu_seqlens=_i32(cu.tolist()),
                          context_lens=_i32(ctx_lens), slot_ids=_i32([0] * R), block_tables=[_dev(tables)], slot_mappings=[None],
                          page_size=page, q_lens_host=q_lens, context_lens_host=ctx_lens, slot_ids_host=[0] * R,
                          max_q_len=max(q_lens), max_kv_len=max(total))
        att = SimpleNamespace(nq=nq, nkv=nkv, d=D, scale=scale, window=window, chunk=chunk, q_row_stride=nq * D,
                              sinks=torch.zeros(nq, device="cuda"))
        out = torch.empty(n, nq * D, dtype=dtype, device="cuda")
        attention_backend.run(att, out, _dev(q), ctx, LayerMemory(pages={"k": _dev(kp), "v": _dev(vp)}, group=0))
        tol = 2e-5 if dtype == torch.float32 else 3e-2
        assert float((out.double().cpu().view(n, nq, D) - want).abs().max()) <= tol * max(1.0, float(want.abs().max()))


@BOTH
@pytest.mark.parametrize("n", [1, 5, 40, 300])
@pytest.mark.parametrize("experts,top,groups", [(9, 3, None), (12, 3, (4, 2)), (80, 5, (16, 3)), (6, 2, (6, 2)), (8, 4, (2, 1)), (192, 6, (64, 2))])
def test_kernel_router_over_groups_with_the_softmax_over_all(dtype, n, experts, top, groups):
    from jax_vllm_amd.ops import kernels as K

    g = torch.Generator().manual_seed(6)
    hidden = 48
    x = torch.randn(n, hidden, generator=g).to(dtype)
    wr = (torch.randn(experts, hidden, generator=g) * 0.3).to(dtype)
    z = x.double() @ wr.double().T
    f = {"router": {"experts": experts, "top": top}}
    if groups:
        f["router"]["groups"] = {"count": groups[0], "keep": groups[1]}
    choice, weight = P.router({"router": wr.double()}, "", f, x.double())
    plan = K.moe_route(None, top, x=_dev(x), w_router=_dev(wr), score="softmax", groups=groups)
    ids, wts = plan.ids.view(n, top).cpu().long(), plan.weights.view(n, top).cpu().double()
    # rows whose choices are no close calls: of experts and of groups
    best = z.view(n, groups[0], -1).amax(-1).sort(-1, descending=True).values if groups else None
    clear = torch.ones(n, dtype=torch.bool)
    if groups and groups[1] < groups[0]:
        clear &= (best[:, groups[1] - 1] - best[:, groups[1]]) > 1e-4
    gaps = z.sort(-1, descending=True).values
    clear &= (gaps[:, :-1] - gaps[:, 1:]).amin(-1) > 1e-5
    assert n < 40 or clear.float().mean() > 0.5
    assert torch.equal(ids[clear], choice[clear])           # in descending order of their scores
    assert torch.allclose(wts[clear], weight[clear], atol=1e-6, rtol=1e-4)
    # the grouping holds every entry once, under its expert
    order, offsets = plan.order.cpu().long(), plan.offsets.cpu().long()
    flat = ids.reshape(-1)
    assert sorted(order.tolist()) == list(range(n * top))
    for e in range(experts):
        assert (flat[order[offsets[e]:offsets[e + 1]]] == e).all()


@BOTH
@pytest.mark.parametrize("n", [1, 7, 33, 200])
@pytest.mark.parametrize("hidden,ff", [(64, 32), (40, 24), (50, 13), (512, 192)])
def test_kernel_experts_without_a_gate(dtype, n, hidden, ff):
    from jax_vllm_amd.ops import kernels as K

    g = torch.Generator().manual_seed(7)
    experts, top = 5, 2
    x = torch.randn(n, hidden, generator=g).to(dtype)
    up = (torch.randn(experts, ff, hidden, generator=g) * hidden ** -0.5).to(dtype)
    down = (torch.randn(experts, hidden, ff, generator=g) * ff ** -0.5).to(dtype)
    logits = torch.randn(n, experts, generator=g)
    plan = K.moe_route(_dev(logits), top, score="softmax", tile_rows=K.moe_tile_rows_for(dtype, hidden, ff, n * top, experts))
    out = torch.empty(top, n, hidden, device="cuda")
    K.moe_experts(_dev(x), plan, None, _dev(up), _dev(down), "relu2", out, weight_on_input=False)
    ids, wts = plan.ids.view(n, top).cpu().long(), plan.weights.view(n, top).cpu().double()
    want = torch.empty(top, n, hidden, dtype=torch.float64)
    for t in range(n):
        for k in range(top):
            z = torch.relu(up[ids[t, k]].double() @ x[t].double()) ** 2
            want[k, t] = wts[t, k] * (down[ids[t, k]].double() @ z)
    tol = 1e-5 if dtype == torch.float32 else 2e-2
    assert float((out.double().cpu() - want).abs().max()) <= tol * float(want.abs().max())


@pytest.mark.parametrize("gated", [False, True], ids=["plain", "gated"])
@pytest.mark.parametrize("n", [1, 3, 16, 40])
@pytest.mark.parametrize("hidden,ff,experts,top", [(64, 32, 5, 2), (40, 24, 8, 3), (2048, 328, 6, 2), (520, 1544, 4, 1)])
def test_kernel_experts_streamed_for_few_tokens(gated, n, hidden, ff, experts, top):
    """Tiles of 16 rows (one expert gets more than a tile): the weights streamed, the inner size shared out to the waves."""
    from jax_vllm_amd.ops import kernels as K

    g = torch.Generator().manual_seed(17)
    bf = torch.bfloat16
    x = torch.randn(n, hidden, generator=g).to(bf)
    gate, up = ((torch.randn(experts, ff, hidden, generator=g) * hidden ** -0.5).to(bf) for _ in range(2))
    down = (torch.randn(experts, hidden, ff, generator=g) * ff ** -0.5).to(bf)
    logits = torch.randn(n, experts, generator=g)
    logits[:, 1] += 3.0
    for on_input in (False, True):
        plan = K.moe_route(_dev(logits), top, score="softmax", tile_rows=16)
        out = torch.empty(top, n, hidden, device="cuda")
        K.moe_experts(_dev(x), plan, _dev(gate) if gated else None, _dev(up), _dev(down), "silu" if gated else "relu2", out, on_input)
        ids, wts = plan.ids.view(n, top).cpu().long(), plan.weights.view(n, top).cpu().double()
        want = torch.empty(top, n, hidden, dtype=torch.float64)
        for t in range(n):
            for k in range(top):
                e, w = ids[t, k], wts[t, k]
                u = up[e].double() @ x[t].double() * (w if on_input else 1.0)
                q = gate[e].double() @ x[t].double() * (w if on_input else 1.0)
                z = torch.nn.functional.silu(q) * u if gated else torch.relu(u) ** 2
                want[k, t] = (1.0 if on_input else w) * (down[e].double() @ z)
        assert float((out.double().cpu() - want).abs().max()) <= 2e-2 * float(want.abs().max())


@pytest.mark.parametrize("n,experts,top,always,groups", [(1, 4, 1, 1, None), (8, 70, 3, 2, (7, 3)), (16, 9, 4, 3, None), (64, 130, 2, 0, (2, 1))])
def test_kernel_router_and_grouping_in_one_launch(n, experts, top, always, groups):
    """Every token has its chosen experts and the ones behind the routed experts; the grouping by experts and tiles; the logits as
    partial sums."""
    from jax_vllm_amd.ops import kernels as K

    g = torch.Generator().manual_seed(18)
    stack = torch.randn(11, n, experts, generator=g)
    logits = stack[0]
    for part in stack[1:]:
        logits = logits + part
    plan = K.moe_route(_dev(stack), top, score="softmax", groups=groups, always=always, tile_rows=16)
    per = top + always
    assert plan.top == per
    ids, wts = plan.ids.view(n, per).cpu().long(), plan.weights.view(n, per).cpu().double()
    f = {"router": {"experts": experts, "top": top}}
    if groups:
        f["router"]["groups"] = {"count": groups[0], "keep": groups[1]}
    choice, weight = P.router({"router": torch.eye(experts, dtype=torch.float64)}, "", f, logits.double())
    assert torch.equal(ids[:, :top], choice) and torch.allclose(wts[:, :top], weight, atol=1e-6)
    assert torch.equal(ids[:, top:], torch.arange(experts, experts + always).expand(n, always)) and (wts[:, top:] == 1).all()
    order, offsets, flat = plan.order.cpu().long(), plan.offsets.cpu().long(), ids.reshape(-1)
    assert sorted(order.tolist()) == list(range(n * per)) and int(offsets[-1]) == n * per
    tiles = []
    for e in range(experts + always):
        lo, hi = int(offsets[e]), int(offsets[e + 1])
        assert (flat[order[lo:hi]] == e).all()
        tiles += [(e, r) for r in range(lo, hi, 16)]
    m = int(plan.meta.cpu()[0])
    assert m == len(tiles) <= plan.max_tiles
    assert list(zip(plan.tile_expert.cpu()[:m].tolist(), plan.tile_row0.cpu()[:m].tolist())) == tiles


@BOTH
def test_kernel_query_latent_alone(dtype):
    """A layer that reads another layer's cache norms its query latent and stores nothing."""
    from jax_vllm_amd.ops import kernels as K

    g = torch.Generator().manual_seed(8)
    rows, weight = torch.randn(9, 24 + 8, generator=g).to(dtype), torch.rand(24, generator=g) + 0.5
    got = K.latent_prepare(_dev(rows), 24, 0, 0, 0, _dev(weight), None, 1e-5, None, None, None, None, 8)
    x = rows.double()[:, :24]
    want = x / torch.sqrt((x * x).mean(-1, keepdim=True) + 1e-5) * weight.double()
    tol = 1e-5 if dtype == torch.float32 else 2e-2
    assert torch.allclose(got.double().cpu(), want, atol=tol, rtol=tol)


@BOTH
def test_kernel_square_of_relu(dtype):
    from jax_vllm_amd.ops import kernels as K

    for rows, cols in ((5, 13), (300, 64), (3, 2056)):
        z = torch.randn(rows, cols, generator=torch.Generator().manual_seed(9)).to(dtype)
        bias = torch.linspace(-1, 1, cols)
        for b in (None, bias):
            y = _dev(z.clone())
            K.bias_act(y, _dev(b) if b is not None else None, "relu2")
            want = torch.relu(z.double() + (b.double() if b is not None else 0.0)) ** 2
            assert torch.allclose(y.double().cpu(), want, atol=1e-6 if dtype == torch.float32 else 1e-2, rtol=1e-5 if dtype == torch.float32 else 1e-2)
