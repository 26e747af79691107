"""Kuditar on the GPU against its plain implementation (``tests/plain/kuditar_plain.py``): each mechanism alone, whole
prompts against portions and token-by-token decoding, unequal requests in one batch against each alone, pages and slots
that are used again, keys just inside and just outside windows, blocks and the first tokens that a window keeps, in prompts
and in decoding, one far key among hundreds, values blended with those of an earlier layer, sinks, capped scores, states that
a portion hands on, choices of experts that the correction changes, long decoding through recorded steps, sizes that are no
multiples of anything, greedy generation through the entry point and its scheduler, and the kernels alone."""
from types import SimpleNamespace

import numpy as np
import pytest
import torch

from tests.kuditar_util import (ALL_SMALL, SMALL_A, SMALL_B, SMALL_C, attention, block_side, check_rows, config, delta_side, dense,
                                expected, layer, linear_side, make_folder, moe, parallel, parallel_2, plain_logits, plain_of,
                                tokens_of, window_side)
from tests.plain import kuditar_plain as P

pytestmark = pytest.mark.gpu
DTYPES = ["float32", "bfloat16"]


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    return {s["name"]: make_folder(s, tmp_path_factory.mktemp(f"ku{s['name']}")) for s in ALL_SMALL}


def entry(rid, tokens, want=None):
    from jax_vllm_amd.engine.entries import StepEntry

    return StepEntry(rid, tokens, range(len(tokens)) if want is None else want)


def make_core(folder, dtype, page_size, pages=64, seqs=4, graphs=False):
    from jax_vllm_amd.config import EngineConfig
    from jax_vllm_amd.engine.core import EngineCore
    from jax_vllm_amd.weights import load_model

    model, _ = load_model(folder, dtype, "cuda", strict=True)
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
TINY = attention(1, 1, 4)                                  # the smallest mixer, beside what is under test
TINY_LEFT, TINY_DELTA, TINY_LINEAR = window_side(1, 1, 4), delta_side(1, 1, 4, 4, conv=1), linear_side(1, 4, 4, rank=1)
TINY_BLOCK = block_side(1, 1, 4)
ALONE = {
    "attention": dict(layers=[layer(TINY)]),
    "constant_on_the_embedding": dict(layers=[layer(TINY)], scale=0.3),
    "part_of_a_head_turned": dict(layers=[layer(attention(3, 3, 16, rot=(6, 200.0)))]),
    "frequencies_under_a_factor": dict(layers=[layer(attention(2, 1, 8, rot=(8, 50.0), factor=4.0))]),
    "values_wider_than_keys": dict(layers=[layer(attention(4, 2, 8, 24, scale=0.7))]),
    "values_narrower_than_keys": dict(layers=[layer(attention(4, 1, 24, 6))]),
    "capped_scores": dict(layers=[layer(attention(2, 2, 16, scale=1.0, softcap=1.5))]),
    "blended_values": dict(layers=[layer(attention(2, 2, 8, 12, v_mix=True)), layer(TINY), layer(attention(4, 2, 16, 12, v_mix=True)),
                                   layer(attention(2, 2, 4, 12, v_mix=False)), layer(attention(6, 2, 6, 12, v_mix=True))]),
    "window": dict(layers=[layer(parallel(window_side(4, 2, 8, size=7), TINY_DELTA))]),
    "window_of_one": dict(layers=[layer(parallel(window_side(2, 1, 8, size=1), TINY_DELTA))]),
    "window_that_keeps_one": dict(layers=[layer(parallel(window_side(2, 2, 8, size=6, keep=1), TINY_DELTA))]),
    "window_that_keeps_more_than_a_page": dict(layers=[layer(parallel(window_side(2, 1, 8, 20, size=5, keep=19, rot=(4, 90.0)), TINY_DELTA))]),
    "window_that_keeps_more_than_there_is": dict(layers=[layer(parallel(window_side(2, 1, 8, size=4, keep=100, softcap=3.0), TINY_DELTA))]),
    "norm_per_head_before_the_rotation": dict(layers=[layer(parallel(window_side(3, 1, 12, 8, rot=(12, 30.0), scale=0.6), TINY_DELTA))]),
    "delta_rule": dict(layers=[layer(parallel(TINY_LEFT, delta_side(4, 2, 12, 8)))]),
    "delta_rule_of_one_tap": dict(layers=[layer(parallel(TINY_LEFT, delta_side(2, 2, 8, 20, conv=1)))]),
    "delta_rule_of_eight_taps": dict(layers=[layer(parallel(TINY_LEFT, delta_side(3, 1, 16, 16, conv=8)))]),
    "blocks": dict(layers=[layer(parallel_2(block_side(4, 2, 8, 12, size=12), TINY_LINEAR))]),
    "blocks_of_one": dict(layers=[layer(parallel_2(block_side(2, 1, 8, size=1), TINY_LINEAR))]),
    "gated_linear_attention": dict(layers=[layer(parallel_2(TINY_BLOCK, linear_side(3, 12, 20, tau=2.0, rank=5)))]),
    "gated_linear_attention_with_fast_decay": dict(layers=[layer(parallel_2(TINY_BLOCK, linear_side(2, 16, 8, tau=0.02, rank=8)))]),
    "clamped_feed_forward": dict(layers=[layer(TINY, dense(24, limit=0.3))]),
    "feed_forward_hardly_clamped": dict(layers=[layer(TINY, dense(13, limit=50.0))]),
    "experts": dict(layers=[layer(TINY, moe(7, 3, 24, limit=0.4, scale=2.5))]),
    "experts_one_chosen": dict(layers=[layer(TINY, moe(4, 1, 10))]),
    "experts_all_chosen": dict(layers=[layer(TINY, moe(3, 3, 16, scale=0.5))]),
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
    """The first tokens see convolutions whose further taps lie before the sequence, a state of zeros and few keys beside
    the sinks: prompts of one to nine tokens in every cut."""
    cfg, w = plain_of(folders[small["name"]])
    toks = [5, 1, 9, 2, 7, 30, 8, 8, 4]
    want = expected(cfg, w, toks, dtype)
    core = make_core(folders[small["name"]], dtype, small["page_size"])
    for rid, cuts in (("one", [1] * 9), ("two", [1, 2, 2, 2, 2]), ("three", [3, 2, 4]), ("whole", [9]), ("late", [8, 1])):
        check_rows(dtype, run_cut(core, rid, toks, cuts), want, rid)


@pytest.mark.parametrize("small", ALL_SMALL, ids=[s["name"] for s in ALL_SMALL])
def test_the_stream_after_every_layer(folders, small):
    """Layer by layer in float32: the stream that every block leaves, with what it still owes it added."""
    from jax_vllm_amd.ops import kernels as K

    cfg, w = plain_of(folders[small["name"]])
    toks = tokens_of(cfg, 40, 3)
    want = []
    P.forward(w, cfg, toks, want)
    core = make_core(folders[small["name"]], "float32", small["page_size"])
    got = []
    for block in (l.block for l in core.model.layers):
        def hooked(h, delta, *rest, forward=block.forward):
            owed = forward(h, delta, *rest)
            stream = h.clone()
            one = torch.ones(h.shape[1], device="cuda")
            K.add_layernorm(stream, owed, one, torch.zeros_like(one), 1e-5, torch.empty_like(h))
            got.append(stream.cpu())
            return owed
        block.forward = hooked
    run_cut(core, "a", toks, [40])
    assert len(got) == len(want)
    for i, (a, b) in enumerate(zip(got, want)):
        assert float((a - b).abs().max()) <= 3e-5 * float(b.abs().max()), f"layer {i}"


# ------------------------------------------------------------------ windows, blocks, kept first tokens
def edge_model(tmp_path, kind, size, keep=None, scale=0.8):
    """One layer whose recurrent side has no weight, with scores of several units: single keys stand out."""
    if kind == "blocks":
        mixer = parallel_2(block_side(4, 2, 16, 16, scale=scale, size=size), TINY_LINEAR)
    else:
        mixer = parallel(window_side(4, 2, 16, 16, scale=scale, size=size, keep=keep, softcap=30.0), TINY_DELTA)
    small = dict(name="edge", seed=23, std=0.35, norm_std=0.1, config=config(32, 50, [layer(mixer)]))
    patch = {"l0.mix.right.out": 0.0}
    if kind == "window":
        patch["l0.mix.left.sink"] = -4.0
    folder = make_folder(small, tmp_path, patch)
    return folder, *plain_of(folder)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind,size,keep", [("window", 16, None), ("window", 37, 5), ("window", 64, 16), ("window", 20, 45),
                                            ("blocks", 16, None), ("blocks", 37, None), ("blocks", 64, None)])
def test_keys_just_inside_and_just_outside(tmp_path, dtype, kind, size, keep):
    """One key more or less at an edge (of the window or block, of the kept first tokens) moves many rows by much on the
    plain implementation.  Whole prompts, portions that end at, one before and one behind edges of blocks, windows, kept
    tokens and pages, and decoding across them."""
    folder, cfg, w = edge_model(tmp_path, kind, size, keep)
    n = 150
    toks = tokens_of(cfg, n, 12)
    plain = plain_logits(cfg, w, toks)
    i, j = torch.arange(n).view(n, 1), torch.arange(n).view(1, n)
    if kind == "blocks":
        seen, first = P.visible_chunk(n, size), i - i % size
    else:
        seen, first = P.visible_window(n, size, keep or 0), torch.clamp(i - size + 1, min=0)
    masks = [seen & ~((j == first) & (j < i)), seen | ((j == first - 1) & (first > 0))]
    if keep:
        masks += [seen & ~((j == keep - 1) & (j < first)), seen | ((j == keep) & (j < first))]
    for mask in masks:
        moved = np.abs(plain_logits(cfg, w, toks, masks={0: mask}) - plain).max(axis=-1)
        assert (moved > 0.005 * np.abs(plain).max()).mean() > 0.15
    want = expected(cfg, w, toks, dtype)
    core = make_core(folder, dtype, 16, pages=12)
    check_rows(dtype, run_cut(core, "whole", toks, [n]), want, "whole")
    check_rows(dtype, run_cut(core, "decoded", toks, [size - 1] + [1] * (n - size + 1)), want, "decoded across every edge")
    check_rows(dtype, run_cut(core, "cut", toks, [15, 1, 1, 15, 4, 2, 7, 1, 18, 1, 64, 21]), want, "portions")
    assert core.cache.num_free_pages(0) == 12       # every page came back


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["blocks", "window"])
def test_one_far_key_among_hundreds_and_page_borders(tmp_path, dtype, kind):
    """Blocks and windows of 400 (the window keeps 20 tokens): rows change by much when the plain implementation is kept
    from seeing keys more than 150 back.  500 tokens over 32 pages: whole, in portions that end at, one before and one after
    page borders, with the last 60 decoded; pages out of sight go back."""
    keep = 20 if kind == "window" else None
    folder, cfg, w = edge_model(tmp_path, kind, 400, keep, scale=0.6)
    n = 500
    toks = tokens_of(cfg, n, 13)
    want = expected(cfg, w, toks, dtype)
    plain = plain_logits(cfg, w, toks)
    seen = P.visible_chunk(n, 400) if kind == "blocks" else P.visible_window(n, 400, keep)
    near = plain_logits(cfg, w, toks, masks={0: seen & P.visible_window(n, 150)})
    assert np.median(np.abs(near[200:400] - plain[200:400]).max(axis=-1)) > 0.01 * np.abs(plain).max()
    if keep:
        lost = plain_logits(cfg, w, toks, masks={0: P.visible_window(n, 400)})
        assert np.median(np.abs(lost[430:] - plain[430:]).max(axis=-1)) > 0.005 * np.abs(plain).max()
    core = make_core(folder, dtype, 16, pages=32)
    check_rows(dtype, run_cut(core, "whole", toks, [n]), want, "whole")
    core.start_request("again")
    got, at = [], 0
    for m in [64, 63, 1, 17, 47, 2, 66, 139, 1, 40] + [1] * 60:
        got.append(core.run([entry("again", toks[at:at + m])]).cpu().numpy())
        at += m
        held = [i for i, t in enumerate(core.cache.block_table("again", 0)) if t]
        lo = at - at % 400 if kind == "blocks" else max(0, at - 399)
        assert held == [i for i in range(-(-at // 16)) if 16 * (i + 1) > lo or (keep and i < 2)]
    assert at == n
    core.finish_request("again")
    check_rows(dtype, np.concatenate(got), want, "portions and decoding")
    assert core.cache.num_free_pages(0) == 32


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_far_key_of_the_attention_over_all_keys(tmp_path, dtype):
    """Scores of several units under a cap over 500 keys: the key that weighs most is often hundreds back."""
    small = dict(name="far", seed=27, std=0.35, norm_std=0.1, config=config(32, 50, [
        layer(attention(4, 2, 16, 24, scale=0.6, softcap=20.0, rot=(8, 1e5), factor=2.5, v_mix=True)),
        layer(attention(2, 2, 32, 24, scale=0.4, softcap=9.0, v_mix=True))]))
    folder = make_folder(small, tmp_path)
    cfg, w = plain_of(folder)
    n = 500
    toks = tokens_of(cfg, n, 13)
    plain = plain_logits(cfg, w, toks)
    near = plain_logits(cfg, w, toks, masks={0: P.visible_window(n, 150), 1: P.visible_window(n, 150)})
    assert np.median(np.abs(near[300:] - plain[300:]).max(axis=-1)) > 0.02 * np.abs(plain).max()
    want = expected(cfg, w, toks, dtype)
    core = make_core(folder, dtype, 16, pages=32)
    check_rows(dtype, run_cut(core, "whole", toks, [n]), want, "whole")
    check_rows(dtype, run_cut(core, "cut", toks, [64, 63, 1, 17, 47, 2, 66, 139, 1, 40] + [1] * 60), want, "portions and decoding")


# ------------------------------------------------------------------ batches, pages and slots used again
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("small", ALL_SMALL, ids=[s["name"] for s in ALL_SMALL])
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
    implementation's argmax; in bfloat16 nearly all tokens are within a margin of the plain maximum given what came before
    (rounding turns a close choice between experts in a few rows of these models, in the plain implementation too)."""
    from jax_vllm_amd import LLM, SamplingParams

    small = {"A": SMALL_A, "C": SMALL_C}[which]
    cfg, w = plain_of(folders[which])
    prompts = [tokens_of(cfg, n, 30 + n) for n in (3, 41, 18, 70)]
    llm = LLM(folders[which], dtype=dtype, block_size=small["page_size"], max_num_seqs=2, max_model_len=128,
              max_num_batched_tokens=24, num_blocks=max(9, 256 // small["page_size"] + 1))
    assert llm.prewarm() > 0.0
    got = llm.generate(prompts, SamplingParams(max_new_tokens=12))
    assert [len(g) for g in got] == [12] * 4
    below = []
    for p, g in zip(prompts, got):
        seq = list(p)
        for i, t in enumerate(g):
            logits = P.forward(w, cfg, seq)[-1]
            if dtype == "float32":
                assert int(torch.argmax(logits)) == t, f"token {i}: engine {t}, plain {int(torch.argmax(logits))}"
            below.append(float(logits.max() - logits[t]) / float(logits.abs().max()))
            seq.append(t)
    assert sum(b > 0.06 for b in below) <= 4 and np.median(below) <= 0.005, sorted(below)[-6:]


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
    """A width that is no multiple of 4, a value head above the matrix-core attention kernels (the float kernel runs in
    bfloat16 too), heads of 6, 10 and 18, seven q heads on one kv head, experts of odd sizes, recurrent heads of 130 keys
    (token by token), pages of 24 tokens."""
    small = dict(name="odd", seed=31, std=0.25, norm_std=0.2, config=config(50, 61, [
        layer(attention(3, 3, 6, 270, scale=0.5, softcap=2.0, v_mix=True), moe(9, 2, 13, scale=1.1)),
        layer(parallel(window_side(7, 1, 18, 10, rot=(10, 300.0), size=29, keep=26), delta_side(3, 1, 130, 5, conv=3)), None),
        layer(parallel_2(block_side(3, 3, 10, 6, size=31), linear_side(1, 130, 9, tau=3.0, rank=7)), moe(3, 1, 5, limit=0.2)),
        layer(attention(6, 3, 10, 270, rot=(10, 77.0), v_mix=True), dense(63, limit=0.7)),
    ], scale=1.3))
    folder = make_folder(small, tmp_path)
    cfg, w = plain_of(folder)
    toks = tokens_of(cfg, 90, 8)
    want = expected(cfg, w, toks, dtype)
    core = make_core(folder, dtype, 24)
    check_rows(dtype, run_cut(core, "whole", toks, [90]), want, "whole")
    check_rows(dtype, run_cut(core, "cut", toks, [33, 2, 1, 17, 1, 1, 15, 20]), want, "portions")


@pytest.mark.parametrize("dtype", DTYPES)
def test_wider_layers_and_a_long_prompt(tmp_path, dtype):
    """Six layers at a width of 288 with heads of 32 to 128 (the sizes at which the matrix-core attention kernels, the
    matrix-core expert products and the streaming products all run, and the attention inputs of many tokens take 16 bytes a
    lane), a prompt of 420 tokens: whole, in portions that end inside pages, and with a decoded tail."""
    small = dict(name="wide", seed=41, std=0.08, norm_std=0.1, config=config(288, 500, [
        layer(parallel_2(block_side(8, 2, 64, scale=0.2, size=128), linear_side(4, 64, 96, tau=8.0, rank=24)), moe(8, 2, 64, limit=0.5, scale=1.4)),
        layer(attention(8, 4, 32, 64, scale=0.6, rot=(32, 5e4), factor=4.0, softcap=4.0, v_mix=True), dense(448, limit=0.5)),
        layer(parallel(window_side(4, 2, 128, 96, scale=0.1, rot=(64, 1e5), softcap=15.0, size=90, keep=33), delta_side(4, 2, 64, 128, conv=4)), None),
        layer(parallel(window_side(6, 6, 64, 64, scale=0.3, rot=(64, 1e5), size=64, keep=4), delta_side(2, 2, 32, 64, conv=2)), moe(16, 4, 64)),
        layer(attention(4, 4, 128, 64, scale=0.1, v_mix=True), moe(4, 1, 192, scale=0.7)),
        layer(parallel_2(block_side(6, 2, 32, 64, size=100), linear_side(2, 128, 64, tau=16.0, rank=8)), dense(96)),
    ], scale=3.5))
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


@BOTH
@pytest.mark.parametrize("n,hidden", [(3, 48), (3, 50), (70, 1536), (5, 2048), (66, 4096), (2, 5000), (65, 1024)])
def test_kernel_layer_norm_with_the_residual_step(dtype, n, hidden):
    """Nothing, rows, a float stack, both, an output under a constant, an output under its norm, and two outputs under norms of
    their own join the stream; then selected rows, which leave the stream alone.  The stream has a mean far from zero."""
    from jax_vllm_amd.ops import kernels as K

    g = torch.Generator().manual_seed(1)
    h = torch.randn(n, hidden, generator=g) + 20.0
    rows = torch.randn(n, hidden, generator=g).to(dtype)
    stack = torch.randn(6, n, hidden, generator=g)
    w, b, wa, wb = (torch.randn(hidden, generator=g) for _ in range(4))
    rms = lambda y, eps: y / torch.sqrt((y * y).mean(-1, keepdim=True) + eps)      # noqa: E731
    r64, s64 = rows.double(), stack.double()
    cases = {
        "nothing": (lambda: None, 0.0),
        "rows": (lambda: _dev(rows), r64),
        "stack": (lambda: _dev(stack[:3]), s64[:3].sum(0)),
        "both": (lambda: (_dev(rows), _dev(stack)), r64 + s64.sum(0)),
        "constant": (lambda: K.pending_scale((_dev(rows), _dev(stack[:1])), 0.3), 0.3 * (r64 + s64[0])),
        "norm": (lambda: K.pending_norm(_dev(stack[:5]), _dev(wa), 1e-3), rms(s64[:5].sum(0), 1e-3) * wa.double()),
        "pair": (lambda: K.PendingPair(_dev(rows), _dev(stack[:4]), _dev(wa), _dev(wb), 1e-2),
                 rms(r64, 1e-2) * wa.double() + rms(s64[:4].sum(0), 1e-2) * wb.double()),
    }
    tol = 2e-5 if dtype == torch.float32 else 2e-2
    pick = [n - 1, 0]
    for name, (delta, share) in cases.items():
        x = h.double() + share
        d = x - x.mean(-1, keepdim=True)
        want = d / torch.sqrt((d * d).mean(-1, keepdim=True) + 1e-5) * w.double() + b.double()
        hd, out = _dev(h.clone()), torch.empty(n, hidden, dtype=dtype, device="cuda")
        some = torch.empty(2, hidden, dtype=dtype, device="cuda")
        K.add_layernorm(hd, delta(), _dev(w), _dev(b), 1e-5, some, _i32(pick))
        assert torch.equal(hd.cpu(), h), name
        K.add_layernorm(hd, delta(), _dev(w), _dev(b), 1e-5, out)
        scale = max(1.0, float(want.abs().max()))
        assert float((out.double().cpu() - want).abs().max()) <= tol * scale, name
        assert float((some.double().cpu() - want[pick]).abs().max()) <= tol * scale, name
        assert torch.allclose(hd.double().cpu(), x, atol=2e-5, rtol=1e-6), name


@BOTH
@pytest.mark.parametrize("n", [5, 300])
@pytest.mark.parametrize("sizes", [(3, 1, 10, 6, 8), (4, 2, 16, 32, 16), (4, 2, 64, 64, 16), (2, 2, 128, 64, 32), (6, 3, 48, 96, 16)])
@pytest.mark.parametrize("what", ["bias", "blend", "weightless"])
def test_kernel_attention_input_with_biases_and_blended_values(dtype, n, sizes, what):
    """Few and many tokens (the forms with a wave a head, with 16 bytes a lane and with the tile writer), part of a head
    turned: q rows (with their zeros), key pages, transposed value pages; some tokens are not stored."""
    from jax_vllm_amd.ops import kernels as K

    nq, nkv, dk, dv, page = sizes
    g = torch.Generator().manual_seed(2)
    dp, dims = K.padded_head_dim(dk, dv), (dk // 4) * 2
    width = (nq + nkv) * dk + nkv * dv
    rows = torch.randn(n, width + 8 + (-width) % 8, generator=g).to(dtype)
    bias = torch.randn(width, generator=g) if what == "bias" else None
    first = torch.randn(n, nkv * dv + 8, generator=g).to(dtype)[:, 8:] if what == "blend" else None
    wq, wk = (torch.ones(dk), torch.ones(dk)) if what == "weightless" else (torch.rand(dk, generator=g) + 0.5, torch.rand(dk, generator=g) + 0.5)
    f = 100.0 ** (-torch.arange(0, dims, 2).double() / dims)
    slot_map = list(range(page + 3, page + 3 + n))
    slot_map[1] = slot_map[-1] = -1
    pages = -(-(page + 3 + n) // page)
    positions = _i32(list(range(n)))
    kp = torch.zeros(pages, nkv, page, dp, dtype=dtype, device="cuda")
    vp = torch.zeros(pages, nkv, dp, page, dtype=dtype, device="cuda")
    firsts = torch.cat([torch.zeros(n, 8, dtype=dtype), first], dim=1).to("cuda")[:, 8:] if first is not None else None
    q = K.attn_prepare_wide(_dev(rows), _dev(bias) if bias is not None else None, _dev(wq), _dev(wk), 1e-3, K.rope_table(positions, _dev(f.float())), dims,
                            _i32(slot_map), kp, vp, page, nq, nkv, dk, dv, dp, norm_per_head=True, v_first=firsts, v_mix=0.3 if first is not None else 0.0)
    x = rows[:, :width].double() + (bias.double() if bias is not None else 0.0)
    ang = torch.arange(n).double().view(n, 1, 1) * f

    def heads(y, count, w):
        y = y.reshape(n, count, dk)
        y = y / torch.sqrt((y * y).mean(-1, keepdim=True) + 1e-3) * w.double()
        u, v = y[..., :dims // 2], y[..., dims // 2:dims]
        return torch.cat([u * ang.cos() - v * ang.sin(), v * ang.cos() + u * ang.sin(), y[..., dims:]], dim=-1)

    want_q, want_k = heads(x[:, :nq * dk], nq, wq), heads(x[:, nq * dk:(nq + nkv) * dk], nkv, wk)
    want_v = x[:, (nq + nkv) * dk:]
    if first is not None:
        want_v = 0.7 * want_v + 0.3 * first.double()
    want_v = want_v.reshape(n, nkv, dv)
    tol = 2e-4 if dtype == torch.float32 else 3e-2
    got_q = q.double().cpu().view(n, nq, dp)
    assert torch.allclose(got_q[..., :dk], want_q, atol=tol, rtol=tol) and not got_q[..., dk:].any()
    sm = torch.tensor(slot_map)
    keep = sm >= 0
    pg, off = (sm // page)[keep], (sm % page)[keep]
    kc, vc = kp.double().cpu(), vp.double().cpu()
    assert torch.allclose(kc[pg, :, off, :dk], want_k[keep], atol=tol, rtol=tol)
    assert torch.allclose(vc[pg, :, :dv, off], want_v[keep], atol=tol, rtol=tol)
    kc[pg, :, off, :dk] = 0
    vc[pg, :, :dv, off] = 0
    assert not kc.any() and not vc.any()           # nothing else was written: pads, other slots, the null page


def paged_case(q_lens, ctx_lens, nq, nkv, D, page, sees, dtype, seed):
    """A step over a paged cache whose tables hold the null page for keys that no query sees; ``sees(pos)``: the keys of the
    query at that position.  Returns (StepContext, q, key pages, value pages, keys and values per request in double)."""
    from jax_vllm_amd.parts.spec import StepContext

    g = torch.Generator().manual_seed(seed)
    R, n = len(q_lens), sum(q_lens)
    total = [c + q for c, q in zip(ctx_lens, q_lens)]
    width = max(-(-t // page) for t in total)
    tables = torch.zeros(R, width, dtype=torch.int32)
    nxt = 1
    for r in range(R):
        need = sorted({j // page for i in range(q_lens[r]) for j in sees(ctx_lens[r] + i)})
        for p in need:
            tables[r, p] = nxt
            nxt += 1
    kp = (torch.randn(nxt, nkv, page, D, generator=g) * 0.5).to(dtype)
    vp = torch.randn(nxt, nkv, D, page, generator=g).to(dtype)
    kp[0] = vp[0] = 0
    q = (torch.randn(n, nq * D, generator=g) * 0.5).to(dtype)
    cu = np.cumsum([0] + q_lens)
    positions = [c + i for c, m in zip(ctx_lens, q_lens) for i in range(m)]
    token_req = [r for r, m in enumerate(q_lens) for _ in range(m)]
    ctx = StepContext(num_tokens=n, num_requests=R, positions=_i32(positions), token_req=_i32(token_req), cu_seqlens=_i32(cu.tolist()),
                      context_lens=_i32(ctx_lens), slot_ids=_i32([0] * R), block_tables=[_dev(tables)], slot_mappings=[None],
                      page_size=page, q_lens_host=q_lens, context_lens_host=ctx_lens, slot_ids_host=[0] * R,
                      max_q_len=max(q_lens), max_kv_len=max(total))
    kv = [(kp.double()[tables[r].long()].permute(0, 2, 1, 3).reshape(-1, nkv, D), vp.double()[tables[r].long()].permute(0, 3, 1, 2).reshape(-1, nkv, D))
          for r in range(R)]
    return ctx, q, kp, vp, kv, positions, token_req


def attend(ctx, q, kp, vp, nq, nkv, D, **what):
    from jax_vllm_amd.parts import attention_backend
    from jax_vllm_amd.parts.spec import LayerMemory

    att = SimpleNamespace(**{**dict(nq=nq, nkv=nkv, d=D, window=None, chunk=None, q_row_stride=nq * D, sinks=None, softcap=None, keep_first=0), **what})
    out = torch.empty(q.shape[0], nq * D, dtype=q.dtype, device="cuda")
    attention_backend.run(att, out, _dev(q), ctx, LayerMemory(pages={"k": _dev(kp), "v": _dev(vp)}, group=0))
    return out.double().cpu().view(-1, nq, D)


@BOTH
@pytest.mark.parametrize("head_dim", [40, 64, 96, 160])
@pytest.mark.parametrize("window,chunk,keep,cap", [(50, None, 20, 2.0), (50, None, 64, None), (1, None, 1, None), (33, None, 200, 5.0), (300, None, 130, None),
                                                   (None, None, 0, 1.0), (None, 64, 0, 3.0)])
def test_kernel_attention_with_kept_first_keys_and_capped_scores(dtype, head_dim, window, chunk, keep, cap):
    """Prompt portions and single tokens of three requests: the float kernel, and in bfloat16 the matrix-core kernels for
    prompts (with 32 and with 16 rows a tile) and for decoded tokens, with a sink."""
    nq, nkv, page, D, scale = 4, 2, 16, head_dim, 0.4

    def sees(pos):
        lo = pos - pos % chunk if chunk else max(0, pos - window + 1) if window else 0
        return sorted(set(range(lo, pos + 1)) | set(range(min(keep, pos + 1))))

    sinks = torch.tensor([0.3, -2.0, 1.5, 0.0])
    for q_lens, ctx_lens in (([150, 5, 1], [0, 120, 700]), ([1, 1, 1], [3, 900, 64])):
        ctx, q, kp, vp, kv, positions, token_req = paged_case(q_lens, ctx_lens, nq, nkv, D, page, sees, dtype, 5)
        want = torch.empty(len(positions), nq, D, dtype=torch.float64)
        for t, (pos, r) in enumerate(zip(positions, token_req)):
            at = sees(pos)
            for h in range(nq):
                s = (kv[r][0][at, h // 2] @ q[t].double().view(nq, D)[h]) * scale
                s = cap * torch.tanh(s / cap) if cap else s
                e = torch.exp(s)
                want[t, h] = e @ kv[r][1][at, h // 2] / (e.sum() + torch.exp(sinks[h].double()))
        got = attend(ctx, q, kp, vp, nq, nkv, D, scale=scale, window=window, chunk=chunk, keep_first=keep, softcap=cap, sinks=_dev(sinks))
        tol = 2e-5 if dtype == torch.float32 else 3e-2
        assert float((got - want).abs().max()) <= tol * max(1.0, float(want.abs().max()))


def test_kernel_decode_with_kept_keys_and_tables_wider_than_a_block_keeps():
    """Tables of 4,500 pages of 8 keys: a block keeps the entries of its own split's keys beside those of the kept first
    keys, and a split whose keys are all kept ones has none of its own."""
    nq, nkv, page, D, window, keep = 2, 1, 8, 64, 700, 100
    sees = lambda pos: sorted(set(range(max(0, pos - window + 1), pos + 1)) | set(range(min(keep, pos + 1))))      # noqa: E731
    ctx, q, kp, vp, kv, positions, token_req = paged_case([1, 1], [35990, 700], nq, nkv, D, page, sees, torch.bfloat16, 6)
    assert ctx.block_tables[0].shape[1] > 4096
    got = attend(ctx, q, kp, vp, nq, nkv, D, scale=0.5, window=window, keep_first=keep, softcap=8.0)
    for t, (pos, r) in enumerate(zip(positions, token_req)):
        at = sees(pos)
        for h in range(nq):
            s = 8.0 * torch.tanh((kv[r][0][at, 0] @ q[t].double().view(nq, D)[h]) * 0.5 / 8.0)
            want = torch.softmax(s, 0) @ kv[r][1][at, 0]
            assert float((got[t, h] - want).abs().max()) <= 3e-2 * max(1.0, float(want.abs().max()))


@pytest.mark.parametrize("cap", [0.5, 30.0])
def test_kernel_cap_on_large_and_small_scores(cap):
    """Scores from a thousandth of the cap to a hundred times it: values that are one-hot per key read the weights back."""
    nq = nkv = 1
    D, page, n = 64, 16, 60
    ctx, q, kp, vp, kv, positions, _ = paged_case([n], [0], nq, nkv, D, page, lambda pos: range(pos + 1), torch.bfloat16, 7)
    q[:] = 0
    q[:, 0] = 1.0
    flat = torch.zeros(kp.shape[0] * page, D)
    flat[page:page + n, 0] = torch.linspace(-1, 1, n) * 100 * cap
    flat[page + 3:page + n:5, 0] *= 1e-5
    kp = flat.view(-1, page, 1, D).permute(0, 2, 1, 3).contiguous().to(torch.bfloat16)
    eye = torch.zeros(vp.shape[0], 1, D, page)
    for j in range(n):
        eye[1 + j // page, 0, j, j % page] = 1.0
    got = attend(ctx, q, kp, eye.to(torch.bfloat16), nq, nkv, D, scale=1.0, softcap=cap)
    keys = kp.double().permute(0, 2, 1, 3).reshape(-1, D)[page:page + n, 0]
    s = cap * torch.tanh(keys / cap)
    for t in (0, 7, n - 1):
        assert torch.allclose(got[t, 0, :t + 1], torch.softmax(s[:t + 1], 0), atol=4e-3, rtol=1e-2)


@BOTH
@pytest.mark.parametrize("dim,vdim", [(8, 8), (12, 20), (64, 80), (128, 96), (130, 7)])
def test_kernel_recurrence_read_after_the_write(dtype, dim, vdim):
    """Four requests of 37, 1, 6 and 90 tokens that continue states of their own, token by token and (up to 128 channels) by
    chunks; decays from almost none to almost all of the state, with an exact zero."""
    from jax_vllm_amd.ops import kernels as K

    g = torch.Generator().manual_seed(8)
    lens, slots, H = [37, 1, 6, 90], [2, 0, 3, 4], 2
    n = sum(lens)
    r, k = (torch.randn(n, H * dim, generator=g).to(dtype) for _ in range(2))
    v = torch.randn(n, H * vdim, generator=g).to(dtype)
    rate = -torch.exp(torch.randn(n, H * dim, generator=g) * 2 - 2)
    rate[50, :] = -200.0
    rate[60, :] = 0.0
    state = torch.randn(6, H, dim, vdim, generator=g)
    want, new = torch.empty(n, H, vdim, dtype=torch.float64), state.double().clone()
    at = 0
    for m, s in zip(lens, slots):
        for t in range(at, at + m):
            for h in range(H):
                c = slice(h * dim, (h + 1) * dim)
                new[s, h] = torch.exp(rate[t, c].double())[:, None] * new[s, h] + torch.outer(k[t, c].double(), v[t, h * vdim:(h + 1) * vdim].double())
                want[t, h] = 0.25 * r[t, c].double() @ new[s, h]
        at += m
    cu = _i32(np.cumsum([0] + lens).tolist())
    plans = [None]
    if dim <= K.WKV_CHUNK_MAX_DIM:
        work, firsts = [], [0]
        for q, m in enumerate(lens):
            start = sum(lens[:q])
            work += [(q, start + b) for b in range(0, m, K.WKV_CHUNK_TOKENS)]
            firsts.append(len(work))
        plans.append((_i32([x for w in work for x in w]), _i32(firsts), len(work)))
    for plan in plans:
        st = _dev(state.clone())
        got = K.wkv_steps(_dev(r), _dev(k), _dev(v), _dev(rate), None, None, st, _i32(slots), cu, H, dim, vdim, chunk_plan=plan, after=True, r_scale=0.25)
        scale = float(want.abs().max())
        assert float((got.double().cpu().view(n, H, vdim) - want).abs().max()) <= 2e-5 * scale
        assert float((st.double().cpu() - new).abs().max()) <= 2e-5 * float(new.abs().max())


@BOTH
@pytest.mark.parametrize("n,channels,rank", [(1, 10, 1), (7, 64, 16), (130, 300, 24), (33, 2048, 16), (5, 70, 37)])
def test_kernel_decays_from_a_small_rank(dtype, n, channels, rank):
    from jax_vllm_amd.ops import kernels as K

    g = torch.Generator().manual_seed(9)
    wide = torch.randn(n, rank + 24, generator=g).to(dtype)
    w = (torch.randn(channels, rank, generator=g) * 3).to(dtype)
    b = torch.randn(channels, generator=g) * 5
    got = K.low_rank_decay(_dev(wide)[:, 8:8 + rank], _dev(w), _dev(b), 7.0)
    want = torch.nn.functional.logsigmoid(wide[:, 8:8 + rank].double() @ w.double().T + b.double()) / 7.0
    assert torch.allclose(got.double().cpu(), want, atol=1e-6, rtol=3e-5)


CLAMPED = ("clamped", 0.8, 1.702)


def clamped(gate, up, limit=0.8, slope=1.702):
    g = gate.clamp(max=limit)
    return g * torch.sigmoid(slope * g) * (up.clamp(-limit, limit) + 1)


@BOTH
@pytest.mark.parametrize("interleaved", [False, True])
@pytest.mark.parametrize("n,inter", [(1, 5), (3, 64), (130, 1032)])
def test_kernel_clamped_activation(dtype, interleaved, n, inter):
    from jax_vllm_amd.ops import kernels as K

    g = torch.Generator().manual_seed(10)
    gate, up = (torch.randn(n, inter, generator=g).to(dtype) * 2 for _ in range(2))
    gate[0, 0], up[0, 0] = 300.0, -300.0
    gate[0, 1], up[0, 1] = -300.0, 300.0
    x = torch.stack([gate, up], dim=-1).reshape(n, 2 * inter) if interleaved else torch.cat([gate, up], dim=1)
    got = K.gated_mul(_dev(x), interleaved=interleaved, activation=CLAMPED)
    tol = 1e-6 if dtype == torch.float32 else 1e-2
    assert torch.allclose(got.double().cpu(), clamped(gate.double(), up.double()), atol=tol, rtol=tol)
    for wrong in ("clamped", ("clamped", 0.0, 1.0), ("clamped", 1.0)):
        with pytest.raises(K.KernelArgumentError):
            K.gated_mul(_dev(x), activation=wrong)


@pytest.mark.parametrize("m", [1, 8, 16, 24, 40])
def test_kernel_clamped_activation_behind_products(m):
    """As the epilogue of every organisation of the few-row products."""
    from jax_vllm_amd.ops import kernels as K

    g = torch.Generator().manual_seed(11)
    k, inter = 1024, 320
    x = torch.randn(m, k, generator=g).to(torch.bfloat16)
    w = (torch.randn(2 * inter, k, generator=g) * k ** -0.5).to(torch.bfloat16)
    y = x.double() @ w.double().T
    want = clamped(y[:, 0::2], y[:, 1::2])
    runs = [K.gemm_skinny(_dev(x), _dev(w), gate_pairs=CLAMPED), K.gemm_tile64(_dev(x), _dev(w), gate_pairs=CLAMPED), K.linear(_dev(x), _dev(w), gate_pairs=CLAMPED)]
    if m <= 32:
        runs.append(K.gemm_skinny(_dev(x), _dev(w), gate_pairs=CLAMPED, block_shape=(-2, 64, 4)))
    for got in runs:
        assert float((got.double().cpu() - want).abs().max()) <= 1.5e-2


@BOTH
@pytest.mark.parametrize("n", [1, 7, 33, 200])
@pytest.mark.parametrize("hidden,ff", [(64, 32), (50, 13), (512, 192)])
def test_kernel_clamped_experts_under_a_corrected_choice(dtype, n, hidden, ff):
    """Streamed, matrix-core and float experts; a chosen expert's weight is its sigmoid times a constant, whatever the
    correction that chose it."""
    from jax_vllm_amd.ops import kernels as K

    g = torch.Generator().manual_seed(12)
    experts, top = 6, 3
    x = torch.randn(n, hidden, generator=g).to(dtype)
    gate, up = ((torch.randn(experts, ff, hidden, generator=g) * hidden ** -0.5).to(dtype) for _ in range(2))
    down = (torch.randn(experts, hidden, ff, generator=g) * ff ** -0.5).to(dtype)
    router = (torch.randn(experts, hidden, generator=g) * hidden ** -0.5).to(dtype)
    correction = torch.randn(experts, generator=g) * 0.3
    plan = K.moe_route(None, top, x=_dev(x), w_router=_dev(router), score="sigmoid_corrected", correction=_dev(correction), weight_scale=1.7,
                       tile_rows=K.moe_tile_rows_for(dtype, hidden, ff, n * top, experts))
    ids, wts = plan.ids.view(n, top).cpu().long(), plan.weights.view(n, top).cpu().double()
    s = torch.sigmoid(x.double() @ router.double().T)
    ranked = (s + correction.double()).sort(-1, descending=True)
    clear = (ranked.values[:, :-1] - ranked.values[:, 1:]).amin(-1) > 1e-5
    assert clear.float().mean() > 0.5 and torch.equal(ids[clear], ranked.indices[clear, :top])
    assert torch.allclose(wts, 1.7 * s.gather(1, ids), atol=1e-5)
    out = torch.empty(top, n, hidden, device="cuda")
    K.moe_experts(_dev(x), plan, _dev(gate), _dev(up), _dev(down), CLAMPED, out, weight_on_input=False)
    want = torch.empty(top, n, hidden, dtype=torch.float64)
    for t in range(n):
        for j in range(top):
            e = ids[t, j]
            want[j, t] = wts[t, j] * (down[e].double() @ clamped(gate[e].double() @ x[t].double(), up[e].double() @ x[t].double()))
    tol = 1e-5 if dtype == torch.float32 else 2e-2
    assert float((out.double().cpu() - want).abs().max()) <= tol * float(want.abs().max())


@pytest.mark.parametrize("n,experts,top", [(1, 4, 1), (16, 9, 4), (60, 130, 2), (300, 12, 12), (5, 300, 7)])
def test_kernel_corrected_choice_from_logits(n, experts, top):
    """The form in registers and the one that scans (above 256 experts), in one launch with the grouping and apart."""
    from jax_vllm_amd.ops import kernels as K

    g = torch.Generator().manual_seed(13)
    z = torch.randn(n, experts, generator=g) * 2
    correction = torch.randn(experts, generator=g)
    s = torch.sigmoid(z.double())
    for corr in (correction, None):
        plan = K.moe_route(_dev(z), top, score="sigmoid_corrected", correction=_dev(corr) if corr is not None else None, weight_scale=0.4)
        ids, wts = plan.ids.view(n, top).cpu().long(), plan.weights.view(n, top).cpu().double()
        ranked = (s + (corr.double() if corr is not None else 0.0)).sort(-1, descending=True)
        clear = (ranked.values[:, :-1] - ranked.values[:, 1:])[:, :top].amin(-1) > 1e-6 if experts > 1 else torch.ones(n, dtype=torch.bool)
        assert clear.float().mean() > 0.5 and torch.equal(ids[clear], ranked.indices[clear, :top])
        assert torch.allclose(wts, 0.4 * s.gather(1, ids), atol=1e-6)


def test_frequencies_under_a_factor_are_computed_in_double():
    from jax_vllm_amd.parts.rotary import RotaryEncoding

    got = RotaryEncoding(64, 500000.0, 48, linear_factor=3.0).inverse_frequencies()
    want = torch.tensor([500000.0 ** (-2.0 * i / 48) / 3.0 for i in range(24)], dtype=torch.float64).to(torch.float32)
    assert torch.equal(got, want)
    with pytest.raises(ValueError):
        RotaryEncoding(8, 100.0, linear_factor=2.0, by_wavelength={"factor": 1.0})


def test_parts_refuse_what_they_do_not_have():
    from jax_vllm_amd.parts.attention import GroupedQueryAttention as A

    for wrong in (dict(keep_first=4), dict(sinks=True, softmax_plus_one=True), dict(value_blend="third"), dict(value_blend="first", qkv_bias=True),
                  dict(qk_norm_weight=False, qk_norm="whole")):
        with pytest.raises(ValueError):
            A(32, 2, 1, 8, **wrong)
