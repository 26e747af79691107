"""Kuditar on the host: its configuration reader, the tensors its ``ModelSpec`` asks for, which layers blend values, what a
request keeps (pages and state), the pages of a window that keeps the first tokens, and the plain implementation's own
consistency."""
import copy
import math

import numpy as np
import pytest
import torch

from tests.kuditar_util import (ALL_SMALL, SMALL_A, SMALL_B, SMALL_C, attention, block_side, config, delta_side, dense, layer,
                                linear_side, make_folder, moe, parallel, parallel_2, plain_logits, plain_of, tokens_of, window_side)
from tests.plain import kuditar_plain as P


def spec_of(cfg_dict):
    from jax_vllm_amd.config.registry import resolve
    from jax_vllm_amd.parts.model import DecoderModel

    arch, cfg, _ = resolve(cfg_dict)
    return arch, cfg, DecoderModel(arch.build_spec(cfg))


def expected_tensors(c):
    """Names and shapes from the configuration alone, written out independently of the product."""
    w = c["width"]
    out = {"embed": (c["vocab"], w), "final.norm": (w,), "final.norm.b": (w,)}

    def softmax_side(p, m):
        H, G, d, v = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        out.update({p + "q": (H * d, w), p + "k": (G * d, w), p + "v": (G * v, w), p + "o": (w, H * v)})

    for i, l in enumerate(c["layers"]):
        p, m = f"l{i}.", l["mixer"]
        out.update({p + "norm1": (w,), p + "norm1.b": (w,)})
        if l["type"] == "attention":
            softmax_side(p + "mix.", m)
            out[p + "mix.g"] = (m["heads"] * m["vdim"], w)
            if m.get("v_mix"):
                out[p + "mix.vmix"] = ()
        else:
            a, b = m["left"], m["right"]
            left, right = p + "mix.left.", p + "mix.right."
            softmax_side(left, a)
            out.update({left + "q.b": (a["heads"] * a["dim"],), left + "k.b": (a["kv_heads"] * a["dim"],),
                        left + "v.b": (a["kv_heads"] * a["vdim"],), left + "q.norm": (a["dim"],), left + "k.norm": (a["dim"],),
                        left + "out": (w,), right + "out": (w,), right + "norm": (b["vdim"],)})
            H, d, v = b["heads"], b["dim"], b["vdim"]
            out.update({right + "v": (H * v, w), right + "g": (H * v, w), right + "o": (w, H * v)})
            if l["type"] == "parallel":
                qk = b["kv_heads"] * d
                out[left + "sink"] = (a["heads"],)
                out.update({right + "q": (qk, w), right + "k": (qk, w), right + "a": (H, w), right + "b": (H, w), right + "A_log": (H,),
                            right + "dt_bias": (H,), right + "q.conv": (qk, b["conv"]), right + "k.conv": (qk, b["conv"]),
                            right + "v.conv": (H * v, b["conv"])})
            else:
                out.update({right + "q": (H * d, w), right + "k": (H * d, w), right + "a1": (b["decay_rank"], w),
                            right + "a2": (H * d, b["decay_rank"]), right + "a2.b": (H * d,)})
        f = l.get("mlp")
        if not f:
            continue
        out.update({p + "norm2": (w,), p + "norm2.b": (w,)})
        if f["kind"] == "dense":
            out.update({p + "mlp.gate": (f["ff"], w), p + "mlp.up": (f["ff"], w), p + "mlp.down": (w, f["ff"])})
        else:
            e, ff = f["router"]["experts"], f["expert"]["ff"]
            out.update({p + "mlp.router": (e, w), p + "mlp.correction": (e,)})
            for j in range(e):
                out.update({f"{p}mlp.e{j}.gate": (ff, w), f"{p}mlp.e{j}.up": (ff, w), f"{p}mlp.e{j}.down": (w, ff)})
    return out


@pytest.mark.parametrize("small", ALL_SMALL, ids=[s["name"] for s in ALL_SMALL])
def test_tensors_schedule_and_memory_plan_follow_the_configuration(small):
    from jax_vllm_amd.parts.spec import state_specs_of

    c = small["config"]
    _, cfg, model = spec_of(c)
    assert {k: tuple(v.shape) for k, v in model.tensor_specs().items()} == expected_tensors(c)
    assert [run.layer for run in model.spec.schedule] == list(range(len(c["layers"])))
    assert cfg.to_dict() == c
    for p, l in zip(model.memory_plan(), c["layers"]):
        m = l["mixer"]
        left, mask = (m, {}) if l["type"] == "attention" else (m["left"], m["left"].get("mask") or {})
        states = {s.name: (s.shape, s.dtype) for s in state_specs_of(p.state)}
        want = {}
        if l["type"] != "attention":
            r = m["right"]
            want["right.S"] = ((r["heads"], r["dim"], r["vdim"]), "float32")
            if l["type"] == "parallel":
                want["right.conv"] = ((r["conv"] - 1, 2 * r["kv_heads"] * r["dim"] + r["heads"] * r["vdim"]), "float32")
        assert states == want
        size = mask.get("size")
        seen = (p.cache.window, p.cache.chunk, p.cache.keep_first)
        assert seen == ((None, size, 0) if l["type"] == "parallel_2" else (size, None, mask.get("keep_first") or 0))
        assert [t.token_shape for t in p.cache.tensors] == [(left["kv_heads"], -(-max(left["dim"], left["vdim"]) // 16) * 16)] * 2
    assert model.replayable()


def test_the_rank_of_the_decay_may_come_from_the_checkpoint():
    c = copy.deepcopy(SMALL_A["config"])
    del c["layers"][2]["mixer"]["right"]["decay_rank"]
    shapes = {k: tuple(v.shape) for k, v in spec_of(c)[2].tensor_specs().items()}
    assert shapes["l2.mix.right.a1"] == (None, 48) and shapes["l2.mix.right.a2"] == (36, None)


def test_the_first_blending_layer_keeps_its_values_and_later_ones_blend():
    model = spec_of(SMALL_A["config"])[2]
    assert [getattr(l.mixer, "value_blend", None) for l in model.layers] == [None, "first", None, None, "later"]
    model = spec_of(SMALL_C["config"])[2]
    assert [getattr(l.mixer, "value_blend", None) for l in model.layers] == ["first", None, None, "later", None, None]


def test_cache_groups_tell_kept_first_tokens_apart():
    from jax_vllm_amd.cache.storage import group_keys_of
    from jax_vllm_amd.parts.spec import PagedCacheSpec, kv_cache_spec, widest_need

    assert group_keys_of(spec_of(SMALL_A["config"])[2].memory_plan()) == [("window", 9, 11), ("full",), ("chunk", 22)]
    assert kv_cache_spec(1, 16, 9).group_key == ("window", 9)
    assert kv_cache_spec(1, 16, keep_first=4).group_key == ("full",)
    assert PagedCacheSpec(kv_cache_spec(1, 16).tensors, chunk=8, keep_first=3).group_key == ("chunk", 8, 3)
    assert widest_need([("window", 4, 9), ("window", 7)]) == ("window", 7, 9)
    assert widest_need([("window", 4, 9), ("chunk", 7)]) == ("full",)


@pytest.mark.parametrize("keep,kept_pages", [(1, 1), (8, 1), (9, 2), (20, 3)])
def test_pages_of_kept_first_tokens_stay_while_the_window_moves_on(keep, kept_pages):
    """A window of 10 over pages of 8: the pages between the kept first ones and the window's go back, whatever the
    portions, and all of them at the end."""
    from jax_vllm_amd.cache import CacheManager

    for portions in ([7, 1, 12, 1, 30, 2, 9, 1, 1], [64], [1] * 64):
        c = CacheManager([("window", 10, keep)], 8, 12, 1, enable_prefix_cache=False, has_state=True)
        c.start("a")
        at = 0
        for n in portions:
            c.reserve("a", n)
            table = c.block_table("a", 0)
            for p in range(at, at + n):
                assert all(table[j // 8] for j in range(p + 1) if p - j < 10 or j < keep)
            c.commit("a", list(range(n)))
            at += n
            first = max(0, at - 9)
            assert [bool(t) for t in c.block_table("a", 0)] == [i < kept_pages or 8 * (i + 1) > first for i in range(-(-at // 8))]
            c.check_invariants()
        c.finish("a")
        assert c.num_free_pages() == 12


def test_attention_plans_count_the_kept_first_keys():
    from jax_vllm_amd.ops import kernels as K
    from jax_vllm_amd.parts.attention_backend import keys_seen, prefill_work_items

    assert keys_seen(1000, 30, 16) == 46 and keys_seen(20, 30, 16) == 20 and keys_seen(70, 0, 16) == 70
    items = prefill_work_items([300], [500], 4, 100, 64, 2, keep=20)
    assert sorted(m for _, a, b in items for m in (a, b) if m >= 0) == list(range(0, 1200, 64))
    assert K.attn_decode_min_splits(4096, 16, 100) == 1
    for width, page, keep in ((5000, 16, 20), (60000, 8, 1000), (4097, 32, 1)):
        splits = K.attn_decode_min_splits(width, page, keep)
        per_split = -(-(-(-width * page // 32)) // splits)      # the kernel library's own condition
        assert per_split * 32 // page + 2 + -(-keep // 32) * 32 // page + 1 <= K.ATTN_DECODE_TABLE_ENTRIES
    with pytest.raises(K.KernelArgumentError):
        K.attn_decode_min_splits(5000, 8, 8 * 2048)


def test_configuration_errors_name_the_place():
    from jax_vllm_amd.config.errors import ConfigError
    from jax_vllm_amd.config.registry import resolve

    def broken(change):
        c = copy.deepcopy(SMALL_A["config"])
        change(c)
        with pytest.raises(ConfigError) as e:
            resolve(c)
        return str(e.value)

    layers = lambda c, i: c["layers"][i]["mixer"]      # noqa: E731
    assert "layers[1].mixer" in broken(lambda c: layers(c, 1).update(heads=4, kv_heads=3))
    assert "layers[1].mixer.rot.dims" in broken(lambda c: layers(c, 1)["rot"].update(dims=22))
    assert "layers[1].mixer.rot.scaling.factor" in broken(lambda c: layers(c, 1)["rot"].update(scaling={"factor": 0}))
    assert "layers[1].mixer.softcap" in broken(lambda c: layers(c, 1).update(softcap=-1.0))
    assert "v_mix" in broken(lambda c: layers(c, 1).update(v_mix=1))
    assert "v_mix must agree" in broken(lambda c: layers(c, 4).update(vdim=16))
    assert "layers[0].mixer.left.mask.size" in broken(lambda c: layers(c, 0)["left"].update(mask={"size": 0}))
    assert "layers[0].mixer.left.mask.keep_first" in broken(lambda c: layers(c, 0)["left"]["mask"].update(keep_first=-1))
    assert "layers[0].mixer.right.conv" in broken(lambda c: layers(c, 0)["right"].update(conv=0))
    assert "layers[0].mixer.right" in broken(lambda c: layers(c, 0)["right"].update(kv_heads=3))
    assert "layers[2].mixer.right.tau" in broken(lambda c: layers(c, 2)["right"].update(tau=0))
    assert "layers[2].mixer.left" in broken(lambda c: layers(c, 2).pop("left"))
    assert "layers[2].type" in broken(lambda c: c["layers"][2].update(type="retention"))
    assert "layers[1].mlp.limit" in broken(lambda c: c["layers"][1]["mlp"].update(limit=0))
    assert "limit" in broken(lambda c: c["layers"][0]["mlp"]["expert"].pop("limit"))
    assert "layers[0].mlp.router.top" in broken(lambda c: c["layers"][0]["mlp"]["router"].update(top=7))
    assert "layers[1].mlp.kind" in broken(lambda c: c["layers"][1]["mlp"].update(kind="glu"))
    assert "scale" in broken(lambda c: layers(c, 1).pop("scale"))
    assert "norm" in broken(lambda c: c.pop("norm"))


def test_random_folder_is_read_back(tmp_path):
    folder = make_folder(SMALL_C, tmp_path)
    w = P.read_weights(folder)
    assert {k: tuple(v.shape) for k, v in w.items()} == expected_tensors(SMALL_C["config"])
    assert P.forward(w, P.read_config(folder), [1, 2, 3]).shape == (3, 97)


def test_plain_pieces():
    """The plain implementation against the equations written out element by element."""
    torch.manual_seed(0)
    f64 = torch.float64
    n = 13
    x = torch.randn(n, 6, dtype=f64)
    a, b = torch.randn(6, dtype=f64), torch.randn(6, dtype=f64)
    got = P.layer_norm(x, a, b, 1e-3)
    for t in (0, 5):
        mean = sum(float(v) for v in x[t]) / 6
        var = sum((float(v) - mean) ** 2 for v in x[t]) / 6
        assert np.allclose(got[t], [(float(x[t, c]) - mean) / math.sqrt(var + 1e-3) * float(a[c]) + float(b[c]) for c in range(6)])
    # what queries see
    seen = P.visible_window(n, 4, 3)
    assert [j for j in range(n) if seen[9, j]] == [0, 1, 2, 6, 7, 8, 9] and [j for j in range(n) if seen[2, j]] == [0, 1, 2]
    assert [j for j in range(n) if P.visible_chunk(n, 5)[8, j]] == [5, 6, 7, 8]
    assert P.visible_window(n).sum() == n * (n + 1) // 2 == P.visible_chunk(n).sum()
    # scores under a cap, a sink that is neither scaled nor capped
    q, k, v = (torch.randn(s, n, 4, dtype=f64) for s in (2, 1, 1))
    sink = torch.tensor([0.5, -30.0], dtype=f64)
    got = P.weigh(q, k, v, seen, 0.7, 1.2, sink)
    for h in (0, 1):
        e = {j: math.exp(1.2 * math.tanh(0.7 * float(q[h, 9] @ k[0, j]) / 1.2)) for j in (0, 1, 2, 6, 7, 8, 9)}
        den = sum(e.values()) + math.exp(float(sink[h]))
        assert torch.allclose(got[9, 4 * h:4 * h + 4], sum(p * v[0, j] for j, p in e.items()) / den)
    # rotation: the factor slows every pair down; a norm without a weight is the same before it
    rot = {"dims": 4, "base": 9.0, "scaling": {"factor": 2.0}}
    y = P.rotate(torch.ones(1, n, 6, dtype=f64), rot)
    for i in (0, 1):
        ang = 7 * 9.0 ** (-2 * i / 4) / 2
        assert float(y[0, 7, i]) == pytest.approx(math.cos(ang) - math.sin(ang)) and float(y[0, 7, 2 + i]) == pytest.approx(math.cos(ang) + math.sin(ang))
    z = torch.randn(2, n, 6, dtype=f64)
    assert torch.allclose(P.by_rms(P.rotate(z, rot), 1e-5), P.rotate(P.by_rms(z, 1e-5), rot)) and torch.equal(y[0, :, 4:], torch.ones(n, 2, dtype=f64))
    # the two walks against sums over the past
    q, k, v = (torch.randn(n, 1, 3, dtype=f64) for _ in range(3))
    al = torch.rand(n, 1, 3, dtype=f64)
    got = P.channel_decay_walk(q, k, v, al)
    t = 6
    want = sum(float(sum(q[t, 0, c] * k[j, 0, c] * al[j + 1:t + 1, 0, c].prod() for c in range(3))) * v[j, 0] for j in range(t + 1))
    assert torch.allclose(got[t, 0], want)
    g, beta = torch.rand(n, 1, dtype=f64), torch.ones(n, 1, dtype=f64)
    k = k / k.norm(dim=-1, keepdim=True)
    # with a write strength of 1 and a unit key the state then reads the value back
    assert torch.allclose(P.delta_walk(k, k, v, g, beta)[:, 0], v[:, 0])
    # the clamped activation and the router
    assert float(P.clamped_glu(torch.tensor(5.0), torch.tensor(-9.0), 2.0)) == pytest.approx(2 / (1 + math.exp(-3.404)) * -1)
    assert float(P.clamped_glu(torch.tensor(-5.0), torch.tensor(0.5), 2.0)) == pytest.approx(-5 / (1 + math.exp(8.51)) * 1.5)
    z = torch.tensor([[0.0, 1.0, -1.0, 0.5]], dtype=f64)
    chosen, weight = P.route(z, torch.tensor([0.0, 0.0, 2.0, 0.0], dtype=f64), 2, 3.0)
    assert chosen.tolist() == [[2, 1]] and torch.allclose(weight, 3 * torch.sigmoid(z[:, [2, 1]]))


def test_registry_knows_the_design():
    from jax_vllm_amd.config.registry import supported_architectures

    assert "Kuditar" in supported_architectures()
    assert SMALL_B["config"]["architecture"] == "Kuditar"
    spec_of(config(32, 40, [layer(attention(1, 1, 4), dense(8)), layer(parallel(window_side(1, 1, 4), delta_side(1, 1, 4, 4))),
                            layer(parallel_2(block_side(1, 1, 4), linear_side(1, 4, 4)), moe(2, 1, 8))]))


# ------------------------------------------------------------------ what a fault in one mechanism would move
@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    return {s["name"]: make_folder(s, tmp_path_factory.mktemp(f"kc{s['name']}")) for s in ALL_SMALL}


FAULTS = {        # mistake -> (function of the plain implementation, what stands in its place)
    "no_sink": ("weigh", lambda plain: lambda q, k, v, seen, scale, cap=None, sink=None: plain(q, k, v, seen, scale, cap, None)),
    "no_cap": ("capped", lambda plain: lambda s, cap: s),
    "cap_before_scale": ("capped", lambda plain: lambda s, cap: plain(s, cap and cap * 0.5)),
    "delta_rule_forgets": ("delta_walk", lambda plain: lambda q, k, v, g, beta: torch.cat([plain(q[:30], k[:30], v[:30], g[:30], beta[:30]), plain(q[30:], k[30:], v[30:], g[30:], beta[30:])])),
    "delta_rule_reads_before_the_write": ("delta_walk", lambda plain: lambda q, k, v, g, beta: torch.cat([torch.zeros_like(v[:1]), plain(q.roll(-1, 0), k, v, g, beta)[:-1]])),
    "linear_attention_forgets": ("channel_decay_walk", lambda plain: lambda q, k, v, a: torch.cat([plain(q[:30], k[:30], v[:30], a[:30]), plain(q[30:], k[30:], v[30:], a[30:])])),
    "decay_of_another_channel": ("channel_decay_walk", lambda plain: lambda q, k, v, a: plain(q, k, v, a.roll(1, -1))),
    "not_clamped": ("clamped_glu", lambda plain: lambda gate, up, limit: plain(gate, up, 1e9)),
    "choice_without_correction": ("route", lambda plain: lambda z, c, top, scale: plain(z, 0 * c, top, scale)),
    "weights_with_correction": ("route", lambda plain: lambda z, c, top, scale: (plain(z, c, top, scale)[0], (torch.sigmoid(z) + c).gather(1, plain(z, c, top, scale)[0]) * scale)),
}


@pytest.mark.parametrize("fault", sorted(FAULTS))
def test_a_fault_in_one_mechanism_would_show(folders, fault, monkeypatch):
    """The small models are made so that a mistake shows: planted in the plain implementation it moves many rows of at
    least one of them by far more than the tests' tolerances; the engine is compared with the unchanged one elsewhere."""
    name, wrong = FAULTS[fault]
    plain = getattr(P, name)
    moved = []
    for small in (SMALL_A, SMALL_C):
        cfg, w = plain_of(folders[small["name"]])
        toks = tokens_of(cfg, 60, 2)
        right = plain_logits(cfg, w, toks)
        monkeypatch.setattr(P, name, wrong(plain))
        off = np.abs(plain_logits(cfg, w, toks) - right).max(axis=-1)
        monkeypatch.setattr(P, name, plain)
        moved.append((off > 0.002 * np.abs(right).max()).mean())
    assert max(moved) > 0.3, moved


def test_a_blend_that_is_left_out_would_show(folders):
    for small, at in ((SMALL_A, "l4.mix.vmix"), (SMALL_C, "l3.mix.vmix")):
        cfg, w = plain_of(folders[small["name"]])
        toks = tokens_of(cfg, 60, 2)
        right = plain_logits(cfg, w, toks)
        off = np.abs(plain_logits(cfg, dict(w, **{at: torch.zeros_like(w[at])}), toks) - right).max(axis=-1)
        assert (off > 0.01 * np.abs(right).max()).mean() > 0.5
