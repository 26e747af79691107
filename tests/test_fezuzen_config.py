"""Fezuzen on the host: its configuration reader, the tensors its ``ModelSpec`` asks for, which layers read another
layer's cache and how long that cache keeps its pages, what a request keeps (pages, state of mixers and blocks), the
pages of a group whose queries see their own block of positions, and the plain implementation's own consistency."""
import copy
import json
import math
import tempfile
from pathlib import Path

import pytest
import torch

from tests.fezuzen_util import (ALL_SMALL, LONG, SMALL_A, SMALL_B, SMALL_C, attention, config, latent, layer, make_folder)
from tests.plain import fezuzen_plain as P


def spec_of(cfg_dict):
    from jax_vllm_amd.config.registry import resolve
    from jax_vllm_amd.parts.model import DecoderModel

    arch, cfg, _ = resolve(cfg_dict)
    return arch, cfg, DecoderModel(arch.build_spec(cfg))


def expected_tensors(c):
    """Names and shapes from the configuration alone, written out independently of the product."""
    w, taps = c["width"], c["canon"]["taps"]
    out = {"embed": (c["vocab"], w), "final.norm": (w,), "head": (c["vocab"], w)}
    for i, l in enumerate(c["layers"]):
        p, m = f"l{i}.", l["mixer"]
        out.update({p + "norm1": (w,), p + "norm1b": (w,), p + "canon1": (w, taps)})
        H, d, v = m["heads"], m["dim"], m["vdim"]
        if l["type"] == "attention":
            G = m["kv_heads"]
            rows = {"q": H * d, "k": G * d, "v": G * v}
            out.update({f"{p}mix.{s}": (n, w) for s, n in rows.items()})
            if m.get("conv"):
                out.update({f"{p}mix.{s}.conv": (n, m["conv"]) for s, n in rows.items()})
            out[p + "mix.g"] = (H * v, w)
        else:
            r, rank, q = m["rot_dim"], m["kv_rank"], m["q_rank"]
            out.update({p + "mix.dq": (q, w), p + "mix.dq.norm": (q,), p + "mix.uq": (H * (d + r), q), p + "mix.uk": (H * d, rank),
                        p + "mix.uv": (H * v, rank)})
            if m.get("kv_from") is None:
                out.update({p + "mix.dkv": (rank + r, w), p + "mix.dkv.norm": (rank,)})
        out[p + "mix.o"] = (w, H * v)
        f = l.get("mlp")
        if f:
            out.update({p + "norm2": (w,), p + "norm2b": (w,), p + "canon2": (w, taps)})
            e, ff = f["router"]["experts"], f["expert"]["ff"]
            out[p + "mlp.router"] = (e, w)
            for j in range(e):
                out.update({f"{p}mlp.e{j}.up": (ff, w), f"{p}mlp.e{j}.down": (w, ff)})
            if f.get("shared"):
                s = f["shared"]["ff"]
                out.update({p + "mlp.shared.up": (s, w), p + "mlp.shared.down": (w, s)})
    return out


@pytest.mark.parametrize("small", ALL_SMALL, ids=[s["name"] for s in ALL_SMALL])
def test_tensors_schedule_and_memory_plan_follow_the_configuration(small):
    from jax_vllm_amd.parts.spec import state_specs_of

    c = small["config"]
    _, _, model = spec_of(c)
    assert {k: tuple(v.shape) for k, v in model.tensor_specs().items()} == expected_tensors(c)
    assert [run.layer for run in model.spec.schedule] == list(range(len(c["layers"])))
    lags = c["canon"]["taps"] - 1
    for p, l in zip(model.memory_plan(), c["layers"]):
        m = l["mixer"]
        states = {s.name: (s.shape, s.dtype) for s in state_specs_of(p.state)}
        want = {"block.canon1": ((lags, c["width"]), "float32")}
        if l.get("mlp"):
            want["block.canon2"] = ((lags, c["width"]), "float32")
        size = (m.get("mask") or {}).get("size")
        if l["type"] == "attention":
            channels = (m["heads"] + m["kv_heads"]) * m["dim"] + m["kv_heads"] * m["vdim"]
            if m.get("conv"):
                want["filter"] = ((m["conv"] - 1, channels), "float32")
            assert p.cache_of is None and (p.cache.chunk, p.cache.window) == (size, None)
            assert [t.token_shape for t in p.cache.tensors] == [(m["kv_heads"], -(-max(m["dim"], m["vdim"]) // 16) * 16)] * 2
        else:
            assert p.cache_of == m.get("kv_from") and (p.cache.chunk, p.cache.window) == (None, size)
            assert [t.token_shape for t in p.cache.tensors] == [(1, m["kv_rank"] + m["rot_dim"])] * 2
        assert states == want
    assert model.replayable()


def test_a_shared_cache_keeps_what_its_widest_reader_sees():
    from jax_vllm_amd.cache.storage import cache_bytes_per_token, group_keys_of, needs_of
    from jax_vllm_amd.parts.spec import widest_need

    assert needs_of(spec_of(SMALL_A["config"])[2].memory_plan()) == {0: ("chunk", 22), 1: ("window", 19), 3: ("chunk", 5)}
    plan = spec_of(SMALL_C["config"])[2].memory_plan()
    assert needs_of(plan) == {0: ("full",), 1: ("chunk", 1), 3: ("chunk", 1000), 4: ("window", 1000)}
    assert group_keys_of(plan) == [("full",), ("chunk", 1), ("chunk", 1000), ("window", 1000)]
    # per token: the vector of layer 0 (read by layer 2 as well) and of layer 4 in two layouts, keys and values of 64
    assert cache_bytes_per_token(plan, torch.bfloat16) == 2 * 2 * (128 + 64 + 64 + 64)
    assert widest_need([("window", 4), ("window", 9)]) == ("window", 9)
    assert widest_need([("chunk", 4), ("chunk", 4)]) == ("chunk", 4)
    for mixed in ([("chunk", 4), ("chunk", 8)], [("window", 4), ("chunk", 4)], [("window", 4), ("full",)]):
        assert widest_need(mixed) == ("full",)


def test_pages_of_finished_blocks_are_given_back():
    """Blocks of 20 positions over pages of 8: a page goes back when the next token lies in a block that starts at or
    behind the page's end, whatever the portions; the page that a block's edge cuts stays until the block behind it ends."""
    from jax_vllm_amd.cache import CacheManager

    for portions in ([7, 1, 12, 1, 30, 2, 9, 1, 1], [64], [1] * 64):
        c = CacheManager([("chunk", 20)], 8, 12, 1, enable_prefix_cache=False, has_state=True)
        c.start("a")
        at = 0
        for n in portions:
            c.reserve("a", n)
            table = c.block_table("a", 0)
            for p in range(at, at + n):                    # every key that the portion's first query, or a later one, sees has a page
                assert all(table[j // 8] for j in range(p - p % 20, p + 1))
            c.commit("a", list(range(n)))
            at += n
            first = at - at % 20
            assert [bool(t) for t in c.block_table("a", 0)] == [8 * (i + 1) > first for i in range(-(-at // 8))]
            c.check_invariants()
        assert at == 64 and c.num_free_pages() == 12 - 1   # position 64 lies in the block from 60: page 7 alone
        c.finish("a")
        assert c.num_free_pages() == 12


def test_prefill_work_items_in_blocks_cover_every_row_and_weigh_their_keys():
    from jax_vllm_amd.ops import kernels as K
    from jax_vllm_amd.parts.attention_backend import keys_seen, prefill_work_items

    items = prefill_work_items([300], [50], 4, K.key_window(None, 100), 64, 2)
    rows = sorted(m for _, a, b in items for m in (a, b) if m >= 0)
    assert rows == list(range(0, 1200, 64))
    assert keys_seen(1000, -100) == 100 and keys_seen(1000, 30) == 30 and keys_seen(20, -100) == 20 and keys_seen(70, 0) == 70
    with pytest.raises(K.KernelArgumentError):
        K.key_window(4, 8)


def test_configuration_errors_name_the_place():
    from jax_vllm_amd.config.errors import ConfigError
    from jax_vllm_amd.config.registry import resolve

    def broken(change):
        c = copy.deepcopy(SMALL_A["config"])
        change(c)
        with pytest.raises(ConfigError) as e:
            resolve(c)
        return str(e.value)

    assert "layers[0].mixer" in broken(lambda c: c["layers"][0]["mixer"].update(kv_heads=3))
    assert "vdim" in broken(lambda c: c["layers"][0]["mixer"].update(vdim=7))
    assert "layers[0].mixer.rot.dims" in broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=14))
    assert "layers[1].mixer.rot.dims" in broken(lambda c: c["layers"][1]["mixer"]["rot"].update(dims=3))
    assert "layers[1].mixer.rot.scaling.factor" in broken(lambda c: c["layers"][1]["mixer"]["rot"].update(scaling=dict(LONG, factor=0)))
    assert "layers[0].mixer.mask.size" in broken(lambda c: c["layers"][0]["mixer"].update(mask={"size": 0}))
    assert "layers[0].mlp.router.top" in broken(lambda c: c["layers"][0]["mlp"]["router"].update(top=7))
    assert "groups" in broken(lambda c: c["layers"][0]["mlp"]["router"].update(groups={"count": 4, "keep": 2}))
    assert "groups" in broken(lambda c: c["layers"][3]["mlp"]["router"].update(groups={"count": 4, "keep": 1}))
    assert "layers[2].type" in broken(lambda c: c["layers"][2].update(type="wkv"))
    assert "layers[0].mlp.kind" in broken(lambda c: c["layers"][0]["mlp"].update(kind="dense"))
    assert "layers[2].mixer.kv_from" in broken(lambda c: c["layers"][2]["mixer"].update(kv_from=2))
    assert "layers[4].mixer.kv_from" in broken(lambda c: c["layers"][4]["mixer"].update(kv_from=3))
    assert "kv_rank differs" in broken(lambda c: c["layers"][2]["mixer"].update(kv_rank=24))
    assert "rot differs" in broken(lambda c: c["layers"][2]["mixer"].update(rot={"dims": 4, "base": 100.0}))
    assert "canon" in broken(lambda c: c.pop("canon"))
    assert "canon.taps" in broken(lambda c: c["canon"].update(taps=0))
    assert "scale" in broken(lambda c: c["layers"][1]["mixer"].pop("scale"))
    assert "layers[0].mixer.heads" in broken(lambda c: c["layers"][0]["mixer"].update(heads=0))
    assert "shared" in broken(lambda c: c["layers"][0]["mlp"]["shared"].update(ff=0))


def test_random_folder_is_read_back(tmp_path):
    from jax_vllm_amd import write_random_model

    folder = write_random_model(tmp_path, SMALL_C["config"], seed=1, std=0.1, norm_std=0.05)
    w = P.read_weights(folder)
    assert {k: tuple(v.shape) for k, v in w.items()} == expected_tensors(SMALL_C["config"])
    assert P.forward(w, P.read_config(folder), [1, 2, 3]).shape == (3, 97)


def test_plain_pieces():
    """The plain implementation against the equations written out element by element."""
    torch.manual_seed(0)
    with tempfile.TemporaryDirectory() as d:
        folder = make_folder(SMALL_A, Path(d))
        cfg, w = P.read_config(folder), P.read_weights(folder, torch.float64)
    assert cfg == json.loads(json.dumps(SMALL_A["config"]))
    n, eps, width = 27, cfg["norm"]["eps"], cfg["width"]
    u = torch.randn(n, width, dtype=torch.float64)
    # a filter: the last tap weighs the token itself, nothing stands before the first
    wt = torch.randn(width, 3, dtype=torch.float64)
    got = P.causal_filter(u, wt)
    for t in (0, 1, 2, 9):
        want = sum(wt[:, j] * u[t - 2 + j] for j in range(3) if t - 2 + j >= 0)
        assert torch.allclose(got[t], want)
    # attention in blocks with turned values, row by row
    m, p = cfg["layers"][0]["mixer"], "l0.mix."
    H, G, D, V, size, dims, base = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["mask"]["size"], m["rot"]["dims"], m["rot"]["base"]

    def turn(vec, pos, dims, base):
        out = vec.clone()
        for i in range(dims // 2):
            a = pos * base ** (-2 * i / dims)
            x, y = vec[2 * i], vec[2 * i + 1]
            out[2 * i], out[2 * i + 1] = x * math.cos(a) - y * math.sin(a), y * math.cos(a) + x * math.sin(a)
        return out

    q, k, v = (P.causal_filter(u @ w[p + s].T, w[p + s + ".conv"]) for s in "qkv")
    gate = torch.sigmoid(u @ w[p + "g"].T)
    out = torch.zeros(n, H * V, dtype=torch.float64)
    for i in (0, 5, size - 1, size, size + 3):
        for h in range(H):
            g = h // (H // G)
            seen = [j for j in range(i + 1) if j // size == i // size]
            qi = turn(q[i, h * D:(h + 1) * D], i, dims, base)
            e = [torch.exp(torch.dot(qi, turn(k[j, g * D:(g + 1) * D], j, dims, base)) * m["scale"]) for j in seen]
            o = sum(x * turn(v[j, g * V:(g + 1) * V], j, V, base) for x, j in zip(e, seen)) / (1 + sum(e))
            out[i, h * V:(h + 1) * V] = turn(o, -i, V, base) * gate[i, h * V:(h + 1) * V]
        want = out[i] @ w[p + "o"].T
        assert torch.allclose(P.attention(w, p, m, u, eps)[i], want, atol=1e-10)
    # turned values: only the distance between query and value matters
    x = torch.randn(5, 2, 6, dtype=torch.float64)
    back = P.turn_values(P.turn_values(x, 50.0), 50.0, -1.0)
    assert torch.allclose(back, x) and torch.equal(P.turn_values(x, 50.0)[0], x[0])
    # rescaled frequencies: pairs that turn often keep theirs, slow ones are slowed by the factor
    f, amp = P.blended_frequencies(16, 100.0, LONG)
    f0 = torch.tensor([100.0 ** (-2 * i / 16) for i in range(8)], dtype=torch.float64)
    assert torch.allclose(f[0], f0[0]) and torch.allclose(f[-1], f0[-1] / LONG["factor"]) and amp == pytest.approx(0.1 * math.log(3.0) + 1.0)
    assert not torch.allclose(f[2], f0[2]) and not torch.allclose(f[2], f0[2] / LONG["factor"])
    # one added to the denominator, also where every score is far below zero
    s = torch.tensor([[[-300.0, -301.0]]], dtype=torch.float64)
    assert float(P.softmax_plus_one(s, torch.ones(1, 2, dtype=torch.bool))[0, 0, 0]) == pytest.approx(math.exp(-300.0), rel=1e-9)
    # the router: weights are the softmax over all experts; the choice stays inside the best groups
    f = cfg["layers"][0]["mlp"]
    choice, weight = P.router(w, "l0.mlp.", f, u)
    s = torch.softmax(u @ w["l0.mlp.router"].T, -1)
    differs = 0
    for t in range(n):
        best = sorted(range(3), key=lambda g: -float(s[t, 2 * g:2 * g + 2].max()))[:2]
        allowed = [e for e in range(6) if e // 2 in best]
        want = sorted(allowed, key=lambda e: -float(s[t, e]))[:2]
        assert choice[t].tolist() == want and torch.equal(weight[t], s[t, want])
        free = sorted(range(6), key=lambda e: -float(s[t, e]))[:2]
        differs += sorted(free) != sorted(want)
    # with one group kept of three the second choice is often not the second largest
    one = {"router": {"experts": 6, "top": 2, "groups": {"count": 3, "keep": 1}}, "expert": f["expert"]}
    c1, _ = P.router(w, "l0.mlp.", one, u)
    assert all(len({int(e) // 2 for e in row}) == 1 for row in c1)
    assert (c1.sort(-1).values != choice.sort(-1).values).any(-1).float().mean() > 0.3


def test_registry_knows_the_design():
    from jax_vllm_amd.config.registry import supported_architectures

    assert "Fezuzen" in supported_architectures()
    assert SMALL_B["config"]["architecture"] == "Fezuzen"
    spec_of(config(32, 40, [layer(attention(1, 1, 4)), layer(latent(1, 4, 4, 4, 4, 8))], taps=1))
