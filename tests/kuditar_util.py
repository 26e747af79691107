"""Small Kuditar configurations of the test-suite and what the tests of that design share.

The configurations differ from one another in every size and constant: widths (also no multiple of 4), head counts and
ratios, key sizes below, at and above the value sizes, part of a head turned or all of it or none, frequencies under a factor
and plain, caps on scores near and far from them and none, windows and blocks of one, of a few and of more tokens than any
prompt and none, no first tokens kept, one, less and more than a page and than the window, layers that blend values and
layers that do not, convolutions of 1 to 8 taps, ranks and exponents of the decay, one, some or all experts chosen, limits
that clamp much and never, the embedding's constant, layers without a feed-forward, and the order of the mixers.
"""
import numpy as np
import torch

from tests.lomozen_util import check_rows  # noqa: F401  (the same judgement of rows serves every design)
from tests.plain import kuditar_plain as P


def heads(count, kv_heads, dim, vdim=None, scale=None, rot=None, factor=None, softcap=None):
    """The keys that the softmax attentions share; ``rot`` (dims, base)."""
    m = {"heads": count, "kv_heads": kv_heads, "dim": dim, "vdim": vdim or dim, "scale": scale if scale is not None else dim ** -0.5}
    if rot:
        m["rot"] = {"dims": rot[0], "base": rot[1]}
        if factor:
            m["rot"]["scaling"] = {"factor": factor}
    if softcap:
        m["softcap"] = softcap
    return m


def attention(*args, v_mix=None, **kw):
    m = heads(*args, **kw)
    if v_mix is not None:
        m["v_mix"] = v_mix
    return {"type": "attention", "mixer": m}


def window_side(*args, size=None, keep=None, **kw):
    m = heads(*args, **kw)
    if size:
        m["mask"] = {"size": size}
        if keep is not None:
            m["mask"]["keep_first"] = keep
    return m


def delta_side(count, kv_heads, dim, vdim, conv=4):
    return {"heads": count, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}


def block_side(*args, size=None, **kw):
    m = heads(*args, **kw)
    if size:
        m["mask"] = {"size": size}
    return m


def linear_side(count, dim, vdim, tau=16.0, rank=4):
    return {"heads": count, "dim": dim, "vdim": vdim, "tau": tau, "decay_rank": rank}


def parallel(left, right):
    return {"type": "parallel", "mixer": {"left": left, "right": right}}


def parallel_2(left, right):
    return {"type": "parallel_2", "mixer": {"left": left, "right": right}}


def dense(ff, limit=3.0):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(experts, top, ff, limit=3.0, scale=None):
    f = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff, "limit": limit}}
    if scale is not None:
        f["router"]["scale"] = scale
    return f


def layer(mixer, mlp=None):
    return dict(mixer, mlp=mlp)


def config(width, vocab, layers, eps=1e-5, scale=None):
    c = {"architecture": "Kuditar", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if scale is not None:
        c["embedding"] = {"scale": scale}
    return c


# everything at once: blended values from the second layer on (a layer between them does not blend), a window that keeps
# more first tokens than it is long, blocks that no page divides
SMALL_A = dict(name="A", seed=3, std=0.25, norm_std=0.1, page_size=8, config=config(48, 131, [
    layer(parallel(window_side(4, 2, 12, 8, scale=0.5, rot=(8, 500.0), softcap=4.0, size=9, keep=11), delta_side(4, 2, 8, 12, conv=3)), moe(6, 2, 24, limit=0.4, scale=1.7)),
    layer(attention(3, 1, 20, 14, scale=0.3, rot=(6, 100.0), factor=3.0, softcap=6.0, v_mix=True), dense(40, limit=0.5)),
    layer(parallel_2(block_side(2, 2, 10, 16, size=22), linear_side(3, 12, 20, tau=8.0, rank=5)), None),
    layer(attention(2, 2, 8, 24, rot=(8, 30.0)), moe(4, 1, 16)),
    layer(attention(6, 1, 16, 14, scale=0.4, rot=(16, 1000.0), factor=1.5, softcap=2.0, v_mix=True), moe(5, 5, 12, scale=0.6)),
], scale=1.5))
# nothing optional, sizes that are no multiples of 4, every earlier key seen
SMALL_B = dict(name="B", seed=4, std=0.2, norm_std=0.2, page_size=16, config=config(90, 301, [
    layer(parallel_2(block_side(3, 1, 10, 6), linear_side(2, 18, 7, tau=1.0, rank=3)), dense(35, limit=100.0)),
    layer(attention(3, 1, 10, 6), moe(5, 1, 18)),
    layer(parallel(window_side(5, 5, 6, 14), delta_side(2, 2, 18, 7, conv=5)), moe(9, 4, 11)),
], eps=1e-6))
# the sizes at which the matrix-core attention kernels run in bfloat16, a window and blocks of one token and beyond every
# prompt, one first token kept and more than a page, heads of the recurrences above a wave
SMALL_C = dict(name="C", seed=5, std=0.2, norm_std=0.05, page_size=32, config=config(64, 97, [
    layer(attention(4, 2, 32, 48, scale=0.3, rot=(32, 250000.0), factor=2.5, softcap=50.0, v_mix=True), moe(4, 2, 40, limit=0.3)),
    layer(parallel(window_side(4, 1, 64, 48, scale=0.2, rot=(32, 100000.0), size=1, keep=1), delta_side(2, 1, 72, 80, conv=8)), dense(96, limit=0.2)),
    layer(parallel_2(block_side(2, 1, 32, 64, size=1), linear_side(1, 72, 80, tau=20.0, rank=8)), moe(3, 3, 24, scale=2.0)),
    layer(attention(2, 2, 96, 48, softcap=1.5, rot=(4, 10.0), v_mix=True), None),
    layer(parallel(window_side(8, 2, 16, 16, scale=0.6, size=1000, keep=40, softcap=3.0, rot=(16, 1e4)), delta_side(4, 4, 16, 16, conv=1)), dense(24)),
    layer(parallel_2(block_side(4, 4, 16, 32, size=1000), linear_side(4, 8, 24, tau=4.0, rank=16)), moe(16, 5, 16)),
], eps=1e-4, scale=0.7))
ALL_SMALL = [SMALL_A, SMALL_B, SMALL_C]


def make_folder(small, tmp_path, patch=None):
    """A model folder with random weights; ``patch`` {tensor name: value or function of the tensor} rewrites some.  What the
    random-weights mode draws small (biases, sinks, corrections, convolutions) is drawn wider, so that all of it counts."""
    from jax_vllm_amd import write_random_model
    from safetensors.torch import load_file, save_file

    folder = write_random_model(tmp_path, small["config"], seed=small["seed"], std=small["std"], norm_std=small["norm_std"])
    path = str(folder / "model.safetensors")
    tensors = load_file(path)
    g = torch.Generator().manual_seed(small["seed"])
    for name, t in sorted(tensors.items()):
        draw = torch.randn(t.shape, generator=g)
        if name.endswith(".conv"):
            draw = draw * 0.5
            draw[:, -1] += 1.0
        elif name.endswith((".q.b", ".k.b", ".v.b")):
            draw = draw * 0.4
        elif name.endswith(".sink"):
            draw = draw + 1.0
        elif name.endswith(".correction"):
            draw = draw * 0.2
        elif not name.endswith(("norm1.b", "norm2.b")):
            continue
        else:
            draw = draw * 0.3
        tensors[name] = draw.to(t.dtype)
    for name, change in (patch or {}).items():
        t = tensors[name]
        new = change(t.float()) if callable(change) else torch.full_like(t.float(), float(change))
        tensors[name] = new.to(t.dtype).contiguous()
    save_file(tensors, path)
    return folder


def plain_of(folder, dtype=torch.float64):
    return P.read_config(folder), P.read_weights(folder, dtype)


def plain_logits(cfg, w, tokens, **kw):
    return P.forward(w, cfg, tokens, **kw).to(torch.float32).numpy()


def expected(cfg, w, tokens, dtype):
    """What ``check_rows`` compares with: the plain logits, and for bfloat16 also the plain logits with every
    matrix product rounded to bfloat16 (the model's own sensitivity to that rounding)."""
    want = plain_logits(cfg, w, tokens)
    if dtype in ("float32", "fp32"):
        return want
    with P.rounded_products(torch.bfloat16):
        return want, plain_logits(cfg, w, tokens)


def tokens_of(cfg, n, seed):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], size=n).tolist()
