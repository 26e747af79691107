"""Small Fezuzen configurations of the test-suite and what the tests of that design share.

The configurations differ from one another in every size and constant: widths (also no multiple of 4), head counts and
ratios, key sizes below, at and above the value sizes, part of a head turned or all of it, filters of 1 to 8 taps (and
none on q, k and v), blocks and windows of 1, of a few and of more tokens than any prompt, layers that read another
layer's latent cache with a wider or narrower window, cached vectors that are and are not a size of the matrix-core
attention kernels, experts in groups (one, some or all kept) and without groups, one, some or all experts chosen, with
and without the shared expert, layers without a feed-forward, with and without the constant on the logits.
"""
import numpy as np
import torch

from tests.lomozen_util import check_rows  # noqa: F401  (the same judgement of rows serves every design)
from tests.plain import fezuzen_plain as P

LONG = {"factor": 3.0, "original": 64, "fast": 8.0, "slow": 0.5}      # rescaled frequencies whose blend lies inside a small head


def attention(heads, kv_heads, dim, vdim=None, scale=None, size=None, conv=4, rot=None):
    """``rot`` (dims, base); ``size``: positions of a block (None: every earlier key)."""
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim or dim, "scale": scale if scale is not None else dim ** -0.5,
         "rot": {"dims": rot[0] if rot else dim, "base": rot[1] if rot else 10000.0}}
    if size:
        m["mask"] = {"size": size}
    if conv:
        m["conv"] = conv
    return {"type": "attention", "mixer": m}


def latent(heads, dim, rot_dim, vdim, q_rank, rank, scale=None, size=None, rot=None, scaling=None, kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": rank,
         "scale": scale if scale is not None else (dim + rot_dim) ** -0.5,
         "rot": {"dims": rot[0] if rot else rot_dim, "base": rot[1] if rot else 10000.0}}
    if scaling:
        m["rot"]["scaling"] = scaling
    if size:
        m["mask"] = {"size": size}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m}


def moe(experts, top, ff, shared=None, groups=None):
    f = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}
    if groups:
        f["router"]["groups"] = {"count": groups[0], "keep": groups[1]}
    if shared:
        f["shared"] = {"ff": shared}
    return f


def layer(mixer, mlp=None):
    return dict(mixer, mlp=mlp)


def config(width, vocab, layers, eps=1e-5, taps=4, logit_scale=None):
    c = {"architecture": "Fezuzen", "vocab": vocab, "width": width, "norm": {"eps": eps}, "canon": {"taps": taps}, "layers": layers}
    if logit_scale is not None:
        c["logit_scale"] = logit_scale
    return c


# everything at once, a reader with a wider and one with a narrower window than the layer whose cache it reads
SMALL_A = dict(name="A", seed=3, std=0.25, norm_std=0.1, page_size=8, config=config(48, 131, [
    layer(attention(4, 2, 12, 8, scale=0.4, size=22, conv=3, rot=(8, 500.0)), moe(6, 2, 24, shared=16, groups=(3, 2))),
    layer(latent(3, 8, 4, 12, 14, 20, scale=0.3, size=9, rot=(4, 100.0), scaling=LONG), moe(4, 1, 16, groups=(2, 1))),
    layer(latent(2, 6, 4, 10, 10, 20, size=19, rot=(4, 100.0), scaling=LONG, kv_from=1), None),
    layer(attention(2, 2, 8, 16, size=5, conv=2), moe(8, 3, 12, shared=24)),
    layer(latent(4, 4, 4, 6, 6, 20, scale=0.5, size=3, rot=(4, 100.0), scaling=LONG, kv_from=1), moe(6, 6, 8, shared=8, groups=(2, 2))),
], taps=3, logit_scale=0.6))
# nothing optional, sizes that are no multiples of 4, filters of two taps, no filters on q, k and v, every earlier key seen
SMALL_B = dict(name="B", seed=4, std=0.2, norm_std=0.2, page_size=16, config=config(90, 301, [
    layer(latent(3, 10, 6, 14, 7, 18, rot=(6, 10.0)), None),
    layer(attention(3, 1, 10, 6, conv=None, rot=(4, 50.0)), moe(5, 1, 18)),
    layer(attention(5, 5, 6, 14, conv=7, rot=(6, 77.0)), moe(9, 4, 11, shared=13, groups=(3, 2))),
], eps=1e-6, taps=2))
# the sizes at which the matrix-core attention kernels run in bfloat16, long filters, a window and blocks of one token
# and windows beyond every prompt, a reader that sees every key of a windowed layer's cache
SMALL_C = dict(name="C", seed=5, std=0.2, norm_std=0.05, page_size=32, config=config(64, 97, [
    layer(latent(2, 32, 32, 48, 24, 96, size=1, rot=(16, 250000.0)), moe(4, 2, 40, shared=48, groups=(4, 2))),
    layer(attention(4, 1, 64, 48, scale=0.1, size=1, conv=8, rot=(32, 100000.0)), moe(3, 1, 24, shared=24)),
    layer(latent(4, 16, 32, 16, 40, 96, scale=0.2, rot=(16, 250000.0), kv_from=0), None),
    layer(attention(2, 1, 32, 64, size=1000, conv=4), moe(16, 5, 16, groups=(8, 3))),
    layer(latent(1, 8, 16, 80, 32, 48, size=1000, rot=(16, 30.0), scaling=dict(LONG, factor=1.5)), moe(2, 2, 8, shared=72)),
], eps=1e-4, taps=8, logit_scale=2.5))
ALL_SMALL = [SMALL_A, SMALL_B, SMALL_C]


def make_folder(small, tmp_path, patch=None):
    """A model folder with random weights; ``patch`` {tensor name: value or function of the tensor} rewrites some.  The
    filters are drawn wider than the random-weights mode draws them, so that every tap counts."""
    from jax_vllm_amd import write_random_model
    from safetensors.torch import load_file, save_file

    folder = write_random_model(tmp_path, small["config"], seed=small["seed"], std=small["std"], norm_std=small["norm_std"])
    path = str(folder / "model.safetensors")
    tensors = load_file(path)
    g = torch.Generator().manual_seed(small["seed"])
    for name, t in sorted(tensors.items()):
        if name.endswith(".conv"):
            w = torch.randn(t.shape, generator=g) * 0.5
            w[:, -1] += 1.0
            tensors[name] = w.to(t.dtype)
        if ".canon" in name:
            tensors[name] = (torch.randn(t.shape, generator=g) * 0.5).to(t.dtype)
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
