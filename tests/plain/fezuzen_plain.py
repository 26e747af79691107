"""Plain, slow, whole-sequence Fezuzen in torch: the oracle of the test-suite for that design.

No cache, no batching, no kernels, one function per mechanism, nothing imported from the
product package.  A model is ``(config dict, {tensor name: tensor})``; every function works
in the type of the tensors it is given (float32, or float64 for a tighter oracle).

The design in this file's notation (n tokens, N(x) = x / sqrt(mean(x^2) + eps) * weight):

* layer:      x += N1b(mixer(C1(N1(x))));  x += N2b(ff(C2(N2(x))))     (the second part only with a feed-forward)
* C(u)_t:     u_t + sum_j w[:, taps - 1 - j] u_{t-j},  j = 0 .. taps - 1, per channel, nothing before the first token
* attention:  grouped-query; q, k, v each through a causal filter over time per channel; the pairs (2i, 2i + 1) of the
              first ``dims`` elements of q and k turn by p base^(-2i / dims), those of all of v by p base^(-2m / vdim);
              token i sees the tokens of its own block of ``size`` positions up to itself; p_ij = exp(s_ij) /
              (1 + sum exp(s_ij)); head outputs turn back by -i base^(-2m / vdim), times sigmoid(W_g u), then W_o;
* latent attention: q = W_uq N(W_dq u) per head [plain | turned];  W_dkv u = [latent, normed | shared turned key part];
              k = [W_uk c | turned part], v = W_uv c per head; turned pairs (2i, 2i + 1), their frequencies blended
              for long contexts, cos and sin times 0.1 ln(factor) + 1; the last ``size`` tokens are seen; ordinary
              softmax; a layer with ``kv_from`` j takes c and the turned key part of layer j;
* feed-forward: s = softmax(W_router u) over all experts; groups of neighbours are ranked by their largest s and the
              best ``keep`` stay; the ``top`` largest s among them are chosen and weigh their experts' outputs as they
              are; expert(u) = W_down relu(W_up u)^2; a shared expert of the same form is added;
* output:     logits = H N(x) * logit_scale.
"""
from __future__ import annotations

import json
import math
from pathlib import Path

import torch


# --------------------------------------------------------------------------- files
def read_config(folder) -> dict:
    return json.loads((Path(folder) / "config.json").read_text())


def read_weights(folder, dtype=torch.float32) -> dict:
    from safetensors.torch import load_file

    out = {}
    for shard in sorted(Path(folder).glob("*.safetensors")):
        for k, v in load_file(str(shard)).items():
            out[k] = v.to(dtype) if v.is_floating_point() else v
    return out


# --------------------------------------------------------------------------- small pieces
def rms_norm(x, weight, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * weight


_ROUND_PRODUCTS_TO = None     # see ``rounded_products``


def rounded(y):
    return y if _ROUND_PRODUCTS_TO is None else y.to(_ROUND_PRODUCTS_TO).to(y.dtype)


def linear(x, w):
    """w is stored [out, in]."""
    return rounded(x @ w.T)


class rounded_products:
    """Within this context every matrix product's result is rounded to ``dtype`` (and widened again), and so are the
    inputs of the sublayers and what the caches keep: what an implementation that keeps its activations in bfloat16
    does to the numbers at the least."""

    def __init__(self, dtype=torch.bfloat16):
        self.dtype = dtype

    def __enter__(self):
        global _ROUND_PRODUCTS_TO
        self.before, _ROUND_PRODUCTS_TO = _ROUND_PRODUCTS_TO, self.dtype

    def __exit__(self, *exc):
        global _ROUND_PRODUCTS_TO
        _ROUND_PRODUCTS_TO = self.before


def causal_filter(u, weight):
    """u [n, channels], weight [channels, taps]: the last column weighs the token itself."""
    taps = weight.shape[1]
    out = torch.zeros_like(u)
    for lag in range(min(taps, u.shape[0])):
        out[lag:] += u[:u.shape[0] - lag] * weight[:, taps - 1 - lag]
    return out


def with_filter(u, weight):
    """A sublayer's input plus its causal filter."""
    return rounded(u + causal_filter(u, weight))


# --------------------------------------------------------------------------- rotation
def blended_frequencies(dims: int, base: float, scaling):
    i = torch.arange(dims // 2, dtype=torch.float64)
    f = torch.tensor(float(base), dtype=torch.float64) ** (-2.0 * i / dims)
    if not scaling:
        return f, 1.0

    def pair_of(turns):
        return dims * math.log(scaling["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(pair_of(scaling["fast"])), 0)
    hi = min(math.ceil(pair_of(scaling["slow"])), dims - 1)
    slowed = torch.clamp((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / scaling["factor"] * slowed + f * (1.0 - slowed), 0.1 * math.log(scaling["factor"]) + 1.0


def turn_pairs(x, angles, amplitude: float = 1.0):
    """x [n, heads, size], angles [n, pairs]: the pairs (2i, 2i + 1) of the leading elements turn."""
    dims = 2 * angles.shape[1]
    cos = (torch.cos(angles) * amplitude).to(x.dtype).unsqueeze(1)
    sin = (torch.sin(angles) * amplitude).to(x.dtype).unsqueeze(1)
    a, b = x[..., 0:dims:2], x[..., 1:dims:2]
    out = x.clone()
    out[..., 0:dims:2] = a * cos - b * sin
    out[..., 1:dims:2] = b * cos + a * sin
    return out


def rotate(x, rot: dict):
    """The rotation of queries and keys of positions 0 .. n - 1."""
    f, amp = blended_frequencies(rot["dims"], rot["base"], rot.get("scaling"))
    return turn_pairs(x, torch.arange(x.shape[0], dtype=torch.float64).view(-1, 1) * f, amp)


def turn_values(x, base: float, sign: float = 1.0):
    """All elements of every head turn by sign * position * base^(-2m / size)."""
    f, _ = blended_frequencies(x.shape[-1], base, None)
    return turn_pairs(x, sign * torch.arange(x.shape[0], dtype=torch.float64).view(-1, 1) * f)


# --------------------------------------------------------------------------- which keys are seen
def chunk_mask(n: int, size):
    i, j = torch.arange(n).view(n, 1), torch.arange(n).view(1, n)
    seen = j <= i
    return seen & (i // size == j // size) if size else seen


def window_mask(n: int, size):
    i, j = torch.arange(n).view(n, 1), torch.arange(n).view(1, n)
    seen = j <= i
    return seen & (i - j < size) if size else seen


def softmax_plus_one(scores, seen):
    """exp(s) / (1 + sum exp(s)) over the seen keys."""
    scores = scores.masked_fill(~seen, float("-inf"))
    top = torch.clamp(scores.amax(-1, keepdim=True), min=0.0)
    e = torch.exp(scores - top)
    return e / (torch.exp(-top) + e.sum(-1, keepdim=True))


# --------------------------------------------------------------------------- mixers
def mask_size(m: dict):
    return (m.get("mask") or {}).get("size")


def attention(w: dict, p: str, m: dict, u, eps: float, mask=None):
    n, H, G, D, V = u.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (rounded(causal_filter(linear(u, w[p + s]), w[p + s + ".conv"])) if m.get("conv") else linear(u, w[p + s])
               for s in "qkv")
    q = rounded(rotate(q.view(n, H, D), m["rot"]))
    k = rounded(rotate(k.view(n, G, D), m["rot"]))
    v = rounded(turn_values(v.view(n, G, V), m["rot"]["base"]))
    kh, vh = k.repeat_interleave(H // G, dim=1), v.repeat_interleave(H // G, dim=1)
    scores = torch.einsum("ihd,jhd->hij", q, kh) * m["scale"]
    probs = softmax_plus_one(scores, chunk_mask(n, mask_size(m)) if mask is None else mask)
    o = rounded(turn_values(torch.einsum("hij,jhv->ihv", probs, vh), m["rot"]["base"], -1.0))
    o = o.reshape(n, H * V) * torch.sigmoid(linear(u, w[p + "g"]))
    return linear(rounded(o), w[p + "o"])


def latent_cache(w: dict, p: str, m: dict, u, eps: float):
    """(normed latent [n, rank], turned key part [n, rot_dim]) that a latent layer with a W_dkv keeps per token."""
    rank = m["kv_rank"]
    down = linear(u, w[p + "dkv"])
    c = rounded(rms_norm(down[:, :rank], w[p + "dkv.norm"], eps))
    return c, rounded(rotate(down[:, rank:].unsqueeze(1), m["rot"]).squeeze(1))


def latent_attention(w: dict, p: str, m: dict, u, eps: float, cache, mask=None):
    n, H, D, R, V = u.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    c, kr = cache
    q = linear(rounded(rms_norm(linear(u, w[p + "dq"]), w[p + "dq.norm"], eps)), w[p + "uq"]).view(n, H, D + R)
    q_plain, q_rot = q[..., :D], rounded(rotate(q[..., D:], m["rot"]))
    k_plain = linear(c, w[p + "uk"]).view(n, H, D)
    v = linear(c, w[p + "uv"]).view(n, H, V)
    scores = (torch.einsum("ihd,jhd->hij", q_plain, k_plain) + torch.einsum("ihr,jr->hij", q_rot, kr)) * m["scale"]
    seen = window_mask(n, mask_size(m)) if mask is None else mask
    probs = torch.softmax(scores.masked_fill(~seen, float("-inf")), dim=-1)
    o = torch.einsum("hij,jhv->ihv", probs, v)
    return linear(rounded(o.reshape(n, H * V)), w[p + "o"])


# --------------------------------------------------------------------------- feed-forward
def squared_relu_ff(w: dict, p: str, u):
    z = torch.relu(linear(u, w[p + "up"]))
    return linear(rounded(z * z), w[p + "down"])


def router(w: dict, p: str, f: dict, u):
    """(chosen experts [n, top], their weights [n, top])."""
    r = f["router"]
    n, experts = u.shape[0], r["experts"]
    s = torch.softmax(u @ w[p + "router"].T, dim=-1)                       # never rounded
    allowed = torch.ones((n, experts), dtype=torch.bool)
    if r.get("groups"):
        count, keep = r["groups"]["count"], r["groups"]["keep"]
        best = s.view(n, count, experts // count).amax(-1)
        kept = torch.zeros((n, count), dtype=torch.bool)
        kept.scatter_(1, torch.topk(best, keep, dim=-1).indices, True)
        allowed = kept.repeat_interleave(experts // count, dim=1)
    choice = torch.topk(s.masked_fill(~allowed, -1.0), r["top"], dim=-1).indices
    return choice, torch.gather(s, 1, choice)


def routed_ff(w: dict, p: str, f: dict, u):
    choice, weight = router(w, p, f, u)
    out = torch.zeros_like(u)
    for e in range(f["router"]["experts"]):
        t, kk = torch.nonzero(choice == e, as_tuple=True)
        if len(t):
            out.index_add_(0, t, weight[t, kk].unsqueeze(1) * squared_relu_ff(w, f"{p}e{e}.", u[t]))
    if f.get("shared"):
        out = out + squared_relu_ff(w, p + "shared.", u)
    return out


# --------------------------------------------------------------------------- the model
def forward(w: dict, cfg: dict, tokens, streams=None, masks=None):
    """Logits [n, vocab] of one sequence from its first token; ``streams``: a list that receives the residual
    stream after every layer; ``masks`` {layer: mask [n, n]}: a test's question, what if that layer saw these keys?"""
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.tensor(list(tokens), dtype=torch.long)]
    caches = {}
    for i, layer in enumerate(cfg["layers"]):
        p, mix, mask = f"l{i}.mix.", layer["mixer"], (masks or {}).get(i)
        u = with_filter(rounded(rms_norm(x, w[f"l{i}.norm1"], eps)), w[f"l{i}.canon1"])
        if layer["type"] == "attention":
            y = attention(w, p, mix, u, eps, mask)
        elif layer["type"] == "latent_attention":
            src = mix.get("kv_from")
            if src is None:
                caches[i] = latent_cache(w, p, mix, u, eps)
            y = latent_attention(w, p, mix, u, eps, caches[i if src is None else src], mask)
        else:
            raise ValueError(layer["type"])
        x = x + rms_norm(y, w[f"l{i}.norm1b"], eps)
        if layer.get("mlp"):
            u = with_filter(rounded(rms_norm(x, w[f"l{i}.norm2"], eps)), w[f"l{i}.canon2"])
            x = x + rms_norm(routed_ff(w, f"l{i}.mlp.", layer["mlp"], u), w[f"l{i}.norm2b"], eps)
        if streams is not None:
            streams.append(x.clone())
    return linear(rounded(rms_norm(x, w["final.norm"], eps)), w["head"]) * cfg.get("logit_scale", 1.0)
