"""Plain, slow, whole-sequence Kuditar in torch: the oracle of the test-suite for that design.

No cache, no batching, no kernels, one function per mechanism, nothing imported from the product
package.  A model is ``(config dict, {tensor name: tensor})``; every function works in the type of
the tensors it is given (float32, or float64 for a tighter oracle).  Recurrences run token by token.

The design in this file's notation (n tokens, width w):

* layer:       x += mixer(L1(x));  x += ff(L2(x)) (with a feed-forward);  L(y) = (y - m) / sqrt(var + eps) * a + b
* attention:   q, k rotated (frequencies over a factor), THEN each head by its own root mean square without a weight;
               score c tanh(scale q.k / c); softmax over all earlier keys; from the second mixing layer on the values
               are (1 - l) v + l v_first with v_first those of the first mixing layer; heads * sigmoid(gate), projected
* parallel:    [attention with biases, weighted head norm before the rotation, capped scores, a window that also keeps the
               first tokens, a sink] and [gated delta rule] side by side
* parallel_2:  [attention with biases, weighted head norm, no rotation, blocks of positions] and [linear attention whose
               decay sigmoid(z)^(1/tau) acts per key channel, read after the write] side by side
               either pair gives (a + b) / 2, a and b the sides' results under RMS norms of their own
* feed-forward: W_down (g sigmoid(1.702 g) (u + 1)) with g = min(gate, c), u = clamp(up, -c, c), dense or as experts: the
               ``top`` experts by sigmoid(z) + correction, weighed by sigmoid(z) times a constant
* output:      L(x), logits = embed @ that
"""
from __future__ import annotations

import json
from pathlib import Path

import torch
import torch.nn.functional as F


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
_ROUND_TO = None     # see ``rounded_products``


class rounded_products:
    """Within this context every matrix product's result (and what else an activation tensor holds between two products)
    is rounded to ``dtype`` and widened again: the least that an implementation with bfloat16 activations does to the
    numbers; the measure of the bfloat16 tests' tolerances."""

    def __init__(self, dtype=torch.bfloat16):
        self.dtype = dtype

    def __enter__(self):
        global _ROUND_TO
        self.before, _ROUND_TO = _ROUND_TO, self.dtype

    def __exit__(self, *exc):
        global _ROUND_TO
        _ROUND_TO = self.before


def rounded(y):
    return y if _ROUND_TO is None else y.to(_ROUND_TO).to(y.dtype)


def linear(x, w, b=None):
    """w is stored [out, in]."""
    y = x @ w.T
    return rounded(y if b is None else y + b)


def by_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def layer_norm(x, weight, bias, eps):
    d = x - x.mean(-1, keepdim=True)
    return rounded(d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * weight + bias)


def silu(z):
    return z * torch.sigmoid(z)


def short_conv(x, taps_w):
    """x [n, channels]; taps_w [channels, taps], the last column weighs the current token, zeros before the first."""
    n, c = x.shape
    taps = taps_w.shape[1]
    padded = torch.cat([x.new_zeros(taps - 1, c), x], dim=0)
    y = x.new_zeros(n, c)
    for j in range(taps):
        y = y + padded[j:j + n] * taps_w[:, j]
    return y


def rotate(x, rot: dict):
    """x [heads, tokens, size]: the first rot['dims'] elements turn by position (element i with i + dims/2), the others
    pass; base^(-2i/dims), over scaling.factor where there is one.  Angles in 32-bit."""
    dims = int(rot["dims"])
    f = torch.tensor([float(rot["base"]) ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=torch.float64)
    if rot.get("scaling"):
        f = f / float(rot["scaling"]["factor"])
    ang = torch.arange(x.shape[1], dtype=torch.float32)[:, None] * f.to(torch.float32)[None, :]
    cos, sin = torch.cos(ang).to(x.dtype), torch.sin(ang).to(x.dtype)
    u, v, rest = x[..., : dims // 2], x[..., dims // 2: dims], x[..., dims:]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, rest], dim=-1)


# --------------------------------------------------------------------------- attention
def visible_window(n: int, size=None, keep_first: int = 0):
    """[query, key]: every earlier key, or those at most size - 1 back and the first ``keep_first``."""
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    seen = j <= i
    return seen if size is None else seen & ((i - j < size) | (j < keep_first))


def visible_chunk(n: int, size=None):
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    seen = j <= i
    return seen if size is None else seen & (i // size == j // size)


def capped(s, cap):
    return s if not cap else cap * torch.tanh(s / cap)


def weigh(q, k, v, seen, scale: float, cap=None, sink=None):
    """q [H, n, d], k [G, n, d], v [G, n, dv], seen [n, n]; returns [n, H * dv]."""
    H, n, _ = q.shape
    per = H // k.shape[0]
    k, v = k.repeat_interleave(per, dim=0), v.repeat_interleave(per, dim=0)
    s = capped((q @ k.transpose(1, 2)) * scale, cap).masked_fill(~seen, float("-inf"))
    if sink is not None:
        s = torch.cat([s, sink.view(H, 1, 1).expand(H, n, 1)], dim=-1)
    p = torch.softmax(s, dim=-1)[..., :n]
    return rounded((p @ v).transpose(0, 1).reshape(n, -1))


def heads_of(y, count: int):
    return y.view(y.shape[0], count, -1).transpose(0, 1)


def seen_by(shared: dict, seen):
    """The layer's own mask, or the one a test puts in its place."""
    return seen if shared.get("mask") is None else shared["mask"]


def attention(w: dict, p: str, m: dict, h, eps: float, shared: dict):
    H, G = int(m["heads"]), int(m["kv_heads"])
    q, k = heads_of(linear(h, w[p + "q"]), H), heads_of(linear(h, w[p + "k"]), G)
    v = heads_of(linear(h, w[p + "v"]), G)
    if m.get("rot"):
        q, k = rotate(q, m["rot"]), rotate(k, m["rot"])
    q, k = rounded(by_rms(q, eps)), rounded(by_rms(k, eps))
    if m.get("v_mix"):
        if "v_first" in shared:
            lam = w[p + "vmix"].reshape(())
            v = rounded((1 - lam) * v + lam * shared["v_first"])
        else:
            shared["v_first"] = v
    o = weigh(q, k, v, seen_by(shared, visible_window(h.shape[0])), float(m["scale"]), m.get("softcap"))
    return linear(rounded(o * torch.sigmoid(linear(h, w[p + "g"]))), w[p + "o"])


def side_attention(w: dict, p: str, m: dict, h, eps: float, seen):
    """The left side of either pair: biases, weighted norm per head before the rotation."""
    H, G = int(m["heads"]), int(m["kv_heads"])
    q, k, v = (heads_of(linear(h, w[p + s], w[p + s + ".b"]), c) for s, c in (("q", H), ("k", G), ("v", G)))
    q, k = by_rms(q, eps) * w[p + "q.norm"], by_rms(k, eps) * w[p + "k.norm"]
    if m.get("rot"):
        q, k = rotate(q, m["rot"]), rotate(k, m["rot"])
    o = weigh(rounded(q), rounded(k), v, seen, float(m["scale"]), m.get("softcap"), w.get(p + "sink"))
    return linear(o, w[p + "o"])


def kept_window_attention(w, p, m, h, eps, shared):
    mask = m.get("mask") or {}
    seen = visible_window(h.shape[0], mask.get("size"), int(mask.get("keep_first") or 0))
    return side_attention(w, p, m, h, eps, seen_by(shared, seen))


def chunked_attention(w, p, m, h, eps, shared):
    return side_attention(w, p, m, h, eps, seen_by(shared, visible_chunk(h.shape[0], (m.get("mask") or {}).get("size"))))


# --------------------------------------------------------------------------- recurrences
def delta_walk(q, k, v, g, beta):
    """q, k [n, G, d], v [n, H, dv], g, beta [n, H]; returns [n, H, dv]."""
    n, H, dv = v.shape
    per = H // q.shape[1]
    out = v.new_zeros(n, H, dv)
    for hd in range(H):
        S = v.new_zeros(q.shape[2], dv)
        for t in range(n):
            S = g[t, hd] * S
            u = beta[t, hd] * (v[t, hd] - S.T @ k[t, hd // per])
            S = S + torch.outer(k[t, hd // per], u)
            out[t, hd] = S.T @ q[t, hd // per]
    return out


def gated_delta(w: dict, p: str, m: dict, h, eps: float):
    n = h.shape[0]
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    q, k, v = (rounded(silu(short_conv(linear(h, w[p + s]), w[p + s + ".conv"]))) for s in "qkv")
    q, k = (y.view(n, G, d) / torch.sqrt((y.view(n, G, d) ** 2).sum(-1, keepdim=True) + 1e-6) for y in (q, k))
    beta = torch.sigmoid(h @ w[p + "b"].T)
    g = torch.exp(-torch.exp(w[p + "A_log"]) * F.softplus(h @ w[p + "a"].T + w[p + "dt_bias"], threshold=1e9))
    o = by_rms(delta_walk(q * d ** -0.5, k, v.view(n, H, dv), g, beta), eps) * w[p + "norm"]
    return linear(rounded(o.reshape(n, H * dv) * silu(linear(h, w[p + "g"]))), w[p + "o"])


def channel_decay_walk(q, k, v, a):
    """q, k, a [n, H, d], v [n, H, dv]: S <- diag(a) S + k v^T, read after the write; returns [n, H, dv]."""
    n, H, dv = v.shape
    out = v.new_zeros(n, H, dv)
    for hd in range(H):
        S = v.new_zeros(q.shape[2], dv)
        for t in range(n):
            S = a[t, hd][:, None] * S + torch.outer(k[t, hd], v[t, hd])
            out[t, hd] = S.T @ q[t, hd]
    return out


def gated_linear(w: dict, p: str, m: dict, h, eps: float):
    n = h.shape[0]
    H, d, dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q, k = linear(h, w[p + "q"]).view(n, H, d) * d ** -0.5, linear(h, w[p + "k"]).view(n, H, d)
    v = linear(h, w[p + "v"]).view(n, H, dv)
    z = linear(linear(h, w[p + "a1"]), w[p + "a2"]) + w[p + "a2.b"]
    a = (torch.sigmoid(z) ** (1.0 / float(m["tau"]))).view(n, H, d)
    o = by_rms(channel_decay_walk(q, k, v, a), eps) * w[p + "norm"]
    return linear(rounded(o.reshape(n, H * dv) * silu(linear(h, w[p + "g"]))), w[p + "o"])


def side_by_side(left, right):
    def run(w, p, m, h, eps, shared):
        a = by_rms(left(w, p + "left.", m["left"], h, eps, shared), eps) * w[p + "left.out"]
        b = by_rms(right(w, p + "right.", m["right"], h, eps), eps) * w[p + "right.out"]
        return (a + b) / 2
    return run


MIXERS = {"attention": attention, "parallel": side_by_side(kept_window_attention, gated_delta),
          "parallel_2": side_by_side(chunked_attention, gated_linear)}


# --------------------------------------------------------------------------- feed-forward
def clamped_glu(gate, up, limit: float):
    g, u = gate.clamp(max=limit), up.clamp(-limit, limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1)


def glu_ff(w: dict, p: str, limit: float, h):
    return linear(rounded(clamped_glu(linear(h, w[p + "gate"]), linear(h, w[p + "up"]), limit)), w[p + "down"])


def route(z, correction, top: int, scale: float):
    """(chosen [n, top], weights [n, top])."""
    s = torch.sigmoid(z)
    chosen = torch.topk(s + correction, top, dim=-1).indices
    return chosen, s.gather(1, chosen) * scale


def feed_forward(w: dict, p: str, f: dict, h):
    if f.get("kind", "dense") == "dense":
        return glu_ff(w, p, float(f["limit"]), h)
    r = f["router"]
    chosen, weights = route(h @ w[p + "router"].T, w[p + "correction"], int(r["top"]), float(r.get("scale", 1.0)))
    out = torch.zeros_like(h)
    for e in range(int(r["experts"])):
        rows, which = (chosen == e).nonzero(as_tuple=True)
        if len(rows):
            out[rows] += weights[rows, which, None] * glu_ff(w, f"{p}e{e}.", float(f["expert"]["limit"]), h[rows])
    return out


# --------------------------------------------------------------------------- the model
def forward(w: dict, cfg: dict, tokens, layers_out: list | None = None, masks: dict | None = None):
    """Logits [n, vocab] of one sequence from position 0; with ``layers_out`` the residual stream after
    every layer is appended to it; ``masks`` {layer: [n, n]} replaces what some layers' queries see."""
    eps = float(cfg["norm"]["eps"])
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)] * float((cfg.get("embedding") or {}).get("scale", 1.0))
    shared: dict = {}
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        shared["mask"] = (masks or {}).get(i)
        h = layer_norm(x, w[p + "norm1"], w[p + "norm1.b"], eps)
        x = x + MIXERS[layer["type"]](w, p + "mix.", layer["mixer"], h, eps, shared)
        if layer.get("mlp") is not None:
            x = x + feed_forward(w, p + "mlp.", layer["mlp"], layer_norm(x, w[p + "norm2"], w[p + "norm2.b"], eps))
        if layers_out is not None:
            layers_out.append(x.clone())
    return layer_norm(x, w["final.norm"], w["final.norm.b"], eps) @ w["embed"].T
