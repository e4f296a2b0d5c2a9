"""The Bulitar decoder written out plainly: whole sequence, no cache, float64, one function per mechanism.

It shares no code with the package.  ``forward(config, weights, ids)`` takes the config.json dictionary, a
name -> tensor dictionary and one request's token ids and returns the logits of every position; with
``streams`` (a list) it also appends the residual stream after every layer run.

Notation: n tokens, stream s [n, width], s_0 = scale * E[token].  A layer run is
    s += mixer(N1 s);  s += ff(N2 s)        (a layer without a feed-forward: the first line alone)
with N(x) = (x - mean x) / sqrt(var x + eps) * w.  A stretch of layers runs several times; before each of its passes
    s <- W [s; s_0] + b_t                    (t the pass)
Mixers: ``attention`` (biased projections through short convolutions, adjacent pairs turned by YaRN angles, heads over
their root mean square after that, keys of the query's own chunk) and ``channel_delta`` (a gated delta rule that
decays channel by channel).  The feed-forward is a sum of gated experts chosen by sigmoid scores.
"""
from __future__ import annotations

import math

import torch


def rms(x, eps):
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def layer_norm(x, weight, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt(d.pow(2).mean(-1, keepdim=True) + eps) * weight


def silu(z):
    return z * torch.sigmoid(z)


# ------------------------------------------------------------------ short convolution
def short_conv(u, taps):
    """u [n, C], taps [C, K]: y_t = sum_j taps[:, j] u_(t - K + 1 + j), zeros before the start."""
    n, C = u.shape
    K = taps.shape[1]
    joined = torch.cat([torch.zeros(K - 1, C, dtype=u.dtype), u])
    y = torch.zeros(n, C, dtype=u.dtype)
    for j in range(K):
        y = y + taps[:, j] * joined[j:j + n]
    return y


# ------------------------------------------------------------------ rotation
def yarn_frequencies(base, dims, scaling):
    """-> (frequency of every pair, factor on cosine and sine)."""
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if scaling is None:
        return f, 1.0
    place = lambda turns: dims * math.log(scaling["original"] / (2 * math.pi * turns)) / (2 * math.log(base))      # noqa: E731
    lo = max(math.floor(place(scaling["fast"])), 0)
    hi = min(math.ceil(place(scaling["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / scaling["factor"] * ramp + fi * (1 - ramp))
    return out, 0.1 * math.log(scaling["factor"]) + 1.0


def turn_neighbours(x, positions, freqs, size):
    """x [n, heads, d]: numbers 2i and 2i + 1 turn together by positions * freqs[i], both results times ``size``."""
    a = positions.to(x.dtype)[:, None] * torch.tensor(freqs, dtype=x.dtype)
    cos, sin = (torch.cos(a) * size)[:, None, :], (torch.sin(a) * size)[:, None, :]
    m = 2 * len(freqs)
    out = x.clone()
    u, v = x[..., 0:m:2], x[..., 1:m:2]
    out[..., 0:m:2] = u * cos - v * sin
    out[..., 1:m:2] = v * cos + u * sin
    return out


# ------------------------------------------------------------------ attention
def visible(n, mask):
    """[n, n]: whether position i sees position j."""
    i = torch.arange(n)[:, None]
    j = torch.arange(n)[None, :]
    seen = j <= i
    if mask is not None:
        seen = seen & (i // mask["size"] == j // mask["size"])
    return seen


def attend(q, k, v, scale, seen):
    """q [n, H, d], k [n, G, d], v [n, G, dv] -> [n, H, dv]"""
    rep = q.shape[1] // k.shape[1]
    scores = torch.einsum("ihd,jhd->hij", q, k.repeat_interleave(rep, 1)) * scale
    weights = torch.softmax(scores.masked_fill(~seen[None], float("-inf")), dim=-1)
    return torch.einsum("hij,jhd->ihd", weights, v.repeat_interleave(rep, 1))


def attention_mixer(h, W, p, m, eps):
    n = h.shape[0]
    H, G, d = m["heads"], m["kv_heads"], m["dim"]
    dv = m.get("vdim", d)
    x = {}
    for name, heads, size in (("q", H, d), ("k", G, d), ("v", G, dv)):
        y = h @ W[f"{p}.{name}"].T + W[f"{p}.{name}.b"]
        if m.get("conv") is not None:
            y = short_conv(y, W[f"{p}.{name}.conv"])
        x[name] = y.view(n, heads, size)
    if m.get("rot") is not None:
        freqs, size = yarn_frequencies(m["rot"]["base"], m["rot"]["dims"], m["rot"].get("scaling"))
        for name in "qk":
            x[name] = turn_neighbours(x[name], torch.arange(n), freqs, size)
    o = attend(rms(x["q"], eps), rms(x["k"], eps), x["v"], m["scale"], visible(n, m.get("mask")))
    return o.reshape(n, H * dv) @ W[f"{p}.o"].T + W[f"{p}.o.b"]


# ------------------------------------------------------------------ delta rule with a decay a channel
def unit(x):
    return x / torch.sqrt(x.pow(2).sum(-1, keepdim=True) + 1e-6)


def delta_scan(q, k, v, g, beta, state=None):
    """q, k [n, H, d], v [n, H, dv], decays g [n, H, d], beta [n, H] -> (o [n, H, dv], S [H, d, dv])"""
    n, H, d = q.shape
    S = torch.zeros(H, d, v.shape[-1], dtype=q.dtype) if state is None else state.clone()
    out = []
    for t in range(n):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - torch.einsum("hij,hi->hj", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        out.append(torch.einsum("hij,hi->hj", S, q[t]))
    return torch.stack(out), S


def channel_decay(h, W, p, H, d):
    z = (h @ W[f"{p}.a1"].T) @ W[f"{p}.a2"].T + W[f"{p}.dt_bias"]
    rate = torch.exp(W[f"{p}.A_log"])[:, None]
    return torch.exp(-rate * torch.nn.functional.softplus(z, threshold=60).view(-1, H, d))


def channel_delta_mixer(h, W, p, m, eps):
    n = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    x = {}
    for name, heads, size in (("q", G, d), ("k", G, d), ("v", H, dv)):
        y = h @ W[f"{p}.{name}"].T
        if m.get("conv") is not None:
            y = short_conv(y, W[f"{p}.{name}.conv"])
        x[name] = silu(y).view(n, heads, size)
    q = unit(x["q"]).repeat_interleave(H // G, 1) * d ** -0.5
    k = unit(x["k"]).repeat_interleave(H // G, 1)
    o, _ = delta_scan(q, k, x["v"], channel_decay(h, W, p, H, d), torch.sigmoid(h @ W[f"{p}.b"].T))
    gate = torch.sigmoid((h @ W[f"{p}.g1"].T) @ W[f"{p}.g2"].T)
    return ((rms(o, eps) * W[f"{p}.norm"]).reshape(n, H * dv) * gate) @ W[f"{p}.o"].T


# ------------------------------------------------------------------ feed-forward
def choose(h, W, p, top, scale, margins=None):
    """-> (experts [n, top], their weights); ``margins`` (a list) gets every token's distance from another choice"""
    s = torch.sigmoid(h @ W[f"{p}.router"].T)
    by = s + W[f"{p}.correction"]
    picked = torch.topk(by, top, dim=-1).indices
    if margins is not None and top < s.shape[-1]:
        order = by.sort(-1, descending=True).values
        margins += (order[:, top - 1] - order[:, top]).tolist()
    return picked, torch.gather(s, 1, picked) * scale


def expert(x, W, p):
    return (silu(x @ W[f"{p}.gate"].T) * (x @ W[f"{p}.up"].T)) @ W[f"{p}.down"].T


def experts_ff(h, W, p, m, margins=None):
    r = m["router"]
    picked, share = choose(h, W, p, r["top"], r["scale"], margins)
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for j in range(r["top"]):
            y[t] += share[t, j] * expert(h[t], W, f"{p}.e{int(picked[t, j])}")
    return y


# ------------------------------------------------------------------ the model
def run_order(config):
    """-> (layer, pass that begins with it or None) in the order of the run"""
    n, loop = len(config["layers"]), config.get("loop")
    if loop is None:
        return [(i, None) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    passes = [(i, t if i == a else None) for t in range(loop["times"]) for i in range(a, b)]
    return [(i, None) for i in range(a)] + passes + [(i, None) for i in range(b, n)]


def begin_pass(s, first, W, t):
    return torch.cat([s, first], dim=-1) @ W["loop.in"].T + W["loop.step"][t]


def forward(config, weights, ids, streams=None, dtype=torch.float64, margins=None):
    W = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in weights.items()}
    eps = config["norm"]["eps"]
    first = W["embed"][torch.as_tensor(ids, dtype=torch.long)] * config["embedding"]["scale"]
    s = first
    for i, t in run_order(config):
        layer, p = config["layers"][i], f"l{i}"
        if t is not None:
            s = begin_pass(s, first, W, t)
        mixer = {"attention": attention_mixer, "channel_delta": channel_delta_mixer}[layer["type"]]
        s = s + mixer(layer_norm(s, W[f"{p}.norm1"], eps), W, f"{p}.mix", layer["mixer"], eps)
        if layer.get("mlp") is not None:
            s = s + experts_ff(layer_norm(s, W[f"{p}.norm2"], eps), W, f"{p}.mlp", layer["mlp"], margins)
        if streams is not None:
            streams.append(s.clone())
    return layer_norm(s, W["final.norm"], eps) @ W["head"].T
