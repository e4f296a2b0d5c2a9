"""The Pokulorn decoder written out plainly: whole sequence, no cache, float64, one function per mechanism.

It shares no code with the package.  ``forward(config, weights, ids)`` takes the config.json dictionary, a
name -> tensor dictionary and one request's token ids and returns the logits of every position; with
``streams`` (a list) it also appends the residual stream after every layer.

Notation: n tokens, stream s [n, width].  A layer is
    s += mixer(N1 s);  s += ff(N2 s)        (a layer without a feed-forward: the first line alone)
with N(x) = x / sqrt(mean(x^2) + eps) * w.  Mixers: ``attention`` (short convolutions on the projections, normed heads,
halves turned by YaRN angles, a sliding window beside kept first tokens, a sink per head, values mixed with those of
the first layer that mixes), ``parallel`` (full attention with an elementwise output gate beside a state space with one
decay a head and step, Mamba-2), ``mlstm`` (matrix memory with exponential gates under a running maximum).  The
feed-forward is a clamped gated unit.
"""
from __future__ import annotations

import math

import torch


def rms(x, eps):
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def rms_norm(x, weight, eps):
    return rms(x, eps) * weight


def silu(z):
    return z * torch.sigmoid(z)


# ------------------------------------------------------------------ short convolution
def short_conv(u, taps, bias=None, before=None):
    """u [n, C], taps [C, K]: y_t = sum_j taps[:, j] u_(t - K + 1 + j) (+ bias); ``before`` [K - 1, C]: the inputs that came
    before (zeros at a sequence's start)."""
    n, C = u.shape
    K = taps.shape[1]
    head = torch.zeros(K - 1, C, dtype=u.dtype) if before is None else before
    joined = torch.cat([head, u])
    y = torch.zeros(n, C, dtype=u.dtype)
    for j in range(K):
        y = y + taps[:, j] * joined[j:j + n]
    return y if bias is None else y + bias


# ------------------------------------------------------------------ rotation
def yarn_frequencies(base, dims, scaling):
    """-> (frequency of every pair, factor on cosine and sine)."""
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if scaling is None:
        return f, 1.0
    turns_at = lambda t: dims * math.log(scaling["original"] / (2 * math.pi * t)) / (2 * math.log(base))      # noqa: E731
    lo = max(math.floor(turns_at(scaling["fast"])), 0)
    hi = min(math.ceil(turns_at(scaling["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / scaling["factor"] * ramp + fi * (1 - ramp))
    return out, 0.1 * math.log(scaling["factor"]) + 1.0


def turn_halves(x, positions, freqs, size):
    """x [n, heads, d]: number i turns with number i + len(freqs) by positions * freqs[i], both results times ``size``."""
    half = len(freqs)
    a = positions.to(x.dtype)[:, None] * torch.tensor(freqs, dtype=x.dtype)
    cos, sin = (torch.cos(a) * size)[:, None, :], (torch.sin(a) * size)[:, None, :]
    u, v = x[..., :half], x[..., half:2 * half]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, x[..., 2 * half:]], dim=-1)


# ------------------------------------------------------------------ attention
def visible(n, mask):
    """[n, n]: whether position i sees position j."""
    i = torch.arange(n)[:, None]
    j = torch.arange(n)[None, :]
    seen = j <= i
    if mask is not None:
        seen = seen & ((i - j < mask["size"]) | (j < mask.get("keep_first", 0)))
    return seen


def sink_softmax(scores, seen, sink=None):
    """scores [H, n, n]; ``sink`` [H]: one more term exp(sink) in every denominator."""
    s = scores.masked_fill(~seen[None], float("-inf"))
    top = s.max(-1, keepdim=True).values
    if sink is not None:
        top = torch.maximum(top, sink[:, None, None])
    e = torch.exp(s - top)
    total = e.sum(-1, keepdim=True)
    if sink is not None:
        total = total + torch.exp(sink[:, None, None] - top)
    return e / total


def attend(q, k, v, scale, seen, sink=None):
    """q [n, H, d], k [n, G, d], v [n, G, dv] -> [n, H, dv]"""
    rep = q.shape[1] // k.shape[1]
    scores = torch.einsum("ihd,jhd->hij", q, k.repeat_interleave(rep, 1)) * scale
    return torch.einsum("hij,jhd->ihd", sink_softmax(scores, seen, sink), v.repeat_interleave(rep, 1))


def mix_values(v, first, lam):
    """What a layer caches as its values when it mixes them with those of the first layer that does."""
    return v if first is None else (1.0 - lam) * v + lam * first


def queries_keys_values(h, W, p, m, eps):
    n = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m.get("vdim", m["dim"])
    out = {}
    for x, heads, size in (("q", H, d), ("k", G, d), ("v", G, dv)):
        y = h @ W[f"{p}.{x}"].T
        if m.get("conv") is not None:
            y = short_conv(y, W[f"{p}.{x}.conv"])
        out[x] = y.view(n, heads, size)
    pos = torch.arange(n)
    freqs, size = yarn_frequencies(m["rot"]["base"], m["rot"]["dims"], m["rot"].get("scaling"))
    for x in "qk":
        out[x] = turn_halves(rms_norm(out[x], W[f"{p}.{x}.norm"], eps), pos, freqs, size)
    return out["q"], out["k"], out["v"]


def attention_mixer(h, W, p, m, eps, first_values=None):
    """-> (output, the layer's own values before mixing)"""
    n = h.shape[0]
    q, k, own = queries_keys_values(h, W, p, m, eps)
    v = mix_values(own, first_values, W[f"{p}.vmix"]) if m.get("v_mix") else own
    o = attend(q, k, v, m["scale"], visible(n, m.get("mask")), W[f"{p}.sink"])
    return o.reshape(n, -1) @ W[f"{p}.o"].T, own


def gated_attention_mixer(h, W, p, m, eps):
    n = h.shape[0]
    q, k, v = queries_keys_values(h, W, p, m, eps)
    o = attend(q, k, v, m["scale"], visible(n, m.get("mask"))).reshape(n, -1)
    return (o * torch.sigmoid(h @ W[f"{p}.g"].T)) @ W[f"{p}.o"].T


# ------------------------------------------------------------------ state space (Mamba-2)
def ssm_scan(x, B, C, dt, A_log, D, state=None):
    """x [n, H, dv], B, C [n, G, N], dt [n, H] (after softplus): S = exp(-exp(A_log) dt) S + dt B x^T, y = S^T C + D x.
    -> (y [n, H, dv], S [H, N, dv])"""
    n, H, dv = x.shape
    G, N = B.shape[1], B.shape[2]
    S = torch.zeros(H, N, dv, dtype=x.dtype) if state is None else state.clone()
    out = []
    for t in range(n):
        b, c = B[t].repeat_interleave(H // G, 0), C[t].repeat_interleave(H // G, 0)
        S = torch.exp(-torch.exp(A_log) * dt[t])[:, None, None] * S + dt[t][:, None, None] * b[:, :, None] * x[t][:, None, :]
        out.append(torch.einsum("hij,hi->hj", S, c) + D[:, None] * x[t])
    return torch.stack(out), S


def grouped_rms(y, groups, eps):
    n, C = y.shape
    return rms(y.view(n, groups, C // groups), eps).view(n, C)


def ssm_mixer(h, W, p, m, eps):
    n = h.shape[0]
    H, dv, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * dv
    z, u, dt = torch.split(h @ W[f"{p}.in"].T, [inner, inner + 2 * G * N, H], dim=-1)
    u = silu(short_conv(u, W[f"{p}.conv"], W[f"{p}.conv.b"]))
    x, B, C = torch.split(u, [inner, G * N, G * N], dim=-1)
    dt = torch.nn.functional.softplus(dt + W[f"{p}.dt_bias"])
    y, _ = ssm_scan(x.view(n, H, dv), B.view(n, G, N), C.view(n, G, N), dt, W[f"{p}.A_log"], W[f"{p}.D"])
    y = grouped_rms(y.reshape(n, inner) * silu(z), m["norm_groups"], eps) * W[f"{p}.norm"]
    return y @ W[f"{p}.o"].T


# ------------------------------------------------------------------ matrix memory (mLSTM)
def mlstm_scan(q, k, v, i, f, state=None):
    """q, k [n, H, d], v [n, H, dv], log gates i, f [n, H] -> (o [n, H, dv], (S [H, d, dv], n [H, d], m [H]))"""
    n, H, d = q.shape
    dv = v.shape[-1]
    if state is None:
        S, z, m = torch.zeros(H, d, dv, dtype=q.dtype), torch.zeros(H, d, dtype=q.dtype), torch.zeros(H, dtype=q.dtype)
    else:
        S, z, m = (t.clone() for t in state)
    out = []
    for t in range(n):
        new = torch.maximum(f[t] + m, i[t])
        keep, take = torch.exp(f[t] + m - new), torch.exp(i[t] - new)
        S = keep[:, None, None] * S + take[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        z = keep[:, None] * z + take[:, None] * k[t]
        m = new
        below = torch.maximum((z * q[t]).sum(-1).abs(), torch.exp(-m)) + 1e-6
        out.append(torch.einsum("hij,hi->hj", S, q[t]) / below[:, None])
    return torch.stack(out), (S, z, m)


def mlstm_gates(h, W, p, cap):
    i = cap * torch.tanh((h @ W[f"{p}.i"].T + W[f"{p}.i.b"]) / cap)
    f = cap * torch.tanh((h @ W[f"{p}.f"].T + W[f"{p}.f.b"]) / cap)
    return i, torch.nn.functional.logsigmoid(f)


def mlstm_mixer(h, W, p, m, eps):
    n = h.shape[0]
    H, d, dv = m["heads"], m["dim"], m.get("vdim", m["dim"])
    q = (h @ W[f"{p}.q"].T).view(n, H, d) * d ** -0.5
    k = (h @ W[f"{p}.k"].T).view(n, H, d)
    v = (h @ W[f"{p}.v"].T).view(n, H, dv)
    o, _ = mlstm_scan(q, k, v, *mlstm_gates(h, W, p, m["gate_cap"]))
    o = rms(o, eps).reshape(n, H * dv) * W[f"{p}.norm"]
    return (o * torch.sigmoid(h @ W[f"{p}.g"].T)) @ W[f"{p}.o"].T


# ------------------------------------------------------------------ feed-forward
def clamped_ff(h, W, p, limit):
    g = (h @ W[f"{p}.gate"].T).clamp(max=limit)
    u = (h @ W[f"{p}.up"].T).clamp(min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ W[f"{p}.down"].T


# ------------------------------------------------------------------ the model
def forward(config, weights, ids, streams=None, dtype=torch.float64):
    W = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in weights.items()}
    eps = config["norm"]["eps"]
    s = W["embed"][torch.as_tensor(ids, dtype=torch.long)]
    first_values = None
    for i, layer in enumerate(config["layers"]):
        p, m = f"l{i}", layer["mixer"]
        h = rms_norm(s, W[f"{p}.norm1"], eps)
        if layer["type"] == "attention":
            y, own = attention_mixer(h, W, f"{p}.mix", m, eps, first_values)
            if m.get("v_mix") and first_values is None:
                first_values = own
        elif layer["type"] == "parallel":
            y = (m["left_scale"] * gated_attention_mixer(h, W, f"{p}.mix.left", m["left"], eps)
                 + m["right_scale"] * ssm_mixer(h, W, f"{p}.mix.right", m["right"], eps))
        elif layer["type"] == "mlstm":
            y = mlstm_mixer(h, W, f"{p}.mix", m, eps)
        else:
            raise ValueError(layer["type"])
        s = s + y
        if layer.get("mlp") is not None:
            s = s + clamped_ff(rms_norm(s, W[f"{p}.norm2"], eps), W, f"{p}.mlp", layer["mlp"]["limit"])
        if streams is not None:
            streams.append(s.clone())
    return rms_norm(s, W["final.norm"], eps) @ W["head"].T
