"""Plain, slow restatement of the Fivitar and Fekulix decoders on the CPU (torch, float64 by default).

TEST INFRASTRUCTURE ONLY: one function per mechanism, every recurrence walked token by token, every attention row
formed on its own.  Shares no code with the product path (``decdec_amd``), which never imports it.

Tensors of one sequence are [tokens, channels]; ``w`` is a dict of weight tensors by name.
"""
from __future__ import annotations

import math

import torch


# ---- small pieces ----------------------------------------------------------------------------------------
def rms_norm(x, weight, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * weight


def silu(z):
    return z / (1 + torch.exp(-z))


def sigmoid(z):
    return 1 / (1 + torch.exp(-z))


def softplus(z):
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


def xielu(z, p, q):
    """Quadratic above zero, exponential below, both with slope 1/2 at zero; p and q pass a softplus."""
    up = softplus(p) * z * z + z / 2
    neg = torch.clamp(z, max=0)
    down = (0.5 + softplus(q)) * (torch.exp(neg) - 1 - neg) + neg / 2
    return torch.where(z > 0, up, down)


def gelu_tanh(z):
    return z / 2 * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def dynamic_tanh(x, alpha, weight, bias):
    return torch.tanh(alpha * x) * weight + bias


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


# ---- rotary positions ------------------------------------------------------------------------------------
def rotary_frequencies(dims, base, scaling=None):
    """(frequency of every pair, magnitude of cos and sin)."""
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if scaling is None:
        return f, 1.0
    factor, original = scaling["factor"], scaling["original"]

    def dim_of(turns):
        return dims * math.log(original / (2 * math.pi * turns)) / (2 * math.log(base))
    lo = max(math.floor(dim_of(scaling["fast"])), 0)
    hi = min(math.ceil(dim_of(scaling["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / factor * ramp + fi * (1 - ramp))
    return out, 0.1 * math.log(factor) + 1.0


def rotate(x, positions, rot):
    """x [..., tokens, n]: pairs (2i, 2i + 1) of the first rot['dims'] elements turned by position * frequency."""
    freq, mag = rotary_frequencies(rot["dims"], rot["base"], rot.get("scaling"))
    y = x.clone()
    for i, f in enumerate(freq):
        ang = positions.to(x.dtype) * f
        c, s = torch.cos(ang) * mag, torch.sin(ang) * mag
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        y[..., 2 * i] = u * c - v * s
        y[..., 2 * i + 1] = v * c + u * s
    return y


# ---- recurrences -----------------------------------------------------------------------------------------
def decayed_sum(q, k, v, decay, state=None):
    """q, k [T, H, D], v [T, H, V], decay [H]: S <- decay S + k v^T, o = S^T q."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=q.dtype) if state is None else state
    out = []
    for t in range(T):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out), S


def channel_decayed_sum(q, k, v, g, state=None):
    """q, k, g [T, H, D], v [T, H, V]: S <- diag(g) S + k v^T, o = S^T q."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=q.dtype) if state is None else state
    out = []
    for t in range(T):
        S = g[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out), S


def channel_delta_rule(q, k, v, g, beta, state=None):
    """The delta rule with one decay per head and key channel: g [T, H, D]."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=q.dtype) if state is None else state
    out = []
    for t in range(T):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out), S


def delta_rule(q, k, v, g, beta, state=None):
    """q, k [T, H, D], v [T, H, V], g, beta [T, H]: S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=q.dtype) if state is None else state
    out = []
    for t in range(T):
        S = g[t][:, None, None] * S
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out), S


def causal_conv(x, taps):
    """x [T, C], taps [C, n]: y[t] = sum_j taps[:, j] x[t - (n - 1) + j], zeros before the start."""
    T, n = x.shape[0], taps.shape[1]
    y = torch.zeros_like(x)
    for t in range(T):
        for j in range(n):
            s = t - (n - 1) + j
            if s >= 0:
                y[t] += taps[:, j] * x[s]
    return y


# ---- mixers ----------------------------------------------------------------------------------------------
def lightning(h, w, cfg, eps):
    T, H, D, V = h.shape[0], cfg["heads"], cfg["dim"], cfg["vdim"]
    q, k, v = (silu(h @ w[n].T).view(T, H, -1) for n in "qkv")
    o, _ = decayed_sum(q, k, v, torch.tensor(cfg["decay"], dtype=h.dtype))
    o = rms_norm(o.reshape(T, H * V), w["norm"], eps) * sigmoid(h @ w["g"].T)
    return o @ w["o"].T


def latent_attention(h, w, cfg, eps):
    T, H, D, R, V, C = h.shape[0], cfg["heads"], cfg["dim"], cfg["rot_dim"], cfg["vdim"], cfg["kv_rank"]
    pos = torch.arange(T)
    q = (h @ w["q"].T).view(T, H, D + R).transpose(0, 1)
    qn, qr = q[..., :D], rotate(q[..., D:], pos, cfg["rot"])
    down = h @ w["dkv"].T
    c = rms_norm(down[:, :C], w["dkv.norm"], eps)
    kr = rotate(down[:, C:], pos, cfg["rot"])
    kn = (c @ w["uk"].T).view(T, H, D).transpose(0, 1)
    v = (c @ w["uv"].T).view(T, H, V).transpose(0, 1)
    out = torch.zeros(T, H, V, dtype=h.dtype)
    for head in range(H):
        for i in range(T):
            s = (kn[head, :i + 1] @ qn[head, i] + kr[:i + 1] @ qr[head, i]) * cfg["scale"]
            m = torch.maximum(s.max(), w["sink"][head])
            e = torch.exp(s - m)
            out[i, head] = (e[:, None] * v[head, :i + 1]).sum(0) / (e.sum() + torch.exp(w["sink"][head] - m))
    return out.reshape(T, H * V) @ w["o"].T


def delta(h, w, cfg, eps):
    T, H, G, D, V = h.shape[0], cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"]
    q, k, v = (silu(causal_conv(h @ w[n].T, w[n + ".conv"])) for n in "qkv")
    q = unit(q.view(T, G, D)) * D ** -0.5
    k = unit(k.view(T, G, D))
    q, k = q.repeat_interleave(H // G, 1), k.repeat_interleave(H // G, 1)
    beta = sigmoid(h @ w["b"].T)
    g = torch.exp(-torch.exp(w["A_log"]) * softplus(h @ w["a"].T + w["dt_bias"]))
    o, _ = delta_rule(q, k, v.view(T, H, V), g, beta)
    o = rms_norm(o, w["norm"], eps) * silu(h @ w["g"].T).view(T, H, V)
    return o.reshape(T, H * V) @ w["o"].T


def sink_attention(q, k, v, scale, sink=0.0):
    """q [H, T, D], k [G, T, D], v [G, T, V]: causal softmax attention, query head h on key head h // (H / G), with a
    valueless score `sink` in the denominator; [T, H, V]."""
    H, T, _ = q.shape
    share = H // k.shape[0]
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for h in range(H):
        kh, vh = k[h // share], v[h // share]
        for i in range(T):
            s = kh[:i + 1] @ q[h, i] * scale
            m = max(float(s.max()), sink)
            e = torch.exp(s - m)
            out[i, h] = (e[:, None] * vh[:i + 1]).sum(0) / (e.sum() + math.exp(sink - m))
    return out


def gated_attention(h, w, cfg, eps):
    """Grouped-query attention with partly rotated queries and keys: read-out.  Normed queries and keys where w has their
    weights, one gate per head where it has one, a sink of score 0 unless cfg says otherwise (None: none)."""
    T, H, G, D, V = h.shape[0], cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"]
    pos = torch.arange(T)
    q, k, v = ((h @ w[n].T).view(T, g, -1) for n, g in (("q", H), ("k", G), ("v", G)))
    if "q.norm" in w:
        q, k = rms_norm(q, w["q.norm"], eps), rms_norm(k, w["k.norm"], eps)
    sink = cfg.get("sink", 0.0)
    o = sink_attention(rotate(q.transpose(0, 1), pos, cfg["rot"]), rotate(k.transpose(0, 1), pos, cfg["rot"]), v.transpose(0, 1),
                       cfg["scale"], -math.inf if sink is None else sink)
    if "g" in w:
        o = o * sigmoid(h @ w["g"].T)[:, :, None]
    return o.reshape(T, H * V)


def gated_linear(h, w, cfg, eps):
    """Gated linear attention with a decay per key channel: read-out."""
    T, H, D, V = h.shape[0], cfg["heads"], cfg["dim"], cfg["vdim"]
    q, k, v = ((h @ w[n].T).view(T, H, -1) for n in "qkv")
    z = (h @ w["a1"].T) @ w["a2"].T + w["a2.b"]
    decay = torch.exp(-softplus(-z) / cfg["tau"]).view(T, H, D)
    o, _ = channel_decayed_sum(q * D ** -0.5, k, v, decay)
    return rms_norm(o, w["norm"], eps).reshape(T, H * V) * silu(h @ w["g"].T)


def parallel(h, w, cfg, eps):
    part = lambda side: {n[len(side) + 1:]: t for n, t in w.items() if n.startswith(side + ".")}
    left, right = part("left"), part("right")
    a = gated_attention(h, left, cfg["left"], eps) @ left["o"].T
    b = gated_linear(h, right, cfg["right"], eps) @ right["o"].T
    return cfg["left_scale"] * a + cfg["right_scale"] * b


def channel_delta(h, w, cfg, eps):
    T, H, G, D, V = h.shape[0], cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"]
    q, k, v = (silu(causal_conv(h @ w[n].T, w[n + ".conv"])) for n in "qkv")
    q, k = unit(q.view(T, G, D)) * D ** -0.5, unit(k.view(T, G, D))
    q, k = q.repeat_interleave(H // G, 1), k.repeat_interleave(H // G, 1)
    beta = sigmoid(h @ w["b"].T)
    step = softplus((h @ w["a1"].T) @ w["a2"].T + w["dt_bias"]).view(T, H, D)
    g = torch.exp(-torch.exp(w["A_log"])[:, None] * step)
    o, _ = channel_delta_rule(q, k, v.view(T, H, V), g, beta)
    o = rms_norm(o, w["norm"], eps) * sigmoid((h @ w["g1"].T) @ w["g2"].T).view(T, H, V)
    return o.reshape(T, H * V) @ w["o"].T


MIXERS = {"lightning": lightning, "latent_attention": latent_attention, "delta": delta, "parallel": parallel,
          "channel_delta": channel_delta}


# ---- the decoder -----------------------------------------------------------------------------------------
def gated(y, h, w, b):
    """Element-wise gate of a sublayer's result by the sublayer's own input."""
    return y * sigmoid(h @ w.T + b)


def fivitar_layer(x, layer, w, eps):
    """Norms and gates on the sublayers' outputs; w: the layer's tensors by name."""
    y = MIXERS[layer["type"]](x, _under(w, "mix."), layer["mixer"], eps)
    x = x + rms_norm(gated(y, x, w["rg1"], w["rg1.b"]), w["norm1"], eps)
    if layer.get("mlp") is not None:
        a = w["mlp.act"]
        y = xielu(x @ w["mlp.up"].T, a[0], a[1]) @ w["mlp.down"].T
        x = x + rms_norm(gated(y, x, w["rg2"], w["rg2.b"]), w["norm2"], eps)
    return x


def fekulix_layer(x, layer, w, eps):
    """Dynamic tanh on the sublayers' inputs."""
    x = x + MIXERS[layer["type"]](dyt(x, w, "norm1"), _under(w, "mix."), layer["mixer"], eps)
    if layer.get("mlp") is not None:
        x = x + gelu_tanh(dyt(x, w, "norm2") @ w["mlp.up"].T) @ w["mlp.down"].T
    return x


def dyt(x, w, name):
    return dynamic_tanh(x, w[name + ".alpha"], w[name], w[name + ".b"])


def _under(w, prefix):
    return {n[len(prefix):]: t for n, t in w.items() if n.startswith(prefix)}


def forward(config, weights, tokens, dtype=torch.float64, layers_out=None):
    """Logits [T, vocab] of one sequence; layers_out (a list) receives the residual stream after every layer."""
    W = {n: t.to(dtype) if t.is_floating_point() else t for n, t in weights.items()}
    eps = config["norm"]["eps"]
    fekulix = config["architecture"] == "Fekulix"
    x = W["embed"][torch.as_tensor(tokens)]
    for i, layer in enumerate(config["layers"]):
        src = i
        while config["layers"][src].get("weights_of") is not None:
            src = config["layers"][src]["weights_of"]
        x = (fekulix_layer if fekulix else fivitar_layer)(x, layer, _under(W, f"l{src}."), eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    if fekulix:
        return dyt(x, W, "final.norm") @ W["head"].T * config["logit_scale"]
    return rms_norm(x, W["final.norm"], eps) @ W["head"].T
