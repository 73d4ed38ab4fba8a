"""A plain, slow Zimorax in PyTorch on the CPU: whole sequences, no cache, one function per mechanism.

It is the yardstick of the tests and shares nothing with the library.  `weights` maps the checkpoint's tensor names to
tensors, `config` is the dictionary of config.json.  Everything runs in float64 unless the caller asks for the
roundings of a bfloat16 model (`rounding="bfloat16"`: what a product or an activation leaves is stored in bfloat16, or a
number: in its place random errors of that size, drawn from that seed; scores, softmax, norms, angles, decays, step sizes, the recurrences with their states and the residual sum stay as they
are).

Notation: x is the residual stream [T, width]; h what a mixer or a feed-forward reads; t, i a token's position, j a
key's.
"""

from __future__ import annotations

import json
import math
import os

import torch

_store = lambda x: x  # noqa: E731


def _bf16(x):
    return x.to(torch.bfloat16).to(x.dtype)


def _noise(seed):
    """In the place of rounding: random errors of the size that bfloat16 storage makes."""
    gen = torch.Generator().manual_seed(seed)
    return lambda x: x * (1 + (torch.rand(x.shape, generator=gen, dtype=x.dtype) * 2 - 1) * (0.75 * 2.0 ** -8))


def load_model_folder(folder):
    """(config dictionary, name -> float64 tensor) of a folder with config.json and model.safetensors."""
    from safetensors.torch import load_file

    with open(os.path.join(folder, "config.json")) as f:
        config = json.load(f)
    weights = {k: (v.double() if v.is_floating_point() else v) for k, v in load_file(os.path.join(folder, "model.safetensors")).items()}
    return config, weights


# ---- norms and activations ---------------------------------------------------------------------------------------------
def layer_norm(v, weight, eps):
    mean = v.mean(-1, keepdim=True)
    var = ((v - mean) ** 2).mean(-1, keepdim=True)
    return (v - mean) / torch.sqrt(var + eps) * weight


def over_rms(v, eps):
    return v / torch.sqrt((v * v).mean(-1, keepdim=True) + eps)


def unit(v):
    return v / torch.sqrt((v * v).sum(-1, keepdim=True) + 1e-6)


def silu(z):
    return z / (1 + torch.exp(-z))


def softplus(z):
    return torch.log1p(torch.exp(-z.abs())) + z.clamp(min=0)


def causal_conv(x, w, bias=None):
    """x [T, C], w [C, taps]: y[t, c] = bias[c] + sum_d w[c, taps - 1 - d] x[t - d, c], zeros before the start."""
    T, C = x.shape
    taps = w.shape[1]
    y = torch.zeros_like(x)
    for d in range(taps):
        if d < T:
            y[d:] += w[:, taps - 1 - d] * x[: T - d]
    return y if bias is None else y + bias


# ---- attention -----------------------------------------------------------------------------------------------------------
def yarn_frequencies(rot):
    """(frequencies, factor on cosines and sines): frequency i of a rotation stretched by `factor`, where dimensions that
    turn more than `fast` times over the original length keep theirs and those below `slow` turns are slowed down."""
    dims, base = rot["dims"], rot["base"]
    s = rot["scaling"]

    def dim_of(turns):
        return dims * math.log(s["original"] / (2 * math.pi * turns)) / (2 * math.log(base))

    lo = max(math.floor(dim_of(s["fast"])), 0)
    hi = min(math.ceil(dim_of(s["slow"])), dims - 1)
    out = []
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / s["factor"] * ramp + f * (1 - ramp))
    return out, 0.1 * math.log(s["factor"]) + 1.0


def rotate_halves(v, positions, rot):
    """v [T, heads, size]: entry i of every head's first rot["dims"] entries turned with entry i + dims/2."""
    half = rot["dims"] // 2
    freqs, gain = yarn_frequencies(rot)
    angle = positions.double()[:, None] * torch.tensor(freqs, dtype=torch.float64)[None, :]
    cos, sin = (gain * torch.cos(angle))[:, None, :], (gain * torch.sin(angle))[:, None, :]
    a, b, rest = v[..., :half], v[..., half : 2 * half], v[..., 2 * half :]
    return torch.cat([a * cos - b * sin, b * cos + a * sin, rest], dim=-1)


def talking_scores(q, k, scale, talk):
    """[H, T, T]: every head's scores against its key head, then mixed over the heads by `talk`."""
    H, G = q.shape[1], k.shape[1]
    s = torch.stack([(q[:, h] @ k[:, h // (H // G)].T) * scale for h in range(H)])
    return torch.einsum("hg,gij->hij", talk, s)


def softmax_with_null_sink(s, visible):
    """exp(s_j) / (1 + sum exp(s_j)) over the visible keys."""
    s = s.masked_fill(~visible, float("-inf"))
    top = s.max(-1, keepdim=True).values.clamp(min=0)
    e = torch.exp(s - top)
    return e / (torch.exp(-top) + e.sum(-1, keepdim=True))


def window(T, size):
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    return (i - j >= 0) & (i - j < size)


def attention(h, w, m, eps, positions):
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = _store(h @ w["q"].T + w["q.b"]).reshape(T, H, D)
    k = _store(h @ w["k"].T + w["k.b"]).reshape(T, G, D)
    v = _store(h @ w["v"].T + w["v.b"]).reshape(T, G, V)
    q = _store(rotate_halves(q, positions, m["rot"]))
    k = _store(rotate_halves(k, positions, m["rot"]))
    v = _store(over_rms(v, eps))
    s = talking_scores(q, k, m["scale"], w["talk"])
    p = softmax_with_null_sink(s, window(T, m["mask"]["size"]))
    out = torch.stack([_store(p[head]) @ v[:, head // (H // G)] for head in range(H)], dim=1)
    return _store(out.reshape(T, H * V)) @ w["o"].T


# ---- recurrences -----------------------------------------------------------------------------------------------------------
def ssd_recurrence(x, B, C, dt, A_log, D):
    """x [T, H, P], B, C [T, G, N], dt [T, H]: per head S <- exp(-exp(A_log) dt) S + dt B x^T, y = S^T C + D x."""
    T, H, P = x.shape
    G, N = B.shape[1:]
    S = torch.zeros(H, N, P, dtype=x.dtype)
    group = torch.arange(H) // (H // G)
    y = torch.zeros_like(x)
    for t in range(T):
        g = torch.exp(-torch.exp(A_log) * dt[t])
        S = g[:, None, None] * S + (dt[t][:, None] * B[t, group])[:, :, None] * x[t][:, None, :]
        y[t] = (S * C[t, group][:, :, None]).sum(1) + D[:, None] * x[t]
    return y


def gated_group_norm(y, z, weight, parts, eps):
    v = (y * silu(z)).reshape(y.shape[0], parts, -1)
    return over_rms(v, eps).reshape(y.shape) * weight


def mamba2(h, w, m, eps):
    T = h.shape[0]
    H, P, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * P
    proj = _store(h @ w["in"].T)
    z, xbc, dt = proj[:, :inner], proj[:, inner : 2 * inner + 2 * G * N], proj[:, 2 * inner + 2 * G * N :]
    xbc = _store(silu(causal_conv(xbc, w["conv"], w["conv.b"])))
    x, B, C = xbc[:, :inner], xbc[:, inner : inner + G * N], xbc[:, inner + G * N :]
    y = ssd_recurrence(x.reshape(T, H, P), B.reshape(T, G, N), C.reshape(T, G, N), softplus(dt + w["dt_bias"]), w["A_log"], w["D"])
    return _store(gated_group_norm(y.reshape(T, inner), z, w["norm"], m["norm_groups"], eps)) @ w["o"].T


def delta_recurrence(q, k, v, beta, decay):
    """q, k [T, H, D], v [T, H, V], beta, decay [T, H]: S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=q.dtype)
    out = torch.zeros_like(v)
    for t in range(T):
        S = decay[t][:, None, None] * S
        u = beta[t][:, None] * (v[t] - torch.einsum("hdv,hd->hv", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = torch.einsum("hdv,hd->hv", S, q[t])
    return out


def delta(h, w, m, eps):
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    conv = {n: _store(silu(causal_conv(_store(h @ w[n].T), w[n + ".conv"]))) for n in ("q", "k", "v")}
    share = torch.arange(H) // (H // G)
    q = (unit(conv["q"].reshape(T, G, D)) * D ** -0.5)[:, share]
    k = unit(conv["k"].reshape(T, G, D))[:, share]
    beta = torch.sigmoid(h @ w["b"].T)
    decay = torch.exp(-torch.exp(w["A_log"]) * softplus(h @ w["a"].T + w["dt_bias"]))
    o = delta_recurrence(q, k, conv["v"].reshape(T, H, V), beta, decay)
    o = over_rms(o, eps) * w["norm"] * silu(h @ w["g"].T).reshape(T, H, V)
    return _store(o.reshape(T, H * V)) @ w["o"].T


def feed_forward(h, w):
    return _store(torch.relu(_store(h @ w["up"].T + w["up.b"])) ** 2) @ w["down"].T + w["down.b"]


# ---- the model -----------------------------------------------------------------------------------------------------------
def run_order(config):
    """[(layer, pass whose first layer this is, or None)] in the order in which layers run."""
    loop = config.get("loop")
    n = len(config["layers"])
    if not loop:
        return [(i, None) for i in range(n)]
    out = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        for i in range(loop["start"], loop["stop"]):
            out.append((i, t if i == loop["start"] else None))
    return out + [(i, None) for i in range(loop["stop"], n)]


def under(weights, prefix):
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


def forward(config, weights, ids, rounding=None, layers_out=None):
    """Logits [T, vocab] of one sequence of token ids; `layers_out` (a list) receives the stream after every layer run."""
    global _store
    _store = _bf16 if rounding == "bfloat16" else (_noise(rounding) if isinstance(rounding, int) else (lambda t: t))
    try:
        eps = config["norm"]["eps"]
        ids = torch.as_tensor(ids, dtype=torch.long)
        positions = torch.arange(len(ids))
        x0 = weights["embed"][ids]
        x = x0
        for i, entered in run_order(config):
            if entered is not None:
                x = _store(torch.cat([x, x0], dim=-1)) @ weights["loop.in"].T
                x = x + weights["loop.step"][entered]
            p, layer = f"l{i}.", config["layers"][i]
            w, m = under(weights, p + "mix."), layer["mixer"]
            h = _store(layer_norm(x, weights[p + "norm1"], eps))
            if layer["type"] == "attention":
                y = attention(h, w, m, eps, positions)
            elif layer["type"] == "mamba2":
                y = mamba2(h, w, m, eps)
            elif layer["type"] == "delta":
                y = delta(h, w, m, eps)
            else:
                raise ValueError(layer["type"])
            x = x + _store(y) * weights[p + "ls1"]
            if layer.get("mlp") is not None:
                h = _store(layer_norm(x, weights[p + "norm2"], eps))
                x = x + _store(feed_forward(h, under(weights, p + "mlp."))) * weights[p + "ls2"]
            if layers_out is not None:
                layers_out.append(x.clone())
        return _store(layer_norm(x, weights["final.norm"], eps)) @ weights["head"].T
    finally:
        _store = lambda t: t  # noqa: E731


def greedy_generate(config, weights, prompt, n_new):
    ids = list(prompt)
    for _ in range(n_new):
        ids.append(int(forward(config, weights, ids)[-1].argmax()))
    return ids[len(prompt):]
