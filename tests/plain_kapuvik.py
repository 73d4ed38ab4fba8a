"""A plain, slow Kapuvik in PyTorch on the CPU: whole sequences, no cache, one function per mechanism.

It is the yardstick of the tests and shares nothing with the library.  `weights` maps the checkpoint's tensor names to
tensors, `config` is the dictionary of config.json.  Everything runs in float64 unless the caller asks for the
roundings of a bfloat16 model (`rounding="bfloat16"`: what a product or an activation leaves is stored in bfloat16, or a
number: in its place random errors of that size, drawn from that seed; scores, softmax, norms, angles, decays, the
recurrences with their states and the residual sum stay as they are).

Notation: x is the residual stream [T, width]; h what a layer's two branches read; t, i a token's position, j a key's.
"""

from __future__ import annotations

import json
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
    weights = {k: v.double() for k, v in load_file(os.path.join(folder, "model.safetensors")).items()}
    return config, weights


# ---- norms, activations, rotation --------------------------------------------------------------------------------------
def over_rms(v, eps):
    return v / torch.sqrt((v * v).mean(-1, keepdim=True) + eps)


def zero_centred_norm(v, w, eps):
    return over_rms(v, eps) * (1 + w)


def silu(z):
    return z / (1 + torch.exp(-z))


def soft_cap(s, cap):
    return cap * torch.tanh(s / cap) if cap else s


def rotate(v, positions, rot, halves):
    """v [T, heads, size]: of every head's first n = rot["dims"] entries, pairs turned by position * base^(-2i/n).
    halves: pair i is entries (i, i + n/2); else entries (2i, 2i + 1)."""
    n = rot["dims"]
    freqs = torch.tensor([float(rot["base"]) ** (-2.0 * i / n) for i in range(n // 2)], dtype=torch.float64)
    angle = positions.double()[:, None] * freqs[None, :]
    cos, sin = torch.cos(angle)[:, None, :], torch.sin(angle)[:, None, :]
    first, second = (slice(0, n // 2), slice(n // 2, n)) if halves else (slice(0, n, 2), slice(1, n, 2))
    out = v.clone()
    out[..., first] = v[..., first] * cos - v[..., second] * sin
    out[..., second] = v[..., second] * cos + v[..., first] * sin
    return out


def causal(T):
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    return j <= i


def softmax_over(s, visible):
    s = s.masked_fill(~visible, float("-inf"))
    e = torch.exp(s - s.max(-1, keepdim=True).values)
    return e / e.sum(-1, keepdim=True)


# ---- attention ---------------------------------------------------------------------------------------------------------
def attention(h, w, m, positions):
    """The concatenated heads [T, heads * vdim], before the output projection."""
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rotate(_store(h @ w["q"].T).reshape(T, H, D), positions, m["rot"], halves=False)
    k = rotate(_store(h @ w["k"].T).reshape(T, G, D), positions, m["rot"], halves=False)
    q, k = _store(q), _store(k)
    v = _store(h @ w["v"].T).reshape(T, G, V)
    heads = []
    for head in range(H):
        g = head // (H // G)
        s = soft_cap((q[:, head] @ k[:, g].T) * m["scale"], m.get("softcap"))
        heads.append(_store(softmax_over(s, causal(T))) @ v[:, g])
    return _store(torch.stack(heads, dim=1).reshape(T, H * V))


def latent_attention(h, w, m, eps, positions):
    T = h.shape[0]
    H, D, P, V, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    rot = {"dims": P, "base": m["rot"]["base"]}
    q = _store(h @ w["q"].T).reshape(T, H, D + P)
    down = _store(h @ w["dkv"].T)
    c = _store(over_rms(down[:, :R], eps) * w["dkv.norm"])
    shared = _store(rotate(down[:, None, R:], positions, rot, halves=False))[:, 0]
    q_rot = _store(rotate(q[..., D:], positions, rot, halves=False))
    k = _store(c @ w["uk"].T).reshape(T, H, D)
    v = _store(c @ w["uv"].T).reshape(T, H, V)
    heads = []
    for head in range(H):
        s = (q[:, head, :D] @ k[:, head].T + q_rot[:, head] @ shared.T) * m["scale"]
        heads.append(_store(softmax_over(s, causal(T))) @ v[:, head])
    return _store(torch.stack(heads, dim=1).reshape(T, H * V)) @ w["o"].T


# ---- recurrences -------------------------------------------------------------------------------------------------------
def linear_recurrence(q, k, v, decay):
    """q, k, decay [T, H, D], v [T, H, V]: S <- diag(decay) S + k v^T; o = S^T q, from S = 0."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=q.dtype)
    out = torch.zeros_like(v)
    for t in range(T):
        S = decay[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out


def retention(h, w, m, eps, positions):
    """The normed and gated heads [T, heads * vdim], before the output projection."""
    T = h.shape[0]
    H, D, V = m["heads"], m["dim"], m["vdim"]
    q = rotate(_store(h @ w["q"].T).reshape(T, H, D), positions, m["rot"], halves=True)
    k = rotate(_store(h @ w["k"].T).reshape(T, H, D), positions, m["rot"], halves=True) * D ** -0.5
    v = _store(h @ w["v"].T).reshape(T, H, V)
    decay = torch.tensor(m["decay"], dtype=h.dtype)[None, :, None].expand(T, H, D)
    o = over_rms(linear_recurrence(q, k, v, decay), eps)
    return _store(o.reshape(T, H * V) * silu(_store(h @ w["g"].T)))


def channel_decays(h, w, m):
    """[T, heads, dim]: sigmoid of a projection through a few numbers, to the power 1 / tau."""
    z = (h @ w["a1"].T) @ w["a2"].T + w["a2.b"]
    return (torch.sigmoid(z) ** (1.0 / m["tau"])).reshape(h.shape[0], m["heads"], m["dim"])


def gla(h, w, m, eps):
    T = h.shape[0]
    H, D, V = m["heads"], m["dim"], m["vdim"]
    q = _store(h @ w["q"].T).reshape(T, H, D) * D ** -0.5
    k = _store(h @ w["k"].T).reshape(T, H, D)
    v = _store(h @ w["v"].T).reshape(T, H, V)
    o = over_rms(linear_recurrence(q, k, v, channel_decays(h, w, m)), eps) * w["norm"]
    return _store(o.reshape(T, H * V) * silu(_store(h @ w["g"].T))) @ w["o"].T


def parallel(h, w, m, eps, positions):
    left = attention(h, under(w, "left."), m["left"], positions) @ w["left.o"].T
    right = retention(h, under(w, "right."), m["right"], eps, positions) @ w["right.o"].T
    return m["left_scale"] * left + m["right_scale"] * right


# ---- feed-forward ------------------------------------------------------------------------------------------------------
def feed_forward(h, w, m):
    g = torch.clamp(_store(h @ w["gate"].T + w["gate.b"]), max=m["limit"])
    u = torch.clamp(_store(h @ w["up"].T + w["up.b"]), -m["limit"], m["limit"])
    y = g / (1 + torch.exp(-1.702 * g)) * (u + 1)
    return _store(y) @ w["down"].T + w["down.b"]


# ---- the model ---------------------------------------------------------------------------------------------------------
def run_order(config):
    """[(layer, number of the pass whose first layer this is, or None)] in the order in which layers run."""
    loop = config.get("loop")
    n = len(config["layers"])
    if not loop:
        return [(i, None) for i in range(n)]
    out = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        out += [(i, t if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
    return out + [(i, None) for i in range(loop["stop"], n)]


def under(weights, prefix):
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


def mixer(kind, h, w, m, eps, positions):
    if kind == "parallel":
        return parallel(h, w, m, eps, positions)
    if kind == "latent_attention":
        return latent_attention(h, w, m, eps, positions)
    if kind == "gla":
        return gla(h, w, m, eps)
    raise ValueError(kind)


def forward(config, weights, ids, rounding=None, layers_out=None):
    """Logits [T, vocab] of one sequence of token ids; `layers_out` (a list) receives the stream after every layer run."""
    global _store
    _store = _bf16 if rounding == "bfloat16" else (_noise(rounding) if isinstance(rounding, int) else (lambda t: t))
    try:
        eps = config["norm"]["eps"]
        ids = torch.as_tensor(ids, dtype=torch.long)
        positions = torch.arange(len(ids))
        x0 = weights["embed"][ids] * config["embedding"]["scale"]
        x = x0
        for i, entered in run_order(config):
            if entered is not None:
                x = (x + x0 if entered > 0 else x) + weights["loop.step"][entered]
            p, layer = f"l{i}.", config["layers"][i]
            h = _store(zero_centred_norm(x, weights[p + "norm1"], eps))
            y = mixer(layer["type"], h, under(weights, p + "mix."), layer["mixer"], eps, positions)
            if layer.get("mlp") is not None:
                y = y + feed_forward(h, under(weights, p + "mlp."), layer["mlp"])
            x = x + _store(y)
            if layers_out is not None:
                layers_out.append(x.clone())
        logits = _store(zero_centred_norm(x, weights["final.norm"], eps)) @ weights["head"].T
        return soft_cap(logits, config.get("logit_softcap"))
    finally:
        _store = lambda t: t  # noqa: E731


def greedy_generate(config, weights, prompt, n_new):
    ids = list(prompt)
    for _ in range(n_new):
        ids.append(int(forward(config, weights, ids)[-1].argmax()))
    return ids[len(prompt):]
