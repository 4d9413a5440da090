"""The Rofetar decoder, plainly: whole sequences, no cache, no carried state, float64, one function per
mechanism.  It shares no code with the engine and exists to be compared with it.

`config` is the decoder's config.json as a dict, `weights` a dict of float64 tensors under the
checkpoint's own names.  The `round_to` argument of `forward` makes the yardstick for ill-conditioned rows:
the same arithmetic with every product's inputs (and the queries, keys and values of the attention) rounded.
"""

from __future__ import annotations

import math
from typing import Mapping, Optional

import torch

F64 = torch.float64


def _r(x, round_to):
    return x if round_to is None else x.to(round_to).to(F64)


def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rms_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    return unit_rms(x, eps) * weight


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z**3)))


# ---- rotations ------------------------------------------------------------------------------------------

def rotary_frequencies(rot: Mapping) -> tuple[torch.Tensor, float]:
    """Turning rates of the dims/2 pairs and the amplitude of cos and sin."""
    dims = int(rot["dims"])
    base = float(rot["base"])
    i = torch.arange(dims // 2, dtype=F64)
    f = base ** (-2.0 * i / dims)
    scaling = rot.get("scaling")
    if not scaling:
        return f, 1.0
    factor = float(scaling["factor"])

    def pair_of(turns: float) -> float:
        return dims * math.log(float(scaling["original"]) / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(pair_of(float(scaling["fast"]))), 0)
    hi = min(math.ceil(pair_of(float(scaling["slow"]))), dims - 1)
    ramp = ((i - lo) / max(hi - lo, 0.001)).clamp(0.0, 1.0)
    return f / factor * ramp + f * (1.0 - ramp), 0.1 * math.log(factor) + 1.0


def rotate_halves(x: torch.Tensor, positions: torch.Tensor, rot: Mapping) -> torch.Tensor:
    """x [T, heads, d]: of the first rot.dims dims of every head, dim i turns with dim i + dims/2; the rest pass."""
    dims = int(rot["dims"])
    f, amplitude = rotary_frequencies(rot)
    angle = positions.to(F64)[:, None] * f[None, :]
    cos = (torch.cos(angle) * amplitude)[:, None, :]
    sin = (torch.sin(angle) * amplitude)[:, None, :]
    u, v = x[..., : dims // 2], x[..., dims // 2 : dims]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, x[..., dims:]], dim=-1)


# ---- mixers ---------------------------------------------------------------------------------------------

def keys_and_values(w, p: str, m: Mapping, h: torch.Tensor, eps: float, round_to=None):
    """Normed and rotated keys [T, G, d] and values [T, G, dv]."""
    T = h.shape[0]
    G, d, dv = int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    k = rms_norm((h @ w[p + "k"].T).view(T, G, d), w[p + "k.norm"], eps)
    v = (h @ w[p + "v"].T).view(T, G, dv)
    if m.get("rot"):
        k = rotate_halves(k, torch.arange(T), m["rot"])
    return _r(k, round_to), _r(v, round_to)


def softmax_plus_one(score: torch.Tensor) -> torch.Tensor:
    """exp(s_j) / (1 + sum exp(s_j)) over the last axis (hidden scores are -inf)."""
    top = torch.clamp(score.max(-1, keepdim=True).values, min=0.0)
    e = torch.exp(score - top)
    return e / (torch.exp(-top) + e.sum(-1, keepdim=True))


def attention(w, p: str, m: Mapping, h: torch.Tensor, eps: float, kept: dict, index: int, round_to=None) -> torch.Tensor:
    """Grouped heads, queries and keys normed per head and rotated, capped scores, one more in the denominator;
    keys and values of its own, or those that layer `kv_from` left in `kept`."""
    T = h.shape[0]
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    hr = _r(h, round_to)
    q = rms_norm((hr @ w[p + "q"].T).view(T, H, d), w[p + "q.norm"], eps)
    if m.get("rot"):
        q = rotate_halves(q, torch.arange(T), m["rot"])
    q = _r(q, round_to)
    if m.get("kv_from") is None:
        kept[index] = keys_and_values(w, p, m, hr, eps, round_to)
        k, v = kept[index]
    else:
        k, v = kept[int(m["kv_from"])]
    hidden = torch.triu(torch.ones(T, T, dtype=torch.bool), 1)
    cap = m.get("softcap")
    out = torch.zeros(T, H, dv, dtype=F64)
    for head in range(H):
        g = head // (H // G)
        score = (q[:, head] @ k[:, g].T) * float(m["scale"])
        if cap:
            score = float(cap) * torch.tanh(score / float(cap))
        out[:, head] = softmax_plus_one(score.masked_fill(hidden, -math.inf)) @ v[:, g]
    return _r(out.reshape(T, H * dv), round_to) @ w[p + "o"].T


def short_conv(x: torch.Tensor, taps: torch.Tensor, bias: Optional[torch.Tensor] = None) -> torch.Tensor:
    """x [T, C], taps [C, n]: y_t = sum_j taps[:, j] x_(t - n + 1 + j) (+ bias), zeros before the start."""
    T, n = x.shape[0], taps.shape[1]
    padded = torch.cat([torch.zeros(n - 1, x.shape[1], dtype=F64), x])
    y = sum(padded[j : j + T] * taps[:, j] for j in range(n))
    return y if bias is None else y + bias


def state_space(q, k, v, log_decay, write) -> torch.Tensor:
    """Per head S_t = exp(log_decay_t) S_(t-1) + write_t k_t v_t^T, o_t = S_t^T q_t.  q, k [T, H, N], v [T, H, P],
    log_decay and write [T, H]."""
    T, H, P = v.shape
    out = torch.zeros(T, H, P, dtype=F64)
    S = torch.zeros(H, k.shape[-1], P, dtype=F64)
    for t in range(T):
        S = torch.exp(log_decay[t])[:, None, None] * S + write[t][:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out


def delta_rule(q, k, v, log_decay, beta) -> torch.Tensor:
    """Per head S <- exp(log_decay) S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q."""
    T, H, P = v.shape
    out = torch.zeros(T, H, P, dtype=F64)
    S = torch.zeros(H, k.shape[-1], P, dtype=F64)
    for t in range(T):
        S = torch.exp(log_decay[t])[:, None, None] * S
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out


def mamba2(w, p: str, m: Mapping, h: torch.Tensor, eps: float, round_to=None) -> torch.Tensor:
    T = h.shape[0]
    H, P, N, G, parts = int(m["heads"]), int(m["vdim"]), int(m["state"]), int(m["groups"]), int(m["norm_groups"])
    inner = H * P
    z, x, b, c, dt = (_r(h, round_to) @ w[p + "in"].T).split([inner, inner, G * N, G * N, H], dim=-1)
    x, b, c = silu(short_conv(torch.cat([x, b, c], -1), w[p + "conv"], w[p + "conv.b"])).split([inner, G * N, G * N], dim=-1)
    dt = torch.nn.functional.softplus(dt + w[p + "dt_bias"])
    x = x.view(T, H, P)
    b = b.view(T, G, N).repeat_interleave(H // G, dim=1)
    c = c.view(T, G, N).repeat_interleave(H // G, dim=1)
    y = state_space(c, b, x, -torch.exp(w[p + "A_log"]) * dt, dt) + w[p + "D"][:, None] * x
    y = y.reshape(T, inner) * silu(z)
    y = unit_rms(y.view(T, parts, inner // parts), eps).reshape(T, inner) * w[p + "norm"]
    return _r(y, round_to) @ w[p + "o"].T


def gated_delta(w, p: str, m: Mapping, h: torch.Tensor, eps: float, round_to=None) -> torch.Tensor:
    T = h.shape[0]
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    hr = _r(h, round_to)
    q, k, v = (silu(short_conv(hr @ w[p + n].T, w[p + n + ".conv"])) for n in ("q", "k", "v"))

    def unit(x):
        return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)

    q = unit(q.view(T, G, d)).repeat_interleave(H // G, dim=1) * d**-0.5
    k = unit(k.view(T, G, d)).repeat_interleave(H // G, dim=1)
    beta = torch.sigmoid(hr @ w[p + "b"].T)
    log_decay = -torch.exp(w[p + "A_log"]) * torch.nn.functional.softplus(hr @ w[p + "a"].T + w[p + "dt_bias"])
    o = delta_rule(q, k, v.view(T, H, dv), log_decay, beta)
    o = (unit_rms(o, eps) * w[p + "norm"]).reshape(T, H * dv) * silu(hr @ w[p + "g"].T)
    return _r(o, round_to) @ w[p + "o"].T


# ---- feed-forward ---------------------------------------------------------------------------------------

def dense_ff(w, p: str, h: torch.Tensor, round_to=None) -> torch.Tensor:
    hr = _r(h, round_to)
    inner = gelu_tanh(hr @ w[p + "gate"].T + w[p + "gate.b"]) * (hr @ w[p + "up"].T + w[p + "up.b"])
    return _r(inner, round_to) @ w[p + "down"].T + w[p + "down.b"]


# ---- the model ------------------------------------------------------------------------------------------

def forward(config: Mapping, weights: Mapping[str, torch.Tensor], tokens, round_to: Optional[torch.dtype] = None):
    """logits [T, vocab] and the stream after every layer [layers, T, width]."""
    w = weights
    eps = float(config["norm"]["eps"])
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    kept: dict = {}
    after = []
    for index, layer in enumerate(config["layers"]):
        p, m = f"l{index}.", layer["mixer"]
        if layer["type"] == "attention":
            y = attention(w, p + "mix.", m, x, eps, kept, index, round_to)
        elif layer["type"] == "mamba2":
            y = mamba2(w, p + "mix.", m, x, eps, round_to)
        elif layer["type"] == "delta":
            y = gated_delta(w, p + "mix.", m, x, eps, round_to)
        else:
            raise ValueError(f"unknown mixer {layer['type']!r}")
        x = x + rms_norm(y, w[p + "norm1"], eps)
        if layer.get("mlp") is not None:
            x = x + rms_norm(dense_ff(w, p + "mlp.", x, round_to), w[p + "norm2"], eps)
        after.append(x)
    return _r(rms_norm(x, w["final.norm"], eps), round_to) @ w["head"].T, torch.stack(after)
