"""The Goguzen decoder, plainly: whole sequences, no cache, no carried state, float64, one function per
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
GLU_SLOPE = 1.702


def _r(x, round_to):
    return x if round_to is None else x.to(round_to).to(F64)


def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rms_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    return unit_rms(x, eps) * weight


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


# ---- positions ------------------------------------------------------------------------------------------

def rotary_frequencies(rot: Mapping) -> torch.Tensor:
    """Turning rates of the dims/2 pairs; with a scaling, pairs whose turn is long against the original length are
    slowed down by a factor, those whose turn is short are kept, the ones between are blended."""
    dims = int(rot["dims"])
    rates = [float(rot["base"]) ** (-2.0 * i / dims) for i in range(dims // 2)]
    scaling = rot.get("scaling")
    if scaling:
        factor, low, high, original = (float(scaling[k]) for k in ("factor", "low", "high", "original"))
        for i, f in enumerate(rates):
            turn = 2.0 * math.pi / f
            if turn > original / low:
                rates[i] = f / factor
            elif turn >= original / high:
                s = 0.0 if high == low else (original / turn - low) / (high - low)
                rates[i] = (1.0 - s) * f / factor + s * f
    return torch.tensor(rates, dtype=F64)


def rotate_halves(x: torch.Tensor, positions: torch.Tensor, rot: Mapping) -> torch.Tensor:
    """x [T, heads, d]: of the first rot.dims dims of every head, dim i turns with dim i + dims/2; the rest pass."""
    n = int(rot["dims"]) // 2
    angle = positions.to(F64)[:, None] * rotary_frequencies(rot)[None, :]
    cos, sin = torch.cos(angle)[:, None, :], torch.sin(angle)[:, None, :]
    u, v = x[..., :n], x[..., n : 2 * n]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, x[..., 2 * n :]], dim=-1)


def query_temperature(positions: torch.Tensor, every: float, coef: float) -> torch.Tensor:
    return 1.0 + coef * torch.log(torch.floor((positions.to(F64) + 1.0) / every) + 1.0)


# ---- attention --------------------------------------------------------------------------------------------

def visible(T: int, mask: Optional[Mapping]) -> torch.Tensor:
    """[T, T] bool, [i, j]: position i sees position j."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    seen = j <= i
    if mask:
        seen = seen & ((i - j < int(mask["size"])) | (j < int(mask.get("keep_first", 0))))
    return seen


def softmax_with_sink(score: torch.Tensor, sink: torch.Tensor) -> torch.Tensor:
    """exp(s_j) / (exp(sink) + sum exp(s_j)) over the last axis (hidden scores are -inf)."""
    top = torch.clamp(score.max(-1, keepdim=True).values, min=float(sink))
    e = torch.exp(score - top)
    return e / (torch.exp(sink - top) + e.sum(-1, keepdim=True))


def attend(q, k, v, scale: float, sinks, seen, round_to=None) -> torch.Tensor:
    """q [T, H, d], k [T, G, d], v [T, G, dv] -> the heads side by side [T, H * dv]."""
    q, k, v = (_r(t, round_to) for t in (q, k, v))
    T, H, G = q.shape[0], q.shape[1], k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for head in range(H):
        g = head // (H // G)
        score = ((q[:, head] @ k[:, g].T) * scale).masked_fill(~seen, -math.inf)
        out[:, head] = softmax_with_sink(score, sinks[head]) @ v[:, g]
    return out.reshape(T, -1)


def window_attention(w, p: str, m: Mapping, h: torch.Tensor, eps: float, round_to=None) -> torch.Tensor:
    """Queries and keys normed over their whole projection, rotated; a window and the first tokens; a sink."""
    T = h.shape[0]
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    hr = _r(h, round_to)
    q = rms_norm(hr @ w[p + "q"].T, w[p + "q.norm"], eps).view(T, H, d)
    k = rms_norm(hr @ w[p + "k"].T, w[p + "k.norm"], eps).view(T, G, d)
    v = (hr @ w[p + "v"].T).view(T, G, dv)
    if m.get("rot"):
        q, k = (rotate_halves(t, torch.arange(T), m["rot"]) for t in (q, k))
    o = attend(q, k, v, float(m["scale"]), w[p + "sink"], visible(T, m.get("mask")), round_to)
    return _r(o, round_to) @ w[p + "o"].T


def keys_as_values(w, p: str, m: Mapping, h: torch.Tensor, eps: float, round_to=None) -> torch.Tensor:
    """Every head normed by itself, the keys before their norm are the values; queries grow with their position;
    every earlier position is seen; a sink."""
    T = h.shape[0]
    H, G, d = int(m["heads"]), int(m["kv_heads"]), int(m["dim"])
    hr = _r(h, round_to)
    plain = (hr @ w[p + "k"].T).view(T, G, d)
    k = rms_norm(plain, w[p + "k.norm"], eps)
    q = rms_norm((hr @ w[p + "q"].T).view(T, H, d), w[p + "q.norm"], eps)
    t = m.get("q_temp")
    if t:
        q = q * query_temperature(torch.arange(T), float(t["every"]), float(t["coef"]))[:, None, None]
    o = attend(q, k, plain, float(m["scale"]), w[p + "sink"], visible(T, None), round_to)
    return _r(o, round_to) @ w[p + "o"].T


# ---- state space --------------------------------------------------------------------------------------------

def short_conv(x: torch.Tensor, taps: torch.Tensor, bias: torch.Tensor) -> torch.Tensor:
    """x [T, C], taps [C, n]: y_t = sum_j taps[:, j] x_(t - n + 1 + j) + bias, zeros before the start."""
    T, n = x.shape[0], taps.shape[1]
    padded = torch.cat([torch.zeros(n - 1, x.shape[1], dtype=F64), x])
    return sum(padded[j : j + T] * taps[:, j] for j in range(n)) + bias


def decayed_sums(q, k, v, log_decay, write) -> torch.Tensor:
    """Per head S_t = exp(log_decay_t) S_(t-1) + write_t k_t v_t^T, o_t = S_t^T q_t.  q, k [T, H, N], v [T, H, P],
    log_decay and write [T, H]."""
    T, H, P = v.shape
    out = torch.zeros(T, H, P, dtype=F64)
    S = torch.zeros(H, k.shape[-1], P, dtype=F64)
    for t in range(T):
        S = torch.exp(log_decay[t])[:, None, None] * S + (write[t][:, None] * k[t])[:, :, None] * v[t][:, None, :]
        out[t] = torch.einsum("hnp,hn->hp", S, q[t])
    return out


def state_space(w, p: str, m: Mapping, h: torch.Tensor, eps: float, round_to=None) -> torch.Tensor:
    T = h.shape[0]
    H, P, N, G, parts = (int(m[n]) for n in ("heads", "vdim", "state", "groups", "norm_groups"))
    inner = H * P
    sums = _r(h, round_to) @ w[p + "in"].T
    z, mixed, dt = sums.split([inner, inner + 2 * G * N, H], dim=-1)
    mixed = silu(short_conv(mixed, w[p + "conv"], w[p + "conv.b"]))
    x = mixed[:, :inner].view(T, H, P)
    b, c = (mixed[:, at : at + G * N].view(T, G, N).repeat_interleave(H // G, dim=1) for at in (inner, inner + G * N))
    dt = torch.nn.functional.softplus(dt + w[p + "dt_bias"])
    y = decayed_sums(c, b, x, -torch.exp(w[p + "A_log"]) * dt, dt) + w[p + "D"][:, None] * x
    y = y.reshape(T, inner) * silu(z)
    y = unit_rms(y.view(T, parts, inner // parts), eps).reshape(T, inner) * w[p + "norm"]
    return _r(y, round_to) @ w[p + "o"].T


def two_mixers(w, p: str, m: Mapping, h: torch.Tensor, eps: float, round_to=None) -> torch.Tensor:
    left = keys_as_values(w, p + "left.", m["left"], h, eps, round_to)
    right = state_space(w, p + "right.", m["right"], h, eps, round_to)
    return 0.5 * (rms_norm(left, w[p + "left.out"], eps) + rms_norm(right, w[p + "right.out"], eps))


# ---- feed-forward ---------------------------------------------------------------------------------------

def clamped_expert(w, p: str, limit: float, h: torch.Tensor, round_to=None) -> torch.Tensor:
    g = torch.clamp(h @ w[p + "gate"].T, max=limit)
    u = torch.clamp(h @ w[p + "up"].T, min=-limit, max=limit)
    return _r(g * torch.sigmoid(GLU_SLOPE * g) * (u + 1.0), round_to) @ w[p + "down"].T


def route(logits: torch.Tensor, top: int) -> torch.Tensor:
    """[T, experts] weights: the softmax over each row's `top` largest logits, zeros elsewhere."""
    value, index = torch.topk(logits, top, dim=-1)
    return torch.zeros_like(logits).scatter(-1, index, torch.softmax(value, -1))


def mixture(w, p: str, f: Mapping, h: torch.Tensor, round_to=None, margins: Optional[list] = None) -> torch.Tensor:
    hr = _r(h, round_to)
    logits = hr @ w[p + "router"].T + w[p + "router.b"]
    top = int(f["router"]["top"])
    if margins is not None and top < logits.shape[1]:  # how far the last chosen expert is from the first that is not
        ordered = logits.sort(-1, descending=True).values
        margins.append(ordered[:, top - 1] - ordered[:, top])
    weight = route(logits, top)
    out = torch.zeros_like(h)
    for e in range(int(f["router"]["experts"])):
        rows = weight[:, e].nonzero()[:, 0]
        if rows.numel():
            out[rows] += weight[rows, e, None] * clamped_expert(w, f"{p}e{e}.", float(f["expert"]["limit"]), hr[rows], round_to)
    if f.get("shared"):
        out = out + clamped_expert(w, p + "shared.", float(f["shared"]["limit"]), hr, round_to)
    return out


# ---- the model ------------------------------------------------------------------------------------------

MIXERS = {"attention": window_attention, "parallel": two_mixers}


def forward(
    config: Mapping, weights: Mapping[str, torch.Tensor], tokens, round_to: Optional[torch.dtype] = None,
    margins: Optional[list] = None,
):
    """logits [T, vocab] and the stream after every layer [layers, T, width].  `margins`: a list that receives, per
    mixture, how close each token's choice of experts was ([T])."""
    w = weights
    eps = float(config["norm"]["eps"])
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)] * float(config["embedding"]["scale"])
    after = []
    for index, layer in enumerate(config["layers"]):
        owner = index
        while config["layers"][owner].get("weights_of") is not None:
            owner = int(config["layers"][owner]["weights_of"])
        p = f"l{owner}."
        x = x + MIXERS[layer["type"]](w, p + "mix.", layer["mixer"], rms_norm(x, w[p + "norm1"], eps), eps, round_to)
        if layer.get("mlp") is not None:
            x = x + mixture(w, p + "mlp.", layer["mlp"], rms_norm(x, w[p + "norm2"], eps), round_to, margins)
        after.append(x)
    logits = (_r(rms_norm(x, w["final.norm"], eps), round_to) @ w["head"].T) * float(config.get("logit_scale", 1.0))
    cap = config.get("logit_softcap")
    if cap:
        logits = float(cap) * torch.tanh(logits / float(cap))
    return logits, torch.stack(after)
