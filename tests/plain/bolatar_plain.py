"""A plain, slow implementation of the Bolatar decoder, one function per mechanism, written from the design's equations
and sharing no code with the engine.  Everything works on one whole sequence at a time: there is no cache, no state and
no batch here, so whatever the engine does with pages, slots and portions has to come out as if it had not happened.
Recurrences are loops over the tokens; attention is a full score matrix with a mask.

Notation: n tokens, d model width.  Linear weights are [out, in] and applied as W x.  Arithmetic is float32 unless the
caller asks for float64.
"""

from __future__ import annotations

import math

import torch

UNIT_EPS = 1e-6          # inside the root of the delta rule's unit vectors
READ_EPS = 1e-6          # beside the denominator of the matrix memory's read-out
GATE_SLOPE = 1.702       # of the feed-forward's sigmoid


# ---- small pieces ----------------------------------------------------------------------------------------------------

def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rms_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    """The same times a weight: one number for all coordinates, or one per coordinate."""
    return unit_rms(x, eps) * weight


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def softplus(z: torch.Tensor) -> torch.Tensor:
    return torch.where(z > 20, z, torch.log1p(torch.exp(z.clamp(max=20))))


def log_sigmoid(z: torch.Tensor) -> torch.Tensor:
    return -softplus(-z)


def soft_cap(z: torch.Tensor, cap: float) -> torch.Tensor:
    return cap * torch.tanh(z / cap)


def embed(tokens: torch.Tensor, table: torch.Tensor, scale: float, places: torch.Tensor) -> torch.Tensor:
    """Scaled token rows plus the (unscaled) vector of every token's position."""
    return table[tokens] * scale + places[:tokens.shape[0]]


# ---- the gated delta rule ----------------------------------------------------------------------------------------------

def causal_convolution(x: torch.Tensor, taps: torch.Tensor) -> torch.Tensor:
    """x [n, channels], taps [channels, t]: y_i = sum_k taps[:, k] x_(i - t + 1 + k), zeros before the start."""
    n, t = x.shape[0], taps.shape[1]
    padded = torch.cat((torch.zeros(t - 1, x.shape[1], dtype=x.dtype), x))
    return sum(padded[k:k + n] * taps[:, k] for k in range(t))


def delta_rule(h: torch.Tensor, w: dict, m: dict, eps: float) -> torch.Tensor:
    n = h.shape[0]
    heads, groups, dim, vdim = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = silu(causal_convolution(h @ w["q"].T, w["q.conv"])).view(n, groups, dim)
    k = silu(causal_convolution(h @ w["k"].T, w["k.conv"])).view(n, groups, dim)
    v = silu(causal_convolution(h @ w["v"].T, w["v.conv"])).view(n, heads, vdim)
    q = q / torch.sqrt((q * q).sum(-1, keepdim=True) + UNIT_EPS) * dim ** -0.5
    k = k / torch.sqrt((k * k).sum(-1, keepdim=True) + UNIT_EPS)
    beta = torch.sigmoid(h @ w["b"].T)
    keep = torch.exp(-torch.exp(w["A_log"]) * softplus(h @ w["a"].T + w["dt_bias"]))
    out = torch.empty(n, heads, vdim, dtype=h.dtype)
    for head in range(heads):
        g = head // (heads // groups)
        state = torch.zeros(dim, vdim, dtype=h.dtype)
        for t in range(n):
            state = keep[t, head] * state
            u = beta[t, head] * (v[t, head] - state.T @ k[t, g])
            state = state + torch.outer(k[t, g], u)
            out[t, head] = state.T @ q[t, g]
    out = rms_norm(out, w["norm"], eps) * silu(h @ w["g"].T).view(n, heads, vdim)
    return out.reshape(n, heads * vdim) @ w["o"].T


# ---- the parallel mixer: attention beside time mixing --------------------------------------------------------------------

def query_temperature(n: int, coef: float, every: int, dtype=torch.float32) -> torch.Tensor:
    """1 + coef * ln(floor((p + 1) / every) + 1) at the positions p = 0 .. n - 1."""
    return torch.tensor([1.0 + coef * math.log(math.floor((p + 1) / every) + 1) for p in range(n)], dtype=dtype)


def distance_bias(n: int, r1: torch.Tensor, r2: torch.Tensor) -> torch.Tensor:
    """[n, n]: r1 ln(1 + r2 (i - j)) for j <= i, zero elsewhere (one head's numbers)."""
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    return r1 * torch.log(1.0 + r2 * (i - j).clamp(min=0).to(r1.dtype))


def biased_attention(h: torch.Tensor, w: dict, m: dict, eps: float) -> torch.Tensor:
    n = h.shape[0]
    heads, groups, dim, vdim = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ w["q"].T).view(n, heads, dim)
    k = (h @ w["k"].T).view(n, groups, dim)
    v = unit_rms((h @ w["v"].T).view(n, groups, vdim), eps)
    temp = m.get("q_temp")
    if temp is not None:
        q = q * query_temperature(n, float(temp["coef"]), int(temp["every"]), h.dtype)[:, None, None]
    hidden = torch.arange(n)[None, :] > torch.arange(n)[:, None]
    out = torch.empty(n, heads, vdim, dtype=h.dtype)
    for head in range(heads):
        g = head // (heads // groups)
        scores = (q[:, head] @ k[:, g].T) * float(m["scale"]) - distance_bias(n, w["r1"][head], w["r2"][head])
        out[:, head] = torch.softmax(scores.masked_fill(hidden, float("-inf")), dim=-1) @ v[:, g]
    return out.reshape(n, heads * vdim) @ w["o"].T


def shifted(h: torch.Tensor) -> torch.Tensor:
    """The row before, zeros for the first."""
    return torch.cat((torch.zeros_like(h[:1]), h[:-1]))


def mixed_states(r, k, v, keep, bonus) -> torch.Tensor:
    """r, k, v, keep [n, heads, dim], bonus [heads, dim] -> the read-outs before their norm."""
    n, heads, dim = r.shape
    out = torch.empty(n, heads, dim, dtype=r.dtype)
    for head in range(heads):
        state = torch.zeros(dim, dim, dtype=r.dtype)
        for t in range(n):
            write = torch.outer(k[t, head], v[t, head])
            out[t, head] = (state + bonus[head][:, None] * write).T @ r[t, head]
            state = keep[t, head][:, None] * state + write
    return out


def time_mixing(h: torch.Tensor, w: dict, m: dict, eps: float) -> torch.Tensor:
    n = h.shape[0]
    heads, dim = m["heads"], m["dim"]
    mixed = {s: h + (shifted(h) - h) * w[f"mu.{s}"] for s in "rkvgw"}
    r, k, v = ((mixed[s] @ w[s].T).view(n, heads, dim) for s in "rkv")
    gate = silu(mixed["g"] @ w["g"].T)
    keep = torch.exp(-torch.exp(torch.tanh(mixed["w"] @ w["w1"].T) @ w["w2"].T + w["w0"])).view(n, heads, dim)
    out = mixed_states(r, k, v, keep, w["u"])
    return (unit_rms(out, eps).reshape(n, heads * dim) * w["norm"] * gate) @ w["o"].T


def parallel(h: torch.Tensor, w: dict, m: dict, eps: float) -> torch.Tensor:
    left = biased_attention(h, sub_weights(w, "left."), m["left"], eps)
    right = time_mixing(h, sub_weights(w, "right."), m["right"], eps)
    return 0.5 * (rms_norm(left, w["left.out"], eps) + rms_norm(right, w["right.out"], eps))


# ---- the matrix memory ---------------------------------------------------------------------------------------------------

def matrix_memory(h: torch.Tensor, w: dict, m: dict, eps: float) -> torch.Tensor:
    n = h.shape[0]
    heads, dim, vdim, cap = m["heads"], m["dim"], m["vdim"], float(m["gate_cap"])
    q = (h @ w["q"].T).view(n, heads, dim) * dim ** -0.5
    k = (h @ w["k"].T).view(n, heads, dim)
    v = (h @ w["v"].T).view(n, heads, vdim)
    into = soft_cap(h @ w["i"].T + w["i.b"], cap)
    keep = log_sigmoid(soft_cap(h @ w["f"].T + w["f.b"], cap))
    out = torch.empty(n, heads, vdim, dtype=h.dtype)
    for head in range(heads):
        state, total = torch.zeros(dim, vdim, dtype=h.dtype), torch.zeros(dim, dtype=h.dtype)
        top = torch.zeros((), dtype=h.dtype)
        for t in range(n):
            new = torch.maximum(keep[t, head] + top, into[t, head])
            a, b = torch.exp(keep[t, head] + top - new), torch.exp(into[t, head] - new)
            top = new
            state = a * state + b * torch.outer(k[t, head], v[t, head])
            total = a * total + b * k[t, head]
            size = torch.maximum((total @ q[t, head]).abs(), torch.exp(-top)) + READ_EPS
            out[t, head] = state.T @ q[t, head] / size
    out = unit_rms(out, eps).reshape(n, heads * vdim) * w["norm"]
    return (out * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


MIXERS = {"delta": delta_rule, "parallel": parallel, "mlstm": matrix_memory}


# ---- feed-forward and model ------------------------------------------------------------------------------------------------

def limited_activation(gate: torch.Tensor, up: torch.Tensor, limit: float) -> torch.Tensor:
    g, u = gate.clamp(max=limit), up.clamp(-limit, limit)
    return g * torch.sigmoid(GATE_SLOPE * g) * (u + 1.0)


def feed_forward(h: torch.Tensor, w: dict, limit: float) -> torch.Tensor:
    return limited_activation(h @ w["gate"].T, h @ w["up"].T, limit) @ w["down"].T


def sub_weights(weights: dict, prefix: str) -> dict:
    return {name[len(prefix):]: tensor for name, tensor in weights.items() if name.startswith(prefix)}


def layer(x: torch.Tensor, weights: dict, index: int, spec: dict, eps: float) -> torch.Tensor:
    p = f"l{index}."
    x = x + MIXERS[spec["type"]](rms_norm(x, weights[p + "norm1"], eps), sub_weights(weights, p + "mix."), spec["mixer"], eps)
    mlp = spec.get("mlp")
    if mlp is None:
        return x
    return x + feed_forward(rms_norm(x, weights[p + "norm2"], eps), sub_weights(weights, p + "mlp."), float(mlp["limit"]))


def forward(config: dict, weights: dict, tokens, dtype=torch.float32, streams: list | None = None) -> torch.Tensor:
    """Logits [n, vocab] of one whole sequence.  `streams`, if given, collects the residual sum after every layer."""
    weights = {name: t.to(dtype) if t.is_floating_point() else t for name, t in weights.items()}
    eps = float(config["norm"]["eps"])
    x = embed(torch.as_tensor(tokens, dtype=torch.long), weights["embed"], float(config["embedding"]["scale"]), weights["pos"])
    for index, spec in enumerate(config["layers"]):
        x = layer(x, weights, index, spec, eps)
        if streams is not None:
            streams.append(x.clone())
    logits = rms_norm(x, weights["final.norm"], eps) @ weights["head"].T
    cap = config.get("logit_softcap")
    return soft_cap(logits, float(cap)) if cap is not None else logits
