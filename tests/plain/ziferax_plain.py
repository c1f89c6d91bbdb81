"""A plain, slow implementation of the Ziferax decoder, one function per mechanism, written from the design's equations
and sharing no code with the engine.  Everything works on one whole sequence at a time: there is no cache and no batch
here, so whatever the engine does with pages, slots and portions has to come out as if it had not happened.  Attention
is a full score matrix with a mask; the routed feed-forward is a loop over the tokens and the experts each of them chose.

Notation: n tokens, d model width.  Linear weights are [out, in] and applied as W x.  Arithmetic is float32 unless the
caller asks for float64.
"""

from __future__ import annotations

import torch

SIGMOID_SLOPE = 1.702


# ---- small pieces ----------------------------------------------------------------------------------------------------

def rms_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) * w over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * weight


def affine(h: torch.Tensor, matrix: torch.Tensor, bias: torch.Tensor) -> torch.Tensor:
    return h @ matrix.T + bias


def turn_pairs(x: torch.Tensor, positions: torch.Tensor, dims: int, base: float) -> torch.Tensor:
    """x [n, heads, width]: of every head's first `dims` dimensions the pair (2i, 2i + 1) is turned by the angle
    position * base^(-2i / dims); the other dimensions pass."""
    out = x.clone()
    for i in range(dims // 2):
        angle = positions.to(x.dtype) * torch.tensor(base ** (-2.0 * i / dims), dtype=torch.float64).to(x.dtype)
        cos, sin = torch.cos(angle)[:, None], torch.sin(angle)[:, None]
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * cos - v * sin
        out[..., 2 * i + 1] = v * cos + u * sin
    return out


def window_mask(n: int, size: int | None) -> torch.Tensor:
    """[n, n] bool: query i sees key j if 0 <= i - j < size (size None: every j <= i)."""
    distance = torch.arange(n)[:, None] - torch.arange(n)[None, :]
    seen = distance >= 0
    return seen if size is None else seen & (distance < size)


def softmax_with_sink(scores: torch.Tensor, seen: torch.Tensor, sink: torch.Tensor) -> torch.Tensor:
    """exp(s_j) / (exp(sink) + sum over the keys that are seen of exp(s_j)), row by row."""
    scores = scores.masked_fill(~seen, float("-inf"))
    highest = torch.maximum(scores.amax(-1, keepdim=True), sink)
    terms = torch.exp(scores - highest)
    return terms / (terms.sum(-1, keepdim=True) + torch.exp(sink - highest))


# ---- attention -------------------------------------------------------------------------------------------------------

def attention(h: torch.Tensor, w: dict, m: dict) -> torch.Tensor:
    """Grouped-query attention whose values are its keys as they were projected, before the rotation."""
    n = h.shape[0]
    heads, groups, dim = m["heads"], m["kv_heads"], m["dim"]
    q = affine(h, w["q"], w["q.b"]).view(n, heads, dim)
    k = affine(h, w["k"], w["k.b"]).view(n, groups, dim)
    values = k.clone()
    if m.get("rot") is not None:
        positions = torch.arange(n)
        q = turn_pairs(q, positions, m["rot"]["dims"], float(m["rot"]["base"]))
        k = turn_pairs(k, positions, m["rot"]["dims"], float(m["rot"]["base"]))
    seen = window_mask(n, m["mask"]["size"] if m.get("mask") is not None else None)
    out = torch.empty(n, heads, dim, dtype=h.dtype)
    for head in range(heads):
        g = head // (heads // groups)
        scores = (q[:, head] @ k[:, g].T) * m["scale"]
        out[:, head] = softmax_with_sink(scores, seen, w["sink"][head]) @ values[:, g]
    return affine(out.reshape(n, heads * dim), w["o"], w["o.b"])


# ---- feed-forward ----------------------------------------------------------------------------------------------------

def clamped_expert(h: torch.Tensor, gate: torch.Tensor, up: torch.Tensor, down: torch.Tensor, limit: float) -> torch.Tensor:
    """g = min(W_gate h, L); u = W_up h held to [-L, L]; W_down (g sigmoid(1.702 g) (u + 1))."""
    g = torch.clamp(h @ gate.T, max=limit)
    u = torch.clamp(h @ up.T, min=-limit, max=limit)
    return (g * torch.sigmoid(SIGMOID_SLOPE * g) * (u + 1.0)) @ down.T


def corrected_choice(h: torch.Tensor, router: torch.Tensor, correction: torch.Tensor, top: int):
    """(chosen outputs of the router [n, top], their weights [n, top]): scores are a softmax over all outputs; the choice
    looks at score + correction, the weights are the chosen outputs' scores divided by their sum."""
    scores = torch.softmax(h @ router.T, dim=-1)
    chosen = torch.sort(scores + correction, dim=-1, descending=True, stable=True).indices[:, :top]
    picked = torch.gather(scores, 1, chosen)
    return chosen, picked / (picked.sum(-1, keepdim=True) + 1e-20)


def routed_feed_forward(h: torch.Tensor, w: dict, mlp: dict) -> torch.Tensor:
    """The chosen experts' outputs times their weights - an identity expert's output is the input itself - plus the
    expert that every token uses."""
    experts = mlp["router"]["experts"]
    chosen, weights = corrected_choice(h, w["router"], w["correction"], mlp["router"]["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, weight in zip(chosen[t].tolist(), weights[t]):
            if e >= experts:
                out[t] += weight * h[t]
            else:
                out[t] += weight * clamped_expert(h[t], w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"], mlp["expert"]["limit"])
    if mlp.get("shared") is not None:
        out = out + clamped_expert(h, w["shared.gate"], w["shared.up"], w["shared.down"], mlp["shared"]["limit"])
    return out


# ---- the model -------------------------------------------------------------------------------------------------------

def sub_weights(weights: dict, prefix: str) -> dict:
    return {name[len(prefix):]: tensor for name, tensor in weights.items() if name.startswith(prefix)}


def owner_of(layers: list, index: int) -> int:
    """The layer whose tensors layer `index` uses."""
    while layers[index].get("weights_of") is not None:
        index = layers[index]["weights_of"]
    return index


def layer(x: torch.Tensor, weights: dict, owner: int, spec: dict, mult: float, eps: float) -> torch.Tensor:
    """One norm, both sublayers read it: x + m (mixer(h) + ff(h))."""
    h = rms_norm(x, weights[f"l{owner}.norm1"], eps)
    branch = attention(h, sub_weights(weights, f"l{owner}.mix."), spec["mixer"])
    if spec.get("mlp") is not None:
        branch = branch + routed_feed_forward(h, sub_weights(weights, f"l{owner}.mlp."), spec["mlp"])
    return x + mult * branch


def forward(config: dict, weights: dict, tokens, dtype=torch.float32, streams: list | None = None) -> torch.Tensor:
    """Logits [n, vocab] of one whole sequence.  `streams`, if given, collects the residual sum after every layer."""
    weights = {name: t.to(dtype) if t.is_floating_point() else t for name, t in weights.items()}
    eps, mult = float(config["norm"]["eps"]), float(config["residual_mult"])
    x = weights["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    for index, spec in enumerate(config["layers"]):
        x = layer(x, weights, owner_of(config["layers"], index), spec, mult, eps)
        if streams is not None:
            streams.append(x.clone())
    return rms_norm(x, weights["final.norm"], eps) @ weights["embed"].T
