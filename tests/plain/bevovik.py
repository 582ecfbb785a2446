"""A plain, slow form of the Bevovik decoder, one function per mechanism, written from the
design's equations with torch on the CPU.  It shares nothing with the package: it takes the raw
config dictionary and a dictionary of tensors by their names in the weight file, runs one whole
sequence at a time, keeps no cache, and returns logits for every position (in the precision of
the tensors it is given).

Notation: matrices are stored [out, in]; x is the stream [tokens, width]; positions count from 0;
t is a token's place, s an earlier one's.
"""

from __future__ import annotations

import math

import torch

GATE_SLOPE = 1.702  # an expert's gate is g * sigmoid(1.702 g)
DECAY_POWER = 8.0  # of the gated linear recurrent unit


def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps), the eps inside the root."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z**3)))


def log_sigmoid(z: torch.Tensor) -> torch.Tensor:
    """ln(sigmoid(z)) without overflow on either side."""
    return torch.where(z < 0, z - torch.log1p(torch.exp(-z.abs())), -torch.log1p(torch.exp(-z.abs())))


def softplus(z: torch.Tensor) -> torch.Tensor:
    return -log_sigmoid(-z)


# ---------------------------------------------------------------- gated linear attention


def key_decays(h, w, prefix: str, m: dict):
    """sigmoid(W_a2 W_a1 h + b) ** (1 / tau), one number per head and key channel: [n, heads, dim]."""
    z = (h @ w[prefix + ".a1"].T) @ w[prefix + ".a2"].T + w[prefix + ".a2.b"]
    return torch.exp(log_sigmoid(z) / float(m["tau"])).view(h.shape[0], m["heads"], m["dim"])


def decayed_outer_sums(q, k, v, alpha):
    """Head by head: S <- diag(alpha_t) S + k_t v_t^T from zero, o_t = S^T q_t; q, k, alpha [n, heads, dim],
    v [n, heads, vdim]."""
    n, heads, dim = q.shape
    S = torch.zeros(heads, dim, v.shape[2], dtype=v.dtype)
    out = []
    for t in range(n):
        S = alpha[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out.append((S * q[t][:, :, None]).sum(dim=1))
    return torch.stack(out)


def gated_linear_attention(h, w, prefix: str, m: dict, eps: float):
    n, H, D = h.shape[0], m["heads"], m["dim"]
    V = m["vdim"]
    q = (h @ w[prefix + ".q"].T).view(n, H, D) * D**-0.5
    k = (h @ w[prefix + ".k"].T).view(n, H, D)
    v = (h @ w[prefix + ".v"].T).view(n, H, V)
    alpha = key_decays(h, w, prefix, m)
    o = unit_rms(decayed_outer_sums(q, k, v, alpha), eps) * w[prefix + ".norm"]
    g = h @ w[prefix + ".g"].T
    return (o.reshape(n, H * V) * g * torch.sigmoid(g)) @ w[prefix + ".o"].T


# ---------------------------------------------------------------- attention through latents


def turn_rates(rot: dict):
    """(rate per pair, factor on cosine and sine).  With `scaling`, pairs that make few turns within
    `original` positions turn `factor` times slower, pairs that make many stay, those between are
    blended linearly in the pair's number."""
    base, dims = float(rot["base"]), int(rot["dims"])
    rates = torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=torch.float64)
    sc = rot.get("scaling")
    if not sc:
        return rates, 1.0
    place = lambda turns: dims * math.log(float(sc["original"]) / (2.0 * math.pi * turns)) / (2.0 * math.log(base))  # noqa: E731
    first = max(math.floor(place(float(sc["fast"]))), 0)
    last = min(math.ceil(place(float(sc["slow"]))), dims - 1)
    share = ((torch.arange(dims // 2, dtype=torch.float64) - first) / max(last - first, 0.001)).clamp(0.0, 1.0)
    factor = float(sc["factor"])
    return rates / factor * share + rates * (1.0 - share), 0.1 * math.log(factor) + 1.0


def rotate_pairs(x: torch.Tensor, positions: torch.Tensor, rot: dict) -> torch.Tensor:
    """Turns the pairs (2i, 2i + 1), i < dims / 2, of the last axis; the rest passes unchanged.
    x is [tokens, ..., size]."""
    dims = int(rot["dims"])
    rates, factor = turn_rates(rot)
    angle = positions.to(torch.float64)[:, None] * rates
    shape = (x.shape[0],) + (1,) * (x.dim() - 2) + (dims // 2,)
    cos = (torch.cos(angle) * factor).to(x.dtype).view(shape)
    sin = (torch.sin(angle) * factor).to(x.dtype).view(shape)
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out = x.clone()
    out[..., 0:dims:2] = u * cos - v * sin
    out[..., 1:dims:2] = v * cos + u * sin
    return out


def latent_attention(h, positions, w, prefix: str, m: dict, eps: float):
    """Queries through a normed latent; keys and values through another, of which one normed part is
    every head's source of keys and values and a second, unnormed part a rotated key that all heads
    share; causal."""
    n = h.shape[0]
    H, D, R, V, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    c_q = unit_rms(h @ w[prefix + ".dq"].T, eps) * w[prefix + ".dq.norm"]
    q = (c_q @ w[prefix + ".uq"].T).view(n, H, D + R)
    down = h @ w[prefix + ".dkv"].T
    c = unit_rms(down[:, :rank], eps) * w[prefix + ".dkv.norm"]
    q_plain, q_rot, k_rot = q[..., :D], q[..., D:], down[:, rank:]
    if R:
        q_rot, k_rot = rotate_pairs(q_rot, positions, m["rot"]), rotate_pairs(k_rot, positions, m["rot"])
    k_plain = (c @ w[prefix + ".uk"].T).view(n, H, D)
    v = (c @ w[prefix + ".uv"].T).view(n, H, V)
    later = torch.arange(n)[None, :] > torch.arange(n)[:, None]
    out = torch.zeros(n, H, V, dtype=h.dtype)
    for head in range(H):
        s = (q_plain[:, head] @ k_plain[:, head].T + q_rot[:, head] @ k_rot.T) * float(m["scale"])
        out[:, head] = torch.softmax(s.masked_fill(later, float("-inf")), dim=-1) @ v[:, head]
    return out.reshape(n, H * V) @ w[prefix + ".o"].T


# ---------------------------------------------------------------- gated linear recurrent unit


def causal_convolution(x: torch.Tensor, taps: torch.Tensor, bias: torch.Tensor) -> torch.Tensor:
    """y[t, c] = bias[c] + sum_k taps[c, K - 1 - k] x[t - k, c], zeros before the start."""
    n, K = x.shape[0], taps.shape[1]
    y = bias.expand_as(x).clone()
    for k in range(min(K, n)):
        y[k:] += taps[:, K - 1 - k] * x[: n - k]
    return y


def block_gate(u, w, name: str, blocks: int):
    """sigmoid of a block-diagonal product with a bias: part b of u meets its own square matrix."""
    n, width = u.shape
    z = torch.einsum("nbi,boi->nbo", u.view(n, blocks, width // blocks), w[name]) + w[name + ".b"]
    return torch.sigmoid(z).reshape(n, width)


def recurrent_sums(log_a, x):
    """S_t = a_t S_(t-1) + sqrt(1 - a_t^2) x_t per channel, from zero."""
    a = torch.exp(log_a)
    share = torch.sqrt(-torch.expm1(2.0 * log_a))
    S, out = torch.zeros_like(x[0]), []
    for t in range(x.shape[0]):
        S = a[t] * S + share[t] * x[t]
        out.append(S)
    return torch.stack(out)


def gated_recurrence(h, w, prefix: str, m: dict):
    blocks = int(m["blocks"])
    y = gelu_tanh(h @ w[prefix + ".y"].T + w[prefix + ".y.b"])
    u = causal_convolution(h @ w[prefix + ".x"].T + w[prefix + ".x.b"], w[prefix + ".conv"], w[prefix + ".conv.b"])
    r = block_gate(u, w, prefix + ".ra", blocks)
    i = block_gate(u, w, prefix + ".ri", blocks)
    S = recurrent_sums(-DECAY_POWER * r * softplus(w[prefix + ".lam"]), i * u)
    return (S * y) @ w[prefix + ".o"].T


# ---------------------------------------------------------------- feed-forward


def expert(h, w, prefix: str, limit: float):
    """g = min(W_gate h, limit), u = clamp(W_up h, -limit, limit); W_down (g sigmoid(1.702 g) (u + 1))."""
    g = (h @ w[prefix + ".gate"].T).clamp(max=limit)
    u = (h @ w[prefix + ".up"].T).clamp(min=-limit, max=limit)
    return (g * torch.sigmoid(GATE_SLOPE * g) * (u + 1.0)) @ w[prefix + ".down"].T


def choose(scores, correction, top: int, count: int, keep: int):
    """The `top` entries of one token's scores + correction, only from the `keep` groups (of `count`
    equal groups of neighbours) whose largest entry is largest.  A list of indices."""
    choice = (scores + correction).tolist()
    size = len(choice) // count
    best = [max(choice[g * size : (g + 1) * size]) for g in range(count)]
    groups = sorted(range(count), key=lambda g: (-best[g], g))[:keep]
    allowed = [e for e in range(len(choice)) if e // size in groups]
    return sorted(allowed, key=lambda e: (-choice[e], e))[:top]


def route(h, w, prefix: str, router: dict):
    """(chosen [n, top], weights [n, top]) over experts and, after them, identity experts."""
    z = h @ w[prefix + ".router"].T
    scores = torch.softmax(z, dim=-1)
    groups = router.get("groups") or {"count": 1, "keep": 1}
    correction = w.get(prefix + ".correction", torch.zeros(z.shape[1], dtype=z.dtype))
    chosen = torch.tensor([choose(s, correction, int(router["top"]), int(groups["count"]), int(groups["keep"])) for s in scores],
                          dtype=torch.long)
    picked = scores.gather(1, chosen)
    return chosen, picked / (picked.sum(-1, keepdim=True) + 1e-20) * float(router.get("scale") or 1.0)


def mixture(h, w, prefix: str, m: dict):
    """Every token's weighted sum of its chosen experts (an identity expert gives the token's own
    input), plus the shared expert."""
    experts = int(m["router"]["experts"])
    chosen, weights = route(h, w, prefix, m["router"])
    out = torch.zeros_like(h)
    for e in range(int(chosen.max()) + 1):
        for slot in range(chosen.shape[1]):
            rows = (chosen[:, slot] == e).nonzero().flatten()
            if rows.numel():
                y = h[rows] if e >= experts else expert(h[rows], w, f"{prefix}.e{e}", float(m["expert"]["limit"]))
                out[rows] += weights[rows, slot, None] * y
    if m.get("shared"):
        out = out + expert(h, w, prefix + ".shared", float(m["shared"]["limit"]))
    return out


# ---------------------------------------------------------------- the whole


def forward(cfg: dict, w: dict, tokens, return_layers: bool = False):
    """Logits [tokens, vocab] of one sequence; with return_layers also the stream after every layer.
    A layer adds each sublayer's output, normed and multiplied element by element, to the stream that
    the sublayer has read as it stands."""
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    positions = torch.arange(tokens.shape[0])
    eps = float(cfg["norm"]["eps"])
    x = w["embed"][tokens]
    streams = []
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}", layer["mixer"]
        if layer["type"] == "latent_attention":
            y = latent_attention(x, positions, w, p + ".mix", m, eps)
        elif layer["type"] == "gla":
            y = gated_linear_attention(x, w, p + ".mix", m, eps)
        elif layer["type"] == "rglru":
            y = gated_recurrence(x, w, p + ".mix", m)
        else:
            raise ValueError(f"unknown mixer type {layer['type']!r}")
        x = x + unit_rms(y, eps) * w[p + ".norm1"] * w[p + ".ls1"]
        if layer.get("mlp"):
            x = x + unit_rms(mixture(x, w, p + ".mlp", layer["mlp"]), eps) * w[p + ".norm2"] * w[p + ".ls2"]
        streams.append(x)
    logits = (unit_rms(x, eps) * w["final.norm"]) @ w["head"].T
    return (logits, torch.stack(streams)) if return_layers else logits


class PlainBevovik:
    """A model folder read once; `logits(ids)`, the stream after every layer, and greedy generation
    over it, in float64 unless told otherwise."""

    def __init__(self, model_dir, dtype=torch.float64):
        import json
        from pathlib import Path

        from safetensors.torch import load_file

        self.cfg = json.loads((Path(model_dir) / "config.json").read_text())
        raw = load_file(str(Path(model_dir) / "model.safetensors"))
        self.weights = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in raw.items()}

    def logits(self, token_ids, rows=None) -> torch.Tensor:
        out = forward(self.cfg, self.weights, list(token_ids))
        return out if rows is None else out[torch.tensor(list(rows), dtype=torch.long)]

    def layers(self, token_ids) -> torch.Tensor:
        return forward(self.cfg, self.weights, list(token_ids), return_layers=True)[1]

    def greedy(self, prompt, max_new_tokens: int) -> list[int]:
        seq, out = list(prompt), []
        for _ in range(max_new_tokens):
            tok = int(torch.argmax(self.logits(seq)[-1]))
            out.append(tok)
            seq.append(tok)
        return out
