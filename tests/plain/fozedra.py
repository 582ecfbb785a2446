"""A plain, slow form of the Fozedra decoder, one function per mechanism, written from the
design's equations with torch on the CPU.  It shares nothing with the package: it takes the
raw config dictionary and a dictionary of tensors by their names in the weight file, runs one
whole sequence at a time, keeps no cache and no state between calls, and returns logits for
every position (in the precision of the tensors it is given).

Notation: W[.] are matrices stored [out, in]; x is the stream [tokens, width], h a sublayer's
normed input; positions count from 0; i is a query's position, j a key's.
"""

from __future__ import annotations

import math

import torch


def dynamic_tanh(x, w, name: str):
    """tanh(alpha x) * weight + bias with one learned alpha: stands where a norm would."""
    return torch.tanh(w[name + ".alpha"] * x) * w[name] + w[name + ".b"]


def unit_rms(x, eps: float):
    """x / sqrt(mean(x^2) + eps), the eps inside the root."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def visible(n: int, mask):
    """vis[i, j]: j <= i, and with a mask also i - j < size or j < keep_first."""
    i = torch.arange(n)[:, None]
    j = torch.arange(n)[None, :]
    vis = j <= i
    if mask:
        vis = vis & ((i - j < int(mask["size"])) | (j < int(mask.get("keep_first", 0))))
    return vis


def short_convolution(u, taps):
    """y_t = sum_j taps[:, j] * u_(t - K + 1 + j) channel by channel; zeros before the start."""
    n, K = u.shape[0], taps.shape[1]
    y = torch.zeros_like(u)
    for t in range(n):
        for j in range(K):
            s = t - K + 1 + j
            if s >= 0:
                y[t] += taps[:, j] * u[s]
    return y


def rotation_rates(rot):
    """(rates [dims / 2] in float64, factor on cosine and sine)."""
    dims, base = int(rot["dims"]), float(rot["base"])
    i = torch.arange(dims // 2, dtype=torch.float64)
    rates = base ** (-2.0 * i / dims)
    sc = rot.get("scaling")
    if not sc:
        return rates, 1.0
    factor = float(sc["factor"])

    def dim_of(turns):
        """The dimension that makes `turns` full turns within the original length."""
        return dims * math.log(float(sc["original"]) / (2 * math.pi * turns)) / (2 * math.log(base))

    lo = max(math.floor(dim_of(float(sc["fast"]))), 0)
    hi = min(math.ceil(dim_of(float(sc["slow"]))), dims - 1)
    ramp = ((i - lo) / max(hi - lo, 0.001)).clamp(0.0, 1.0)
    return rates / factor * ramp + rates * (1.0 - ramp), 0.1 * math.log(factor) + 1.0


def rotate_halves(x, positions, rot):
    """Turns the pairs (i, i + dims / 2) of the last axis by position * rate_i; what lies beyond
    `dims` passes unchanged.  x is [tokens, ..., size]."""
    if not rot or not int(rot["dims"]):
        return x
    dims = int(rot["dims"])
    rates, factor = rotation_rates(rot)
    angle = positions.to(torch.float64)[:, None] * rates
    shape = (x.shape[0],) + (1,) * (x.dim() - 2) + (dims // 2,)
    cos = (torch.cos(angle) * factor).to(x.dtype).view(shape)
    sin = (torch.sin(angle) * factor).to(x.dtype).view(shape)
    u, v = x[..., : dims // 2], x[..., dims // 2 : dims]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, x[..., dims:]], dim=-1)


def projected(h, w, name: str, taps: int):
    """W h + b, then the short convolution where the layer has one."""
    y = h @ w[name].T + w[name + ".b"]
    return short_convolution(y, w[name + ".conv"]) if taps else y


def keys_values(h, positions, w, prefix: str, m: dict):
    """Keys [n, G, 2, D] as a cache holds them (convolved, rotated) and values [n, G, V]."""
    n, G, D, V = h.shape[0], m["kv_heads"], m["dim"], m["vdim"]
    k = projected(h, w, prefix + ".k", int(m.get("conv") or 0)).view(n, G, 2, D)
    v = projected(h, w, prefix + ".v", int(m.get("conv") or 0)).view(n, G, V)
    return rotate_halves(k, positions, m.get("rot")), v


def lambda_of(w, prefix: str, diff: float):
    """exp(lq1 . lk1) - exp(lq2 . lk2) + diff: the weight of the second map, one number a layer."""
    a = torch.exp((w[prefix + ".lq1"] * w[prefix + ".lk1"]).sum())
    b = torch.exp((w[prefix + ".lq2"] * w[prefix + ".lk2"]).sum())
    return a - b + diff


def one_map(q, k, v, scale: float, vis):
    """Ordinary softmax attention of one head: q [n, D], k [n, D], v [n, V]."""
    return torch.softmax(((q @ k.T) * scale).masked_fill(~vis, float("-inf")), dim=-1) @ v


def combine_maps(a1, a2, lam, diff: float, eps: float):
    """a1 - lambda a2, brought to unit root mean square over the value's elements, times 1 - diff."""
    return unit_rms(a1 - lam * a2, eps) * (1.0 - diff)


def differential_attention(h, positions, w, prefix: str, m: dict, eps: float, kv=None):
    """Two attentions per head over the same values, combined; `kv`: another layer's (keys,
    values) to read instead of projecting one's own.  Returns (output, (keys, values))."""
    n = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = projected(h, w, prefix + ".q", int(m.get("conv") or 0)).view(n, H, 2, D)
    q = rotate_halves(q, positions, m.get("rot"))
    if kv is None:
        kv = keys_values(h, positions, w, prefix, m)
    k, v = kv
    vis = visible(n, m.get("mask"))
    diff = float(m["diff"])
    lam = lambda_of(w, prefix, diff)
    gate = torch.sigmoid(h @ w[prefix + ".g"].T)  # [n, H]
    out = torch.zeros(n, H, V, dtype=h.dtype)
    for head in range(H):
        g = head // (H // G)
        a1, a2 = (one_map(q[:, head, c], k[:, g, c], v[:, g], float(m["scale"]), vis) for c in (0, 1))
        out[:, head] = combine_maps(a1, a2, lam, diff, eps) * gate[:, head, None]
    return out.reshape(n, H * V) @ w[prefix + ".o"].T, kv


def silu(z):
    return z * torch.sigmoid(z)


def lightning_recurrence(q, k, v, decay):
    """o_t = S_t^T q_t with S_t = decay S_(t-1) + k_t v_t^T for one head, S zero at the start."""
    S = torch.zeros(q.shape[1], v.shape[1], dtype=q.dtype)
    out = torch.zeros(q.shape[0], v.shape[1], dtype=q.dtype)
    for t in range(q.shape[0]):
        S = decay * S + torch.outer(k[t], v[t])
        out[t] = S.T @ q[t]
    return out


def lightning(h, w, prefix: str, m: dict, eps: float):
    """Linear attention with a fixed decay per head; the heads side by side are normed together,
    weighted, gated and projected."""
    n, H, D, V = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = silu(h @ w[prefix + ".q"].T).view(n, H, D)
    k = silu(h @ w[prefix + ".k"].T).view(n, H, D)
    v = silu(h @ w[prefix + ".v"].T).view(n, H, V)
    o = torch.stack([lightning_recurrence(q[:, a], k[:, a], v[:, a], float(m["decay"][a])) for a in range(H)], dim=1)
    y = unit_rms(o.reshape(n, H * V), eps) * w[prefix + ".norm"] * torch.sigmoid(h @ w[prefix + ".g"].T)
    return y @ w[prefix + ".o"].T


def feed_forward(h, w, prefix: str, m: dict):
    if m["kind"] != "dense":
        raise ValueError(f"unknown feed-forward kind {m['kind']!r}")
    return torch.relu(h @ w[prefix + ".up"].T) ** 2 @ w[prefix + ".down"].T


def forward(cfg: dict, w: dict, tokens, return_layers: bool = False):
    """Logits [tokens, vocab] of one sequence; with return_layers also the stream after every layer."""
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    positions = torch.arange(tokens.shape[0])
    eps, mult = float(cfg["norm"]["eps"]), float(cfg["residual_mult"])
    x = w["embed"][tokens]
    kept = {}  # keys and values by layer, for layers that read another's
    streams = []
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}", layer["mixer"]
        h = dynamic_tanh(x, w, p + ".norm1")
        if layer["type"] == "lightning":
            y = lightning(h, w, p + ".mix", m, eps)
        elif layer["type"] == "attention":
            source = m.get("kv_from")
            y, kept[i] = differential_attention(h, positions, w, p + ".mix", m, eps,
                                                kv=None if source is None else kept[int(source)])
        else:
            raise ValueError(f"unknown mixer type {layer['type']!r}")
        x = x + mult * y
        if layer.get("mlp"):
            x = x + mult * feed_forward(dynamic_tanh(x, w, p + ".norm2"), w, p + ".mlp", layer["mlp"])
        streams.append(x)
    logits = dynamic_tanh(x, w, "final.norm") @ w["embed"].T
    return (logits, torch.stack(streams)) if return_layers else logits


class PlainFozedra:
    """A model folder read once; `logits(ids)`, the stream after every layer, and greedy
    generation over it, in float64 unless told otherwise."""

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
