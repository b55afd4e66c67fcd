"""Plain, slow, whole-sequence Kisusun decoder used only as the test oracle.

One function per mechanism, written from the design's equations in this file's own notation; no cache, no batching,
position-by-position loops in attention, token-by-token loops in the routed experts, and no import from the product
package.  Everything runs in one floating type chosen by the caller (float64 by default).

Notation: a sequence is T tokens at positions 0..T-1; W is the model's width; every linear map is stored [out, in] and
applied as y = x @ M.T;  RMS(x, w) = x / sqrt(mean x^2 + eps) * w.

The design
* x = scale * embed[token]; a sublayer reads x as it is, and only what it returns is normalised:
  x <- x + RMS(mixer(x), norm1);  x <- x + RMS(ff(x), norm2)   (the second line may be missing)
* mixer: grouped-query attention; q and k are RMS-normalised over *all* heads' entries at once, then the first ``rot.dims``
  entries of every head turn in half-split pairs with frequencies divided by a constant; scores are scaled and capped, one is
  added to the softmax's denominator, a query sees itself and the mask.size - 1 tokens before it; values may be a blend of the
  layer's own with those of the first blending layer; every entry of the heads' results is gated by a sigmoid of its own
* feed-forward: down(silu(gate h) * up h), or experts of the clamped gated form chosen by sigmoid scores inside the best groups
  (a group counts as the sum of its two best), weighted by score * scale, with a shared expert beside them
* logits = logit_scale * embed RMS(x, final.norm)
"""
from __future__ import annotations

import json
from pathlib import Path

import torch
from safetensors import safe_open


# --------------------------------------------------------------------------- files
def read_config(model_dir) -> dict:
    return json.loads((Path(model_dir) / "config.json").read_text())


def read_weights(model_dir, dtype=torch.float64) -> dict:
    out = {}
    for f in sorted(Path(model_dir).glob("*.safetensors")):
        with safe_open(str(f), framework="pt") as fh:
            for name in fh.keys():
                out[name] = fh.get_tensor(name).to(dtype)
    return out


# --------------------------------------------------------------------------- small pieces
def same(x):
    return x


def rounder(act_dtype):
    """x as an engine that stores activations in ``act_dtype`` would hold it (None: exact); applied to what products and
    activations leave and to what products read, never to the residual stream, norms' insides or scores."""
    return same if act_dtype is None else (lambda x: x.to(act_dtype).to(x.dtype))


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps) * w


def silu(z):
    return z / (1.0 + torch.exp(-z))


def clamped_glu(g, u, limit):
    g = torch.clamp(g, max=limit)
    u = torch.clamp(u, min=-limit, max=limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1.0)


def cap_scores(s, cap):
    return s if cap is None else cap * torch.tanh(s / cap)


# --------------------------------------------------------------------------- rotation
def frequencies(dims, base, factor=1.0):
    return torch.tensor([base ** (-2.0 * i / dims) / factor for i in range(dims // 2)], dtype=torch.float64)


def rotate(x, positions, freqs):
    """x [T, heads, width]: entries i and i + n (n pairs) become (u cos a - v sin a, v cos a + u sin a), a = position *
    frequency i; entries past the 2 n-th pass."""
    n = freqs.numel()
    y = x.clone()
    for i in range(n):
        a = positions.to(torch.float64) * freqs[i]
        c, s = torch.cos(a).to(x.dtype)[:, None], torch.sin(a).to(x.dtype)[:, None]
        u, v = x[..., i], x[..., i + n]
        y[..., i] = u * c - v * s
        y[..., i + n] = v * c + u * s
    return y


# --------------------------------------------------------------------------- attention
def one_plus_softmax(s):
    """exp(s_j) / (1 + sum exp(s)) over the last dimension: a softmax with one more score, 0, that is dropped again."""
    m = torch.clamp(s.max(dim=-1, keepdim=True).values, min=0.0)
    e = torch.exp(s - m)
    return e / (torch.exp(-m) + e.sum(dim=-1, keepdim=True))


def windowed_attention(q, k, v, scale, cap=None, window=None):
    """q [T, H, D], k [T, G, D], v [T, G, E], one position at a time: query head h reads key/value head h // (H / G)."""
    T, H = q.shape[:2]
    rep = H // k.shape[1]
    k, v = k.repeat_interleave(rep, dim=1), v.repeat_interleave(rep, dim=1)
    out = torch.empty(T, H, v.shape[2], dtype=q.dtype)
    for n in range(T):
        lo = 0 if window is None else max(0, n - window + 1)
        s = cap_scores(torch.einsum("hd,jhd->hj", q[n], k[lo:n + 1]) * scale, cap)
        out[n] = torch.einsum("hj,jhe->he", one_plus_softmax(s), v[lo:n + 1])
    return out


def blend_values(v, first, lam):
    return (1.0 - lam) * v + lam * first


def attention(h, w, p, m, eps, positions, first_values, rnd=same):
    """(the mixer's output, the layer's own values before any blending).  ``first_values``: those of the first layer that
    blends, or None when this layer does not blend (or is that first one)."""
    T = h.shape[0]
    H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_norm(rnd(h @ w[p + "q"].T), w[p + "q.norm"], eps).view(T, H, D)
    k = rms_norm(rnd(h @ w[p + "k"].T), w[p + "k.norm"], eps).view(T, G, D)
    v = own = rnd(h @ w[p + "v"].T)
    rot = m.get("rot")
    if rot is not None and rot["dims"]:
        f = frequencies(rot["dims"], float(rot["base"]), float((rot.get("scaling") or {}).get("factor", 1.0)))
        q, k = rotate(q, positions, f), rotate(k, positions, f)
    if first_values is not None:
        v = blend_values(v, first_values, w[p + "vmix"])
    window = m["mask"]["size"] if m.get("mask") is not None else None
    o = windowed_attention(rnd(q), rnd(k), rnd(v).view(T, G, E), float(m["scale"]), m.get("softcap"), window)
    o = o.reshape(T, H * E) * torch.sigmoid(rnd(h @ w[p + "g"].T))
    return rnd(rnd(o) @ w[p + "o"].T), own


# --------------------------------------------------------------------------- feed-forwards
def dense(h, w, p, rnd=same):
    return rnd(rnd(silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T)


def expert(h, w, p, limit, rnd=same):
    return rnd(rnd(clamped_glu(h @ w[p + "gate"].T, h @ w[p + "up"].T, limit)) @ w[p + "down"].T)


def route(z, top, scale, groups=None):
    """z [T, E] -> (chosen [T][top], weights [T][top]); ``groups``: (count, keep)."""
    ids, weights = [], []
    for row in z:
        s = [float(a) for a in torch.sigmoid(row)]
        allowed = list(range(len(s)))
        if groups is not None:
            count, keep = groups
            size = len(s) // count
            worth = [sum(sorted(s[g * size:(g + 1) * size], reverse=True)[:2]) for g in range(count)]
            best = sorted(range(count), key=lambda g: (-worth[g], g))[:keep]
            allowed = [e for e in allowed if e // size in best]
        chosen = sorted(allowed, key=lambda e: (-s[e], e))[:top]
        ids.append(chosen)
        weights.append([s[e] * scale for e in chosen])
    return ids, weights


def routed_experts(h, w, p, mlp, rnd=same):
    r = mlp["router"]
    groups = (r["groups"]["count"], r["groups"]["keep"]) if r.get("groups") is not None else None
    ids, weights = route(h @ w[p + "router"].T, r["top"], float(r["scale"]), groups)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, a in zip(ids[t], weights[t]):
            out[t] += a * expert(h[t:t + 1], w, f"{p}e{e}.", float(mlp["expert"]["limit"]), rnd)[0]
    if mlp.get("shared") is not None:
        out = out + expert(h, w, p + "shared.", float(mlp["shared"]["limit"]), rnd)
    return out


def feed_forward(h, w, p, mlp, rnd=same):
    return dense(h, w, p, rnd) if mlp["kind"] == "dense" else routed_experts(h, w, p, mlp, rnd)


# --------------------------------------------------------------------------- the model
def forward(cfg, w, tokens, act_dtype=None, dtype=torch.float64, streams=None):
    """Logits [T, vocab] of one whole sequence.  ``streams``: a list that receives the residual stream after every layer."""
    rnd = rounder(act_dtype)
    w = {k: v.to(dtype) for k, v in w.items()}
    eps = float(cfg["norm"]["eps"])
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    positions = torch.arange(tokens.numel())
    x = w["embed"][tokens] * float(cfg["embedding"]["scale"])
    first_values = None
    for i, entry in enumerate(cfg["layers"]):
        p, m = f"l{i}.", entry["mixer"]
        if entry["type"] != "attention":
            raise ValueError(f"no mixer {entry['type']!r}")
        y, own = attention(rnd(x), w, p + "mix.", m, eps, positions, first_values if m.get("v_mix") else None, rnd)
        if m.get("v_mix") and first_values is None:
            first_values = own
        x = x + rms_norm(y, w[p + "norm1"], eps)
        if entry.get("mlp") is not None:
            x = x + rms_norm(feed_forward(rnd(x), w, p + "mlp.", entry["mlp"], rnd), w[p + "norm2"], eps)
        if streams is not None:
            streams.append(x)
    return rnd(rms_norm(x, w["final.norm"], eps)) @ w["embed"].T * float(cfg["logit_scale"])
