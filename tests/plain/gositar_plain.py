"""Plain, slow, whole-sequence Gositar decoder used only as the test oracle.

One function per mechanism, written from the design's equations in this file's own notation; no cache, no batching,
position-by-position loops in attention, token-by-token loops in the routed experts, and no import from the product
package.  Everything runs in one floating type chosen by the caller (float64 by default).

Notation: a sequence is T tokens at positions 0..T-1; W is the model's width; every linear map is stored [out, in] and
applied as y = x @ M.T;  LN(x, w) = (x - mean x) / sqrt(var x + eps) * w;  RMS(x, w) = x / sqrt(mean x^2 + eps) * w.

The design
* S streams X[s] of width W, all equal to embed[token] at the start
* a layer has two sublayers (mixer, feed-forward; the second may be missing), and each of them reads and writes the
  streams through numbers of its own:  u = sum_s a[s] X[s];  y = sublayer(LN(u));  X[t] <- sum_s M[s, t] X[s] + b[t] y
* mixers: ``latent_attention`` (neighbouring entries rotated in pairs, one gate per head) and ``latent_attention_2``
  (half-split pairs, no gate); both read keys and values through a normalised low-rank latent and share one rotated key
  part among the heads
* feed-forward: down(relu(up h)^2), or routed experts chosen inside the best groups, with a shared expert beside them
* logits = head LN(sum_s X[s], final.norm)
"""
from __future__ import annotations

import json
import math
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
    activations leave, never to the streams, norms' insides, scores or the router."""
    return same if act_dtype is None else (lambda x: x.to(act_dtype).to(x.dtype))


def layer_norm(x, w, eps):
    dev = x - x.mean(dim=-1, keepdim=True)
    return dev / torch.sqrt((dev * dev).mean(dim=-1, keepdim=True) + eps) * w


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps) * w


def relu_squared(z):
    return torch.where(z > 0, z * z, torch.zeros_like(z))


def clamped_glu(g, u, limit):
    g = torch.clamp(g, max=limit)
    u = torch.clamp(u, min=-limit, max=limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1.0)


# --------------------------------------------------------------------------- rotation
def yarn(dims, base, scaling=None):
    """(frequencies, one per pair, in double; the number that cosines and sines are multiplied by).  With ``scaling`` a
    pair's frequency goes from f (pairs that turn often within ``original`` positions) to f / factor (pairs that turn
    seldom) along a ramp over the pair's index, whose ends are where a pair turns ``fast`` and ``slow`` times."""
    n = dims // 2
    f = [base ** (-2.0 * i / dims) for i in range(n)]
    if scaling is None:
        return torch.tensor(f, dtype=torch.float64), 1.0
    factor, original, fast, slow = (float(scaling[k]) for k in ("factor", "original", "fast", "slow"))

    def index_of(turns):
        return dims * math.log(original / (turns * 2.0 * math.pi)) / (2.0 * math.log(base))

    lo, hi = max(math.floor(index_of(fast)), 0), min(math.ceil(index_of(slow)), dims - 1)
    out = []
    for i in range(n):
        r = (i - lo) / max(hi - lo, 0.001)
        r = min(max(r, 0.0), 1.0)
        out.append(f[i] / factor * r + f[i] * (1.0 - r))
    return torch.tensor(out, dtype=torch.float64), 0.1 * math.log(factor) + 1.0


def rotate(x, positions, freqs, gain, interleaved):
    """x [T, ..., width]: pair (u, v) of entries -> gain (u cos a - v sin a, v cos a + u sin a), a = position * frequency.
    Pairs are entries (2i, 2i + 1), or (i, i + n) for n pairs; entries past the 2 n-th pass."""
    n = freqs.numel()
    y = x.clone()
    for i in range(n):
        a = positions.to(torch.float64) * freqs[i]
        c, s = (gain * torch.cos(a)).to(x.dtype), (gain * torch.sin(a)).to(x.dtype)
        shape = [-1] + [1] * (x.dim() - 2)
        c, s = c.view(shape), s.view(shape)
        iu, iv = (2 * i, 2 * i + 1) if interleaved else (i, i + n)
        u, v = x[..., iu], x[..., iv]
        y[..., iu] = u * c - v * s
        y[..., iv] = v * c + u * s
    return y


# --------------------------------------------------------------------------- attention
def causal_attention(q, k, v, scale):
    """q, k [T, H, D], v [T, H, E]: softmax over the keys up to the token itself, one position at a time."""
    T, H = q.shape[:2]
    out = torch.empty(T, H, v.shape[2], dtype=q.dtype)
    for n in range(T):
        s = torch.einsum("hd,jhd->hj", q[n], k[:n + 1]) * scale
        s = s - s.max(dim=1, keepdim=True).values
        p = torch.exp(s)
        p = p / p.sum(dim=1, keepdim=True)
        out[n] = torch.einsum("hj,jhe->he", p, v[:n + 1])
    return out


def latent_attention(h, w, p, m, eps, positions, interleaved, gated, rnd=same):
    T = h.shape[0]
    H, D, R, E, C = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    freqs, gain = yarn(m["rot"]["dims"], float(m["rot"]["base"]), m["rot"].get("scaling"))
    q = rnd(h @ w[p + "q"].T).view(T, H, D + R)
    down = rnd(h @ w[p + "dkv"].T)
    c = rnd(rms_norm(down[:, :C], w[p + "dkv.norm"], eps))
    kr = rnd(rotate(down[:, C:], positions, freqs, gain, interleaved))
    qr = rnd(rotate(q[..., D:], positions, freqs, gain, interleaved))
    kf = rnd(c @ w[p + "uk"].T).view(T, H, D)
    v = rnd(c @ w[p + "uv"].T).view(T, H, E)
    o = causal_attention(torch.cat([q[..., :D], qr], dim=-1), torch.cat([kf, kr[:, None, :].expand(T, H, R)], dim=-1), v,
                         float(m["scale"]))
    if gated:
        o = o * torch.sigmoid(rnd(h @ w[p + "g"].T))[:, :, None]
    return rnd(rnd(o).reshape(T, H * E) @ w[p + "o"].T)


# --------------------------------------------------------------------------- feed-forwards
def dense(h, w, p, rnd=same):
    return rnd(rnd(relu_squared(rnd(h @ w[p + "up"].T))) @ w[p + "down"].T)


def expert(h, w, p, limit, rnd=same):
    return rnd(rnd(clamped_glu(rnd(h @ w[p + "gate"].T), rnd(h @ w[p + "up"].T), limit)) @ w[p + "down"].T)


def route(z, correction, top, groups=None):
    """z [T, E] -> (chosen [T][top], weights [T][top]); ``groups``: (count, keep)."""
    ids, weights = [], []
    for row in z:
        s = torch.softmax(row, dim=0)
        choice = s + correction if correction is not None else s
        allowed = list(range(row.numel()))
        if groups is not None:
            count, keep = groups
            size = row.numel() // count
            best = sorted(range(count), key=lambda g: (-float(choice[g * size:(g + 1) * size].max()), g))[:keep]
            allowed = [e for e in allowed if e // size in best]
        chosen = sorted(allowed, key=lambda e: (-float(choice[e]), e))[:top]
        total = sum(float(s[e]) for e in chosen) + 1e-20
        ids.append(chosen)
        weights.append([float(s[e]) / total for e in chosen])
    return ids, weights


def routed_experts(h, w, p, mlp, rnd=same):
    r = mlp["router"]
    groups = (r["groups"]["count"], r["groups"]["keep"]) if r.get("groups") is not None else None
    ids, weights = route(h @ w[p + "router"].T, w.get(p + "correction"), r["top"], groups)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, a in zip(ids[t], weights[t]):
            out[t] += a * expert(h[t:t + 1], w, f"{p}e{e}.", float(mlp["expert"]["limit"]), rnd)[0]
    if mlp.get("shared") is not None:
        out = out + expert(h, w, p + "shared.", float(mlp["shared"]["limit"]), rnd)
    return out


def feed_forward(h, w, p, mlp, rnd=same):
    return dense(h, w, p, rnd) if mlp["kind"] == "dense" else routed_experts(h, w, p, mlp, rnd)


# --------------------------------------------------------------------------- streams
def read_streams(X, a):
    """X [S, T, W], a [S] -> [T, W]"""
    u = torch.zeros_like(X[0])
    for s in range(X.shape[0]):
        u = u + a[s] * X[s]
    return u


def write_streams(X, M, b, y):
    """X[t] <- sum_s M[s, t] X[s] + b[t] y, all from the old streams."""
    S = X.shape[0]
    out = []
    for t in range(S):
        new = b[t] * y
        for s in range(S):
            new = new + M[s, t] * X[s]
        out.append(new)
    return torch.stack(out)


# --------------------------------------------------------------------------- the model
def forward(cfg, w, tokens, act_dtype=None, dtype=torch.float64, streams=None):
    """Logits [T, vocab] of one whole sequence.  ``streams``: a list that receives the sum of the streams after every
    layer."""
    rnd = rounder(act_dtype)
    w = {k: v.to(dtype) for k, v in w.items()}
    eps = float(cfg["norm"]["eps"])
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    positions = torch.arange(tokens.numel())
    X = torch.stack([w["embed"][tokens]] * int(cfg["streams"]))
    for i, entry in enumerate(cfg["layers"]):
        p, kind = f"l{i}.", entry["type"]
        if kind not in ("latent_attention", "latent_attention_2"):
            raise ValueError(f"no mixer {kind!r}")
        h = rnd(layer_norm(read_streams(X, w[p + "hc1.in"]), w[p + "norm1"], eps))
        y = latent_attention(h, w, p + "mix.", entry["mixer"], eps, positions, kind == "latent_attention",
                             kind == "latent_attention", rnd)
        X = write_streams(X, w[p + "hc1.mix"], w[p + "hc1.out"], y)
        if entry.get("mlp") is not None:
            h = rnd(layer_norm(read_streams(X, w[p + "hc2.in"]), w[p + "norm2"], eps))
            X = write_streams(X, w[p + "hc2.mix"], w[p + "hc2.out"], feed_forward(h, w, p + "mlp.", entry["mlp"], rnd))
        if streams is not None:
            streams.append(X.sum(dim=0))
    h = rnd(layer_norm(X.sum(dim=0), w["final.norm"], eps))
    return h @ w["head"].T
