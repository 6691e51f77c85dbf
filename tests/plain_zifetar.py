"""A plain, slow implementation of Zifetar in float64, one function per mechanism, written from
the design's equations.  It shares no code with the package: the tests compare the engine
against it.

Notation.  x: the residual stream [T, W].  rms(t) = t / sqrt(mean(t^2) + eps) over the last axis,
N(t) = rms(t) (1 + w).  The embedding is N(scale * row(token) + pair row(previous token, token)).  A
layer is x <- x + N1b(mixer(N1(x))); x <- x + N2b(ff(N2(x))) (the second only with a feed-forward).
Mixers: a delta rule with a decay per head and key channel behind short convolutions; retention, a
linear attention with a fixed decay per head; attention in chunks of positions beside a linear
attention with a decay per key channel.  Feed-forward: a routed mixture of small gated ones.
"""
import math

import torch

F64 = torch.float64


def rms(t, eps):
    return t / torch.sqrt((t * t).mean(dim=-1, keepdim=True) + eps)


def norm(t, eps, w):
    return rms(t, eps) * (1.0 + w)


def silu(t):
    return t * torch.sigmoid(t)


def softplus(t):
    return torch.log1p(torch.exp(-t.abs())) + torch.clamp(t, min=0)


# ---- embedding --------------------------------------------------------------------------------------

def pair_rows(ids, b):
    """The row of the pair table for every token; the last row for the first token of a sequence."""
    out = [b["buckets"]]
    for before, cur in zip(ids[:-1], ids[1:]):
        out.append((int(before) * b["mul_prev"] + int(cur) * b["mul_cur"]) % b["buckets"])
    return out


def embedding(w, cfg, ids):
    ids = [int(i) for i in ids]
    x = w["embed"][ids] * cfg["embedding"]["scale"]
    b = cfg["embedding"].get("bigram")
    if b:
        x = x + w["bigram"][pair_rows(ids, b)]
    return norm(x, cfg["norm"]["eps"], w["embed.norm"])


# ---- positions --------------------------------------------------------------------------------------

def frequencies(rot):
    """Angles per position of the dims/2 pairs: base^(-2i/dims), and with `scaling` divided by `factor`
    where the wavelength is longer than original/low, kept where it is shorter than original/high, a
    mixture between."""
    base, dims, sc = float(rot["base"]), rot["dims"], rot.get("scaling")
    out = []
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if sc:
            length = 2 * math.pi / f
            if length > sc["original"] / sc["low"]:
                f = f / sc["factor"]
            elif length >= sc["original"] / sc["high"]:
                s = (sc["original"] / length - sc["low"]) / (sc["high"] - sc["low"])
                f = (1 - s) * f / sc["factor"] + s * f
        out.append(f)
    return torch.tensor(out, dtype=F64)


def rotate(t, pos, rot):
    """t [T, heads, d]: the first `dims` channels of every head turned by pos * f_i, channel i with i + dims/2."""
    if not rot or not rot["dims"]:
        return t
    half = rot["dims"] // 2
    a = pos.to(F64)[:, None, None] * frequencies(rot)
    c, s = torch.cos(a).to(t.dtype), torch.sin(a).to(t.dtype)
    u, v = t[..., :half], t[..., half:2 * half]
    return torch.cat([u * c - v * s, v * c + u * s, t[..., 2 * half:]], dim=-1)


# ---- recurrences ------------------------------------------------------------------------------------

def short_conv(u, w):
    """silu of a causal convolution per channel: u [T, C], w [C, taps], the last tap on the present row."""
    taps = w.shape[1]
    padded = torch.cat([torch.zeros(taps - 1, u.shape[1], dtype=u.dtype), u])
    return silu(sum(padded[j:j + len(u)] * w[:, j] for j in range(taps)))


def unit(t):
    return t / torch.sqrt((t * t).sum(dim=-1, keepdim=True) + 1e-6)


def linear_heads(q, k, v, g, beta=None, S=None, left=None):
    """q, k, g [T, H, d], v [T, H, dv]: S <- g S + k u^T, o = S^T q, row by row; u = v, or with `beta`
    [T, H] the delta rule's beta (v - (g S)^T k).  `left`: a list that receives, per row, what is left of o when its
    terms have cancelled (its length over the length of the sum of their magnitudes, times sqrt(d): about 1 for terms of
    any sign; the smallest of the heads): a norm over the head makes what is left large again, with the rounding of the
    terms."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[-1], dtype=q.dtype) if S is None else S
    out, kept = [], []
    for t in range(T):
        S = g[t][:, :, None] * S
        u = v[t]
        if beta is not None:
            u = beta[t][:, None] * (u - (S * k[t][:, :, None]).sum(dim=1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out.append((S * q[t][:, :, None]).sum(dim=1))
        kept.append(d ** 0.5 * (out[-1].norm(dim=-1) / (S * q[t][:, :, None]).abs().sum(dim=1).norm(dim=-1).clamp(min=1e-30)).min())
    if left is not None:
        left.append(torch.stack(kept))
    return torch.stack(out), S


def delta_inputs(h, w, p, m):
    """q, k, v, the decays and beta of a delta rule's rows, every one per head."""
    T, H, G, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (short_conv(h @ w[p + n].T, w[p + n + ".conv"]) for n in "qkv")
    q = (unit(q.view(T, G, d)) * d ** -0.5).repeat_interleave(H // G, dim=1)
    k = unit(k.view(T, G, d)).repeat_interleave(H // G, dim=1)
    z = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "dt_bias"]
    g = torch.exp(-torch.exp(w[p + "A_log"])[:, None] * softplus(z).view(T, H, d))
    return q, k, v.view(T, H, dv), g, torch.sigmoid(h @ w[p + "b"].T)


def channel_delta(h, w, p, m, pos, eps, left=None):
    T, H, dv = h.shape[0], m["heads"], m["vdim"]
    o, _ = linear_heads(*delta_inputs(h, w, p, m), left=left)
    gate = torch.sigmoid((h @ w[p + "g1"].T) @ w[p + "g2"].T)
    return ((rms(o, eps) * w[p + "norm"]).reshape(T, H * dv) * gate) @ w[p + "o"].T


def retention(h, w, p, m, pos, eps, left=None):
    T, H, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = rotate((h @ w[p + "q"].T).view(T, H, d), pos, m.get("rot"))
    k = rotate((h @ w[p + "k"].T).view(T, H, d), pos, m.get("rot")) * d ** -0.5
    v = (h @ w[p + "v"].T).view(T, H, dv)
    g = torch.tensor(m["decay"], dtype=h.dtype)[None, :, None].expand(T, H, d)
    o, _ = linear_heads(q, k, v, g, left=left)
    return (rms(o, eps).reshape(T, H * dv) * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def gated_linear(h, w, p, m, eps, left=None):
    T, H, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].T).view(T, H, d) * d ** -0.5
    k = (h @ w[p + "k"].T).view(T, H, d)
    v = (h @ w[p + "v"].T).view(T, H, dv)
    z = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "a2.b"]
    o, _ = linear_heads(q, k, v, torch.sigmoid(z).pow(1.0 / m["tau"]).view(T, H, d), left=left)
    return ((rms(o, eps) * w[p + "norm"]).reshape(T, H * dv) * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


# ---- attention --------------------------------------------------------------------------------------

def chunk_mask(pos, size):
    """[T, T] bool: row i sees column j iff j <= i and both lie in one run of `size` positions."""
    ok = pos[:, None] >= pos[None, :]
    return ok & (pos[:, None] // size == pos[None, :] // size) if size else ok


def chunked_attention(h, w, p, m, pos, eps):
    T, H, G, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].T + w[p + "q.b"]).view(T, H, d)
    k = (h @ w[p + "k"].T + w[p + "k.b"]).view(T, G, d)
    v = (h @ w[p + "v"].T + w[p + "v.b"]).view(T, G, dv).repeat_interleave(H // G, dim=1)
    q = rotate(rms(q, eps) * w[p + "q.norm"], pos, m.get("rot"))
    k = rotate(rms(k, eps) * w[p + "k.norm"], pos, m.get("rot")).repeat_interleave(H // G, dim=1)
    s = (q.transpose(0, 1) @ k.permute(1, 2, 0)) * m["scale"]
    s = s.masked_fill(~chunk_mask(pos, (m.get("mask") or {}).get("size"))[None], -math.inf)
    o = torch.softmax(s, dim=-1) @ v.transpose(0, 1)
    return o.transpose(0, 1).reshape(T, H * dv) @ w[p + "o"].T


def parallel(h, w, p, m, pos, eps, left=None):
    return (m["left_scale"] * chunked_attention(h, w, p + "left.", m["left"], pos, eps)
            + m["right_scale"] * gated_linear(h, w, p + "right.", m["right"], eps, left))


MIXERS = {"channel_delta": channel_delta, "retention": retention, "parallel": parallel}


# ---- feed-forward -----------------------------------------------------------------------------------

def gated_expert(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route(h, w, p, top, margins=None):
    """[T, E] weights: the softmax over the `top` largest logits (of equal ones the smaller index), 0
    elsewhere.  `margins`: a list that receives, per row, by how much the last chosen one was ahead."""
    z = h @ w[p + "router"].T + w[p + "router.b"]
    order = torch.sort(z, dim=-1, descending=True, stable=True)
    if margins is not None:
        margins.append(order.values[:, top - 1] - order.values[:, top] if top < z.shape[1]
                       else torch.full((len(z),), math.inf, dtype=z.dtype))
    picked = torch.softmax(order.values[:, :top], dim=-1)
    return torch.zeros_like(z).scatter_(1, order.indices[:, :top], picked)


def routed_ff(h, w, p, mlp, margins=None):
    wt = route(h, w, p, mlp["router"]["top"], margins)
    y = torch.zeros(h.shape[0], w[p + "e0.down"].shape[0], dtype=h.dtype)
    for e in range(mlp["router"]["experts"]):
        rows = (wt[:, e] != 0).nonzero().flatten()
        if len(rows):
            y[rows] += wt[rows, e:e + 1] * gated_expert(h[rows], w, f"{p}e{e}.")
    return y


# ---- the model --------------------------------------------------------------------------------------

def forward(w, cfg, ids, dtype=F64, streams=None, margins=None, left=None):
    """Logits [T, vocab] of one sequence.  `streams`: a list that receives the stream after every
    layer; `margins`: see `route`; `left`: see `linear_heads`."""
    w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in w.items()}
    eps = cfg["norm"]["eps"]
    pos = torch.arange(len(ids))
    x = embedding(w, cfg, ids)
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        y = MIXERS[layer["type"]](norm(x, eps, w[p + "norm1"]), w, p + "mix.", layer["mixer"], pos, eps, left)
        x = x + norm(y, eps, w[p + "norm1b"])
        if layer.get("mlp"):
            y = routed_ff(norm(x, eps, w[p + "norm2"]), w, p + "mlp.", layer["mlp"], margins)
            x = x + norm(y, eps, w[p + "norm2b"])
        if streams is not None:
            streams.append(x)
    return norm(x, eps, w["final.norm"]) @ w["head"].T


def generate_greedy(w, cfg, ids, n, dtype=F64):
    ids = list(ids)
    out = []
    for _ in range(n):
        t = int(torch.argmax(forward(w, cfg, ids, dtype)[-1]))
        out.append(t)
        ids.append(t)
    return out


def tensor_shapes(cfg, ranks=(16, 16)):
    """Names and shapes; `ranks`: the inner sizes of the decays' and gates' two-step projections (delta rule, linear
    attention), which the tensors alone give."""
    W, V = cfg["width"], cfg["vocab"]
    s = {"embed": (V, W), "head": (V, W), "final.norm": (W,), "embed.norm": (W,)}
    if cfg["embedding"].get("bigram"):
        s["bigram"] = (cfg["embedding"]["bigram"]["buckets"] + 1, W)
    for i, layer in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", layer["mixer"], layer.get("mlp")
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if f else ()):
            s[p + n] = (W,)
        p += "mix."
        if layer["type"] == "parallel":
            a, r = m["left"], m["right"]
            H, G, d, dv = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            for n, size in (("q", H * d), ("k", G * d), ("v", G * dv)):
                s.update({f"{p}left.{n}": (size, W), f"{p}left.{n}.b": (size,)})
            s.update({p + "left.q.norm": (d,), p + "left.k.norm": (d,), p + "left.o": (W, H * dv)})
            p, H, d, dv, R = p + "right.", r["heads"], r["dim"], r["vdim"], ranks[1]
            s.update({p + "q": (H * d, W), p + "k": (H * d, W), p + "v": (H * dv, W), p + "g": (H * dv, W), p + "o": (W, H * dv),
                      p + "norm": (dv,), p + "a1": (R, W), p + "a2": (H * d, R), p + "a2.b": (H * d,)})
        else:
            H, d, dv = m["heads"], m["dim"], m["vdim"]
            G = m["kv_heads"] if layer["type"] == "channel_delta" else H
            for n, size in (("q", G * d), ("k", G * d), ("v", H * dv)):
                s[p + n] = (size, W)
                if layer["type"] == "channel_delta":
                    s[p + n + ".conv"] = (size, m["conv"])
            if layer["type"] == "channel_delta":
                R = ranks[0]
                s.update({p + "b": (H, W), p + "A_log": (H,), p + "norm": (dv,), p + "a1": (R, W), p + "a2": (H * d, R),
                          p + "dt_bias": (H * d,), p + "g1": (R, W), p + "g2": (H * dv, R)})
            else:
                s[p + "g"] = (H * dv, W)
            s[p + "o"] = (W, H * dv)
        if f:
            p, E, ff = f"l{i}.mlp.", f["router"]["experts"], f["expert"]["ff"]
            for e in range(E):
                s.update({f"{p}e{e}.gate": (ff, W), f"{p}e{e}.up": (ff, W), f"{p}e{e}.down": (W, ff)})
            s.update({p + "router": (E, W), p + "router.b": (E,)})
    return s


def random_weights(cfg, seed, gain=1.0, dtype=torch.bfloat16, ranks=(16, 16)):
    """Weights of the tests' own making: products N(0, gain / sqrt(fan in)), norms near their neutral value,
    decays from nearly none to nearly all."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg, ranks).items():
        leaf = name.split(".")[-1]
        r = torch.randn(shape, generator=g)
        if name.endswith("mix.norm") or name.endswith("right.norm") or ".q.norm" in name or ".k.norm" in name:
            t = 1.0 + 0.3 * r
        elif "norm" in leaf:
            t = 0.3 * r
        elif leaf == "A_log":
            t = -1.0 + 1.2 * r
        elif leaf == "dt_bias":
            t = -2.5 + 1.5 * r
        elif name.endswith("a2.b"):
            t = 1.0 + r
        elif leaf == "b" and len(shape) == 1:
            t = 0.5 * r
        elif leaf == "conv":
            t = 0.3 * r + torch.eye(1, shape[1]).flip(1)[0]
        elif name in ("embed", "bigram"):
            t = r if name == "bigram" else r / cfg["embedding"]["scale"]
        elif leaf == "router":
            t = 2.0 * r / math.sqrt(shape[1])
        else:
            t = gain * r / math.sqrt(shape[-1])
        out[name] = t.to(dtype)
    return out
