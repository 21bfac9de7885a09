"""A plain, slow implementation of the Balenex design, one function per
mechanism, written from the design's equations in float64.  It shares no code
with the package: tests compare the engine against it.

Notation: x is the residual stream [n, width] of ONE sequence, processed whole;
position t is row t.  Attention is computed query by query over explicit lists
of keys, the recurrence token by token.
"""

from __future__ import annotations

import json
import math
import os

import torch

F64 = torch.float64


# -- norms and activations ------------------------------------------------------

def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def rms_norm(x, w, eps):
    return unit_rms(x, eps) * w


def group_norm(x, w, groups, eps):
    """Each of ``groups`` equal consecutive parts over its own root mean square."""
    parts = x.reshape(*x.shape[:-1], groups, x.shape[-1] // groups)
    return unit_rms(parts, eps).reshape(x.shape) * w


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


# -- short convolution ------------------------------------------------------------

def short_conv(u, w):
    """u [n, C], w [C, taps]: y_t = sum_j w[:, j] u_(t - taps + 1 + j)."""
    n, taps = u.shape[0], w.shape[1]
    out = torch.zeros_like(u)
    for t in range(n):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                out[t] += w[:, j] * u[s]
    return out


# -- rotation ---------------------------------------------------------------------

def rotate(v, pos: float, base: float, dims: int):
    """Rows of v [..., size]: dims m and m + dims/2 turn by pos * base^(-2m/dims),
    m < dims/2; dims past ``dims`` stay."""
    half = dims // 2
    out = v.clone()
    for m in range(half):
        a = pos * base ** (-2.0 * m / dims)
        c, s = math.cos(a), math.sin(a)
        out[..., m] = v[..., m] * c - v[..., m + half] * s
        out[..., m + half] = v[..., m + half] * c + v[..., m] * s
    return out


# -- what a query sees ---------------------------------------------------------------

def keys_first_and_window(i: int, size: int, keep: int) -> list:
    return [j for j in range(i + 1) if i - j < size or j < keep]


def keys_window(i: int, size: int) -> list:
    return [j for j in range(i + 1) if i - j < size]


def pooled_seen(i: int, size: int, pool: int) -> int:
    """How many blocks 0, 1, ... of ``pool`` positions lie wholly before the
    window of position i."""
    b = 0
    while b * pool + pool - 1 <= i - size:
        b += 1
    return b


def attend(q, keys, values, scale):
    """q [H, dim], keys [H, N, dim], values [H, N, vdim] -> [H, vdim]."""
    s = (keys * q.unsqueeze(1)).sum(-1) * scale
    p = torch.exp(s - s.max(dim=1, keepdim=True).values)
    p = p / p.sum(dim=1, keepdim=True)
    return (p.unsqueeze(-1) * values).sum(1)


# -- mixers -------------------------------------------------------------------------

def conv_attention(h, w, m, eps):
    """The left half of a parallel layer.  m: heads, kv_heads, dim, vdim, scale,
    conv, mask {size, keep_first}, rot {base, dims}."""
    n = h.shape[0]
    nh, ng, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = short_conv(h @ w["q"].T + w["q.b"], w["q.conv"]).view(n, nh, d)
    k = short_conv(h @ w["k"].T + w["k.b"], w["k.conv"]).view(n, ng, d)
    v = short_conv(h @ w["v"].T + w["v.b"], w["v.conv"]).view(n, ng, dv)
    q = rms_norm(q, w["q.norm"], eps)
    k = rms_norm(k, w["k.norm"], eps)
    base, dims = m["rot"]["base"], m["rot"]["dims"]
    q = torch.stack([rotate(q[t], t, base, dims) for t in range(n)])
    k = torch.stack([rotate(k[t], t, base, dims) for t in range(n)])
    v = torch.stack([rotate(v[t], t, base, dv) for t in range(n)])
    of = torch.arange(nh) // (nh // ng)
    out = torch.zeros(n, nh, dv, dtype=F64)
    for i in range(n):
        seen = keys_first_and_window(i, m["mask"]["size"], m["mask"]["keep_first"])
        o = attend(q[i], k[seen][:, of].transpose(0, 1), v[seen][:, of].transpose(0, 1),
                   m["scale"])
        out[i] = rotate(o, -i, base, dv)
    return out.reshape(n, nh * dv) @ w["o"].T


def gated_linear_attention(h, w, m, eps):
    """The right half of a parallel layer.  m: heads, dim, vdim, tau."""
    n = h.shape[0]
    nh, d, dv = m["heads"], m["dim"], m["vdim"]
    q = (h @ w["q"].T).view(n, nh, d) * d ** -0.5
    k = (h @ w["k"].T).view(n, nh, d)
    v = (h @ w["v"].T).view(n, nh, dv)
    z = (h @ w["a1"].T) @ w["a2"].T + w["a2.b"]
    alpha = (sigmoid(z) ** (1.0 / m["tau"])).view(n, nh, d)
    state = torch.zeros(nh, d, dv, dtype=F64)
    out = torch.zeros(n, nh, dv, dtype=F64)
    for t in range(n):
        state = alpha[t].unsqueeze(-1) * state + k[t].unsqueeze(-1) * v[t].unsqueeze(1)
        out[t] = (state * q[t].unsqueeze(-1)).sum(1)
    out = rms_norm(out, w["norm"], eps).reshape(n, nh * dv)
    return (out * silu(h @ w["g"].T)) @ w["o"].T


def parallel(h, w, m, eps):
    lw = {k[5:]: t for k, t in w.items() if k.startswith("left.")}
    rw = {k[6:]: t for k, t in w.items() if k.startswith("right.")}
    left = conv_attention(h, lw, m["left"], eps)
    right = gated_linear_attention(h, rw, m["right"], eps)
    return 0.5 * (rms_norm(left, lw["out"], eps) + rms_norm(right, rw["out"], eps))


def pooled_attention(h, w, m, eps):
    """m: heads, kv_heads, dim, vdim, scale, mask {size, pool}."""
    n = h.shape[0]
    nh, ng, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = unit_rms((h @ w["q"].T + w["q.b"]).view(n, nh, d), eps)
    k = unit_rms((h @ w["k"].T + w["k.b"]).view(n, ng, d), eps)
    v = (h @ w["v"].T + w["v.b"]).view(n, ng, dv)
    size, pool = m["mask"]["size"], m["mask"]["pool"]
    of = torch.arange(nh) // (nh // ng)
    out = torch.zeros(n, nh, dv, dtype=F64)
    for i in range(n):
        seen = keys_window(i, size)
        keys, vals = [k[seen]], [v[seen]]
        for b in range(pooled_seen(i, size, pool)):
            keys.append(k[b * pool:(b + 1) * pool].mean(0, keepdim=True))
            vals.append(v[b * pool:(b + 1) * pool].mean(0, keepdim=True))
        kk, vv = torch.cat(keys)[:, of], torch.cat(vals)[:, of]
        out[i] = attend(q[i], kk.transpose(0, 1), vv.transpose(0, 1), m["scale"])
    return out.reshape(n, nh * dv) @ w["o"].T + w["o.b"]


# -- feed-forward ---------------------------------------------------------------------

def gated_ff(h, w):
    a = silu(h @ w["gate"].T + w["gate.b"]) * (h @ w["up"].T + w["up.b"])
    return a @ w["down"].T + w["down.b"]


# -- the model ------------------------------------------------------------------------

def _sub(w: dict, prefix: str) -> dict:
    return {k[len(prefix):]: v.to(F64) for k, v in w.items() if k.startswith(prefix)}


def forward(cfg: dict, w: dict, tokens: list, layers_out: list | None = None):
    """Logits [n, vocab] of one sequence; ``layers_out`` collects the stream
    after every layer."""
    eps, groups = cfg["norm"]["eps"], cfg["norm"]["groups"]
    norm = lambda v, name: group_norm(v, w[name].to(F64), groups, eps)
    x = w["embed"].to(F64)[torch.tensor(tokens)]
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        mixer = {"parallel": parallel, "attention": pooled_attention}[layer["type"]]
        y = mixer(norm(x, p + "norm1"), _sub(w, p + "mix."), layer["mixer"], eps)
        x = x + norm(y, p + "norm1b")
        if layer.get("mlp") is not None:
            y = gated_ff(norm(x, p + "norm2"), _sub(w, p + "mlp."))
            x = x + norm(y, p + "norm2b")
        if layers_out is not None:
            layers_out.append(x.clone())
    return norm(x, "final.norm") @ w["head"].to(F64).T


# -- making small models ----------------------------------------------------------------

def mixer_shapes(kind: str, m: dict, width: int, rank: int = 5) -> dict:
    """Tensor names (short) and shapes of one mixer; ``rank``: rows of the
    decay's inner projection."""
    if kind == "attention":
        nh, ng, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        return {"q": (nh * d, width), "q.b": (nh * d,), "k": (ng * d, width), "k.b": (ng * d,),
                "v": (ng * dv, width), "v.b": (ng * dv,), "o": (width, nh * dv), "o.b": (width,)}
    s = {}
    a = m["left"]
    nh, ng, d, dv, taps = a["heads"], a["kv_heads"], a["dim"], a["vdim"], a["conv"]
    for n, rows in (("q", nh * d), ("k", ng * d), ("v", ng * dv)):
        s.update({f"left.{n}": (rows, width), f"left.{n}.b": (rows,),
                  f"left.{n}.conv": (rows, taps)})
    s.update({"left.q.norm": (d,), "left.k.norm": (d,), "left.o": (width, nh * dv),
              "left.out": (width,)})
    r = m["right"]
    nh, d, dv = r["heads"], r["dim"], r["vdim"]
    s.update({"right.q": (nh * d, width), "right.k": (nh * d, width),
              "right.v": (nh * dv, width), "right.g": (nh * dv, width),
              "right.o": (width, nh * dv), "right.norm": (dv,), "right.a1": (rank, width),
              "right.a2": (nh * d, rank), "right.a2.b": (nh * d,), "right.out": (width,)})
    return s


def tensor_shapes(cfg: dict, rank: int = 5) -> dict:
    width, vocab = cfg["width"], cfg["vocab"]
    shapes = {"embed": (vocab, width), "final.norm": (width,), "head": (vocab, width)}
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        shapes.update({p + "norm1": (width,), p + "norm1b": (width,)})
        for n, s in mixer_shapes(layer["type"], layer["mixer"], width, rank).items():
            shapes[p + "mix." + n] = s
        if layer.get("mlp") is not None:
            ff = layer["mlp"]["ff"]
            shapes.update({p + "norm2": (width,), p + "norm2b": (width,),
                           p + "mlp.gate": (ff, width), p + "mlp.gate.b": (ff,),
                           p + "mlp.up": (ff, width), p + "mlp.up.b": (ff,),
                           p + "mlp.down": (width, ff), p + "mlp.down.b": (width,)})
    return shapes


def random_tensor(name: str, shape, g):
    """Values that keep activations O(1)."""
    leaf = name.split(".")[-1]
    if "norm" in leaf or leaf == "out":
        return 1.0 + 0.2 * torch.randn(shape, generator=g)
    if leaf == "embed":
        return torch.randn(shape, generator=g)
    if leaf == "b":
        return 0.5 * torch.randn(shape, generator=g)
    if leaf == "conv":
        t = 0.4 * torch.randn(shape, generator=g)
        t[..., -1] += 0.7
        return t
    if leaf == "a2":
        return 2.0 * torch.randn(shape, generator=g) / math.sqrt(shape[-1])
    return torch.randn(shape, generator=g) / math.sqrt(shape[-1])


def random_weights(cfg: dict, seed: int = 0, dtype=torch.bfloat16, rank: int = 5) -> dict:
    """Rounded to ``dtype`` so that engine and oracle start from the same numbers."""
    g = torch.Generator().manual_seed(seed)
    return {n: random_tensor(n, s, g).to(dtype) for n, s in tensor_shapes(cfg, rank).items()}


def write_model(path: str, cfg: dict, weights: dict) -> None:
    from safetensors.torch import save_file

    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in weights.items()},
              os.path.join(path, "model.safetensors"))
