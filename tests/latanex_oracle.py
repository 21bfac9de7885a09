"""A plain, slow implementation of the Latanex design, one function per
mechanism, written from the design's equations in float64.  It shares no code
with the package: tests compare the engine against it.

Notation: x is the residual stream [n, width] of ONE sequence, processed whole;
position t is row t.  Attention is computed query by query over explicit lists
of keys, the recurrence and the experts token by token.
"""

from __future__ import annotations

import json
import math
import os

import torch

F64 = torch.float64


# -- norms and activations ------------------------------------------------------

def tanh_norm(x, alpha, w, b):
    """No statistics: every element on its own."""
    return torch.tanh(alpha * x) * w + b


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return torch.log1p(torch.exp(-z.abs())) + torch.clamp(z, min=0.0)


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


# -- attention --------------------------------------------------------------------

def keys_window(i: int, size: int) -> list:
    return [j for j in range(i + 1) if i - j < size]


def attend(q, keys, values, scale, cap, sink):
    """q [H, dim], keys [H, N, dim], values [H, N, vdim], sink [H] -> [H, vdim].
    The sink is one more exponential in the denominator, as it is."""
    s = cap * torch.tanh((keys * q.unsqueeze(1)).sum(-1) * scale / cap)
    m = torch.maximum(s.max(dim=1).values, sink)
    p = torch.exp(s - m.unsqueeze(1))
    den = p.sum(dim=1) + torch.exp(sink - m)
    return (p.unsqueeze(-1) * values).sum(1) / den.unsqueeze(-1)


def attention(h, w, m, eps, v_first):
    """m: heads, kv_heads, dim, vdim, scale, softcap, mask {size}, v_mix.
    ``v_first``: values of the first mixing layer, None in that layer itself.
    Returns (rows, this layer's values)."""
    n = h.shape[0]
    nh, ng, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    # the norm's mean runs over all heads at once
    q = (unit_rms(h @ w["q"].T + w["q.b"], eps) * w["q.norm"]).view(n, nh, d)
    k = (unit_rms(h @ w["k"].T + w["k.b"], eps) * w["k.norm"]).view(n, ng, d)
    v = h @ w["v"].T + w["v.b"]
    if m["v_mix"] and v_first is not None:
        lam = w["vmix"]
        v = (1.0 - lam) * v + lam * v_first
    vh = v.view(n, ng, dv)
    of = torch.arange(nh) // (nh // ng)
    out = torch.zeros(n, nh, dv, dtype=F64)
    for i in range(n):
        seen = keys_window(i, m["mask"]["size"])
        out[i] = attend(q[i], k[seen][:, of].transpose(0, 1), vh[seen][:, of].transpose(0, 1),
                        m["scale"], m["softcap"], w["sink"])
    return out.reshape(n, nh * dv) @ w["o"].T, v


# -- gated delta rule ----------------------------------------------------------------

def unit_vectors(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta(h, w, m, eps):
    """m: heads, kv_heads, dim, vdim, conv."""
    n = h.shape[0]
    nh, ng, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(short_conv(h @ w[c].T, w[c + ".conv"])) for c in "qkv")
    q = unit_vectors(q.view(n, ng, d)) * d ** -0.5
    k = unit_vectors(k.view(n, ng, d))
    v = v.view(n, nh, dv)
    beta = sigmoid(h @ w["b"].T)
    g = torch.exp(-torch.exp(w["A_log"]) * softplus(h @ w["a"].T + w["dt_bias"]))
    out = torch.zeros(n, nh, dv, dtype=F64)
    for head in range(nh):
        qk = head // (nh // ng)
        state = torch.zeros(d, dv, dtype=F64)
        for t in range(n):
            state = g[t, head] * state
            u = beta[t, head] * (v[t, head] - state.T @ k[t, qk])
            state = state + torch.outer(k[t, qk], u)
            out[t, head] = state.T @ q[t, qk]
    out = (unit_rms(out, eps) * w["norm"]).reshape(n, nh * dv)
    return (out * silu(h @ w["g"].T)) @ w["o"].T


# -- feed-forward ---------------------------------------------------------------------

def dense_ff(h, w):
    return (silu(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


def clamped_expert(h, w, limit):
    g = torch.clamp(h @ w["gate"].T, max=limit)
    u = torch.clamp(h @ w["up"].T, min=-limit, max=limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w["down"].T


def route(z, correction, r):
    """One token's chosen experts and weights, z [E] logits."""
    s = sigmoid(z)
    choice = (s + correction).tolist()
    n = len(choice)
    groups = r.get("groups") or {"count": 1, "keep": 1}
    size = n // groups["count"]
    score = [sum(sorted(choice[a * size:(a + 1) * size])[-2:]) for a in range(groups["count"])]
    kept = sorted(range(groups["count"]), key=lambda a: -score[a])[:groups["keep"]]
    allowed = [e for e in range(n) if e // size in kept]
    ids = sorted(allowed, key=lambda e: -choice[e])[:r["top"]]
    total = sum(float(s[e]) for e in ids) + 1e-20
    return ids, [float(s[e]) / total * r["scale"] for e in ids]


def moe(h, w, f):
    out = torch.zeros_like(h)
    z = h @ w["router"].T
    for t in range(h.shape[0]):
        for e, weight in zip(*route(z[t], w["correction"], f["router"])):
            ew = {k: w[f"e{e}.{k}"] for k in ("gate", "up", "down")}
            out[t] += weight * clamped_expert(h[t], ew, f["expert"]["limit"])
    if f.get("shared"):
        sw = {k: w[f"shared.{k}"] for k in ("gate", "up", "down")}
        out = out + clamped_expert(h, sw, f["shared"]["limit"])
    return out


def feed_forward(h, w, f):
    return dense_ff(h, w) if f["kind"] == "dense" else moe(h, w, f)


# -- the model ------------------------------------------------------------------------

def _sub(w: dict, prefix: str) -> dict:
    return {k[len(prefix):]: v.to(F64) for k, v in w.items() if k.startswith(prefix)}


def forward(cfg: dict, w: dict, tokens: list, layers_out: list | None = None):
    """Logits [n, vocab] of one sequence; ``layers_out`` collects the stream
    after every layer."""
    eps = cfg["norm"]["eps"]

    def norm(v, name):
        t = lambda s: w[name + s].to(F64)
        return tanh_norm(v, t(".alpha"), t(""), t(".b"))

    x = w["embed"].to(F64)[torch.tensor(tokens)] * cfg["embedding"]["scale"]
    v_first = None
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        h, mw, m = norm(x, p + "norm1"), _sub(w, p + "mix."), layer["mixer"]
        if layer["type"] == "attention":
            y, v = attention(h, mw, m, eps, v_first)
            if m["v_mix"] and v_first is None:
                v_first = v
        else:
            y = delta(h, mw, m, eps)
        x = x + norm(y, p + "norm1b")
        if layer.get("mlp") is not None:
            y = feed_forward(norm(x, p + "norm2"), _sub(w, p + "mlp."), layer["mlp"])
            x = x + norm(y, p + "norm2b")
        if layers_out is not None:
            layers_out.append(x.clone())
    return norm(x, "final.norm") @ w["head"].to(F64).T * cfg["logit_scale"]


# -- making small models ----------------------------------------------------------------

def mixer_shapes(kind: str, m: dict, width: int) -> dict:
    """Tensor names (short) and shapes of one mixer."""
    nh, ng, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    if kind == "attention":
        return {"q": (nh * d, width), "q.b": (nh * d,), "k": (ng * d, width), "k.b": (ng * d,),
                "v": (ng * dv, width), "v.b": (ng * dv,), "q.norm": (nh * d,),
                "k.norm": (ng * d,), "sink": (nh,), "o": (width, nh * dv),
                **({"vmix": ()} if m["v_mix"] else {})}
    s = {"b": (nh, width), "a": (nh, width), "A_log": (nh,), "dt_bias": (nh,), "norm": (dv,),
         "g": (nh * dv, width), "o": (width, nh * dv)}
    for n, rows in (("q", ng * d), ("k", ng * d), ("v", nh * dv)):
        s.update({n: (rows, width), n + ".conv": (rows, m["conv"])})
    return s


def ff_shapes(f: dict, width: int) -> dict:
    one = lambda p, ff: {p + "gate": (ff, width), p + "up": (ff, width), p + "down": (width, ff)}
    if f["kind"] == "dense":
        return one("", f["ff"])
    n = f["router"]["experts"]
    s = {"router": (n, width), "correction": (n,)}
    for e in range(n):
        s.update(one(f"e{e}.", f["expert"]["ff"]))
    if f.get("shared"):
        s.update(one("shared.", f["shared"]["ff"]))
    return s


def norm_shapes(name: str, width: int) -> dict:
    return {name: (width,), name + ".b": (width,), name + ".alpha": ()}


def tensor_shapes(cfg: dict) -> dict:
    width, vocab = cfg["width"], cfg["vocab"]
    shapes = {"embed": (vocab, width), "head": (vocab, width), **norm_shapes("final.norm", width)}
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        names = ["norm1", "norm1b"] + (["norm2", "norm2b"] if layer.get("mlp") else [])
        for n in names:
            shapes.update(norm_shapes(p + n, width))
        for n, s in mixer_shapes(layer["type"], layer["mixer"], width).items():
            shapes[p + "mix." + n] = s
        if layer.get("mlp") is not None:
            for n, s in ff_shapes(layer["mlp"], width).items():
                shapes[p + "mlp." + n] = s
    return shapes


def random_tensor(name: str, shape, g):
    """Values that keep activations O(1) and every branch in use."""
    leaf = name.split(".")[-1]
    randn = torch.randn(shape, generator=g)
    rand = torch.rand(shape, generator=g)
    if leaf == "alpha":
        return 0.4 + 0.5 * rand
    if leaf in ("vmix", "dt_bias"):
        return 0.2 + 0.6 * rand
    if leaf.startswith("norm"):
        return 1.0 + 0.2 * randn
    if leaf == "embed":
        return randn
    if leaf in ("sink", "A_log"):
        return 0.7 * randn
    if leaf == "correction":
        return 0.3 * randn - 0.4        # choice scores of either sign
    if leaf == "b" and len(shape) == 1:
        return 0.3 * randn
    if leaf == "conv":
        t = 0.4 * randn
        t[..., -1] += 0.7
        return t
    if leaf in ("gate", "up", "router"):
        return 2.0 * randn / math.sqrt(shape[-1])
    return randn / math.sqrt(shape[-1])


def random_weights(cfg: dict, seed: int = 0, dtype=torch.bfloat16) -> dict:
    """Rounded to ``dtype`` so that engine and oracle start from the same numbers."""
    g = torch.Generator().manual_seed(seed)
    return {n: random_tensor(n, s, g).to(dtype) for n, s in tensor_shapes(cfg).items()}


def write_model(path: str, cfg: dict, weights: dict) -> None:
    from safetensors.torch import save_file

    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in weights.items()},
              os.path.join(path, "model.safetensors"))
