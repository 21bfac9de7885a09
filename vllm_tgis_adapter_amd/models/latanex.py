"""Latanex: a decoder-only model with an f32 residual stream and a norm without
statistics before and after every sublayer,

    x <- x + N1b(mixer(N1(x))),   x <- x + N2b(ff(N2(x))),
    N(y) = tanh(alpha y) * w + b.

The mixer of a layer is one of

  attention  grouped-query attention over a sliding window, without positions:
             query/key norm over the whole projection, soft-capped scores, a
             learned sink per head; in every layer with ``v_mix`` but the first
             such one the values are mixed with that first layer's values of
             the same token before they are cached
  delta      gated delta rule: short convolutions, a matrix state per head

and the feed-forward is a gated silu MLP, a mixture of small experts with a
clamped gate behind a sigmoid router with expert groups (plus an optional
shared expert), or absent.  The head is the final norm and a linear map times
``logit_scale``.

Sizes and constants all come from config.json:

  vocab, width, norm.eps, embedding.scale, logit_scale,
  layers[i] = {type, mixer{...}, mlp{...} | null}
  attention:  heads, kv_heads, dim, vdim, scale, softcap, mask.size, v_mix
  delta:      heads, kv_heads, dim, vdim, conv
  mlp dense:  ff
  mlp moe:    expert{ff, limit}, router{experts, top, scale, groups{count, keep}},
              shared{ff, limit}

Tensors: embed, head, <norm>{, .alpha, .b} for final.norm and l<i>.{norm1,
norm1b, norm2, norm2b}, l<i>.mix.* (per mixer, see models/blocks.py),
l<i>.mlp.{gate, up, down} or l<i>.mlp.{router, correction, e<j>.*, shared.*}.
"""

from __future__ import annotations

from typing import Optional

import torch
import torch.nn as nn

from .. import ops
from ..engine.config import ModelConfig
from ..engine.metadata import AttnMetadata
from ..parallel import get_tp_world_size
from .blocks import (
    CappedAttention,
    DeltaMixer,
    GatedDenseMLP,
    GatedRoutedExperts,
    StreamTanhNorm,
)

# positions are unbounded in this design; the default bounds block tables and
# capture buffers and can be raised with --max-model-len
_DEFAULT_MAX_LEN = 32768

MIXERS = ("attention", "delta")


def build_mixer(kind: str, m: dict, width: int, eps: float, dtype: torch.dtype,
                mixes_values: bool = False):
    dim = int(m["dim"])
    common = dict(heads=int(m["heads"]), kv_heads=int(m.get("kv_heads", m["heads"])), dim=dim,
                  vdim=int(m.get("vdim", dim)), eps=eps, dtype=dtype)
    if kind == "attention":
        return CappedAttention(
            width, **common, scale=float(m["scale"]), softcap=float(m.get("softcap") or 0.0),
            window=int((m.get("mask") or {}).get("size") or 0), mixes_values=mixes_values)
    if kind == "delta":
        return DeltaMixer(width, **common, taps=int(m["conv"]))
    raise ValueError(f"unknown mixer type {kind!r}")


class SharedAndRouted(nn.Module):
    """Routed experts and, for every token, a shared one.  Returns the two
    results; the caller's residual kernel adds them."""

    def __init__(self, width: int, mlp: dict, dtype: torch.dtype):
        super().__init__()
        r, e = mlp["router"], mlp["expert"]
        g = r.get("groups") or {}
        self.routed = GatedRoutedExperts(
            width, experts=int(r["experts"]), top=int(r["top"]), ff=int(e["ff"]), dtype=dtype,
            correction=True, groups=(int(g.get("count", 1)), int(g.get("keep", 1))),
            renormalise=True, weight_scale=float(r.get("scale", 1.0)), limit=float(e["limit"]))
        s = mlp.get("shared")
        self.shared = None if not s else GatedDenseMLP(width, int(s["ff"]), dtype, act="clamped",
                                                       limit=float(s["limit"]))

    def load(self, t: dict) -> None:
        n = range(self.routed.experts)
        self.routed.load(t["router"], *[[t[f"e{e}.{k}"] for e in n]
                                        for k in ("gate", "up", "down")], t["correction"])
        if self.shared is not None:
            self.shared.load(t["shared.gate"], t["shared.up"], t["shared.down"])

    def forward(self, h: torch.Tensor):
        return self.routed(h), None if self.shared is None else self.shared(h)


def build_ff(mlp: Optional[dict], width: int, dtype: torch.dtype):
    if mlp is None:
        return None
    kind = mlp.get("kind", "dense")
    if kind == "dense":
        return GatedDenseMLP(width, int(mlp["ff"]), dtype, act="silu")
    if kind == "moe":
        return SharedAndRouted(width, mlp, dtype)
    raise ValueError(f"unknown feed-forward kind {kind!r}")


def _ff_size(mlp: dict) -> int:
    if mlp.get("kind", "dense") == "dense":
        return int(mlp["ff"])
    return int(mlp["expert"]["ff"])


def first_value_layer(layers: list) -> Optional[int]:
    """Index of the first layer whose values later layers mix in."""
    for i, e in enumerate(layers):
        if e["type"] == "attention" and e["mixer"].get("v_mix"):
            return i
    return None


def _check_layers(layers: list) -> None:
    first = first_value_layer([e for e in layers if e.get("type") in MIXERS])
    for i, e in enumerate(layers):
        if e.get("type") not in MIXERS:
            raise ValueError(f"layer {i}: unknown mixer type {e.get('type')!r}")
        if e["type"] == "attention" and e["mixer"].get("v_mix"):
            m, f = e["mixer"], layers[first]["mixer"]
            size = lambda a: (int(a.get("kv_heads", a["heads"])), int(a.get("vdim", a["dim"])))
            if size(m) != size(f):
                raise ValueError(f"layer {i}: mixed values must have the first layer's shape")


def model_config_from_json(model: str, hf: dict) -> ModelConfig:
    layers = hf["layers"]
    _check_layers(layers)
    att = [e["mixer"] for e in layers if e["type"] == "attention"]
    return ModelConfig(
        model=model,
        architecture="latanex",
        vocab_size=int(hf["vocab"]),
        hidden_size=int(hf["width"]),
        intermediate_size=max((_ff_size(e["mlp"]) for e in layers if e.get("mlp")), default=0),
        num_layers=len(layers),
        num_heads=max(int(e["mixer"]["heads"]) for e in layers),
        num_kv_heads=max((int(a.get("kv_heads", a["heads"])) for a in att), default=1),
        head_dim=max((int(a["dim"]) for a in att), default=1),
        rope_theta=0.0,
        rms_norm_eps=float((hf.get("norm") or {}).get("eps", 1e-5)),
        max_model_len=int(hf.get("max_len", _DEFAULT_MAX_LEN)),
        tie_word_embeddings=False,
        dtype=torch.bfloat16,
        # num_experts stays 0: that field describes the mixtral expert layout;
        # the routed layers here are shape-static
        hf_config=hf,
    )


def native_extensions(cfg: ModelConfig) -> list[str]:
    """Residual kernels, attention inputs, attention of any shape, the delta
    recurrence, router and gates live in the sequence extension; an attention
    mixer whose shape the matrix-core kernels take needs the attention
    extension too."""
    for e in cfg.hf_config["layers"]:
        if e["type"] != "attention":
            continue
        m = e["mixer"]
        dim = int(m["dim"])
        if ops.capped_attention_uses_matrix_cores(
                cfg.dtype, int(m["heads"]), int(m.get("kv_heads", m["heads"])), dim,
                int(m.get("vdim", dim))):
            return ["_C_seq", "_C_attn"]
    return ["_C_seq"]


class LatanexLayer(nn.Module):
    def __init__(self, entry: dict, width: int, eps: float, dtype: torch.dtype,
                 mixes_values: bool):
        super().__init__()
        self.dtype = dtype
        self.mix = build_mixer(entry["type"], entry["mixer"], width, eps, dtype, mixes_values)
        self.mlp = build_ff(entry.get("mlp"), width, dtype)
        self.norm1 = StreamTanhNorm(width)
        self.norm1b = StreamTanhNorm(width)
        if self.mlp is not None:
            self.norm2 = StreamTanhNorm(width)
            self.norm2b = StreamTanhNorm(width)

    def cache_shapes(self, block_size: int) -> list:
        return self.mix.cache_shapes(block_size)

    def forward(self, x, h, positions, cache, meta, next_norm):
        """x: f32 stream, updated in place; h: N1(x).  Returns ``next_norm`` of
        the updated stream, which the next layer (or the head) reads."""
        add = lambda a, b, norm, nxt: ops.stream_add_tanh_norm(
            x, a, norm.triple(), b=b, next_norm=nxt.triple(), out_dtype=self.dtype)
        y = self.mix(h, positions, cache, meta)
        h = add(y, None, self.norm1b, next_norm if self.mlp is None else self.norm2)
        if self.mlp is None:
            return h
        y = self.mlp(h)
        a, b = y if isinstance(y, tuple) else (y, None)
        return add(a, b, self.norm2b, next_norm)


class LatanexForCausalLM(nn.Module):
    uses_seq_state = True

    def __init__(self, cfg: ModelConfig):
        super().__init__()
        if get_tp_world_size() != 1:
            raise ValueError("Latanex is not sharded yet; run it with tensor_parallel_size 1")
        hf = cfg.hf_config
        _check_layers(hf["layers"])
        self.cfg = cfg
        dtype, width = cfg.dtype, cfg.hidden_size
        self.embed_scale = float((hf.get("embedding") or {}).get("scale", 1.0))
        self.logit_scale = float(hf.get("logit_scale", 1.0))
        self.embed = nn.Parameter(
            torch.empty(cfg.vocab_size, width, dtype=dtype).normal_(0.0, 1.0),
            requires_grad=False)
        self.first_values = first_value_layer(hf["layers"])
        self.layers = nn.ModuleList([
            LatanexLayer(e, width, cfg.rms_norm_eps, dtype,
                         mixes_values=bool(e["type"] == "attention" and e["mixer"].get("v_mix")
                                           and i != self.first_values))
            for i, e in enumerate(hf["layers"])])
        self.final_norm = StreamTanhNorm(width)
        self.head = nn.Parameter(
            torch.empty(cfg.vocab_size, width, dtype=dtype).normal_(0.0, width ** -0.5),
            requires_grad=False)
        # set by the test harness to collect the stream after every layer
        self.stream_probe: Optional[list] = None

    # -- cache layout (asked for by the worker) ----------------------------
    @staticmethod
    def _bytes(shape, dtype) -> int:
        n = 1
        for s in shape:
            n *= s
        return n * torch.tensor([], dtype=dtype).element_size()

    def _cache_bytes(self, kind: str, block_size: int) -> int:
        return sum(self._bytes(shape, dt) for layer in self.layers
                   for k, shape, dt in layer.cache_shapes(block_size) if k == kind)

    def cache_bytes_per_block(self, block_size: int) -> int:
        return max(1, self._cache_bytes("paged", block_size))

    def state_bytes_per_slot(self) -> int:
        return self._cache_bytes("slot", 1)

    def allocate_caches(self, num_blocks: int, block_size: int, num_slots: int,
                        device) -> list:
        """Per layer the tensors it names, paged ones [blocks, ...] and
        per-sequence ones [slots, ...]; a layer that mixes values gets the first
        such layer's value cache behind its own."""
        lead = {"paged": num_blocks, "slot": max(num_slots, 1)}
        out = []
        for layer in self.layers:
            entry = [torch.zeros((lead[kind],) + tuple(shape), dtype=dt, device=device)
                     for kind, shape, dt in layer.cache_shapes(block_size)]
            if isinstance(layer.mix, CappedAttention) and layer.mix.mixes_values:
                entry.append(out[self.first_values][1])
            out.append(tuple(entry))
        return out

    # -- forward -----------------------------------------------------------
    def forward(self, input_ids, positions, kv_caches, meta: AttnMetadata) -> torch.Tensor:
        x = ops.embedding_scaled(input_ids, self.embed, self.embed_scale)      # f32 stream
        nexts = [layer.norm1 for layer in self.layers[1:]] + [self.final_norm]
        h = ops.stream_add_tanh_norm(x, None, None, next_norm=self.layers[0].norm1.triple(),
                                     out_dtype=self.cfg.dtype)
        for layer, cache, nxt in zip(self.layers, kv_caches, nexts):
            h = layer(x, h, positions, cache, meta, nxt)
            if self.stream_probe is not None:
                self.stream_probe.append(x.clone())
        return h

    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        return ops.scale_logits(ops.linear(hidden, self.head), self.logit_scale)

    # -- weights -----------------------------------------------------------
    @staticmethod
    def _sub(weights: dict, prefix: str) -> dict:
        return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}

    def load_weights(self, weights: dict[str, torch.Tensor]) -> None:
        dtype = self.cfg.dtype

        def norm(mod: StreamTanhNorm, name: str) -> None:
            mod.load(weights[name], weights[name + ".alpha"], weights[name + ".b"])

        self.embed.data.copy_(weights["embed"].to(dtype))
        self.head.data.copy_(weights["head"].to(dtype))
        norm(self.final_norm, "final.norm")
        for i, layer in enumerate(self.layers):
            p = f"l{i}."
            for n in ["norm1", "norm1b"] + (["norm2", "norm2b"] if layer.mlp is not None else []):
                norm(getattr(layer, n), p + n)
            layer.mix.load(self._sub(weights, p + "mix."))
            if layer.mlp is None:
                continue
            t = self._sub(weights, p + "mlp.")
            if isinstance(layer.mlp, SharedAndRouted):
                layer.mlp.load(t)
            else:
                layer.mlp.load(t["gate"], t["up"], t["down"])
