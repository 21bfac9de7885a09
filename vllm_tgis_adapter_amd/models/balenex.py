"""Balenex: a decoder-only model with an f32 residual stream and a norm before
and after every sublayer,

    x <- x + N1b(mixer(N1(x))),   x <- x + N2b(ff(N2(x))),

each N an RMS norm of ``norm.groups`` equal parts of the row with a plain
weight.  The mixer of a layer is one of

  parallel   two mixers fed the same normed input, half the sum of their
             RMS-normed outputs: windowed attention that also keeps the first
             tokens of the sequence (short convolutions and query/key norms
             ahead of a rotation; values are rotated too and the output turned
             back), and gated linear attention with a matrix state per head
  attention  windowed attention without positions in which everything before
             the window is seen through mean-pooled blocks of keys and values

and the feed-forward is a gated silu MLP with biases, or absent.  The head is
the final norm and a linear map.

Sizes and constants all come from config.json:

  vocab, width, norm{eps, groups}, layers[i] = {type, mixer{...}, mlp{...} | null}
  parallel.left:   heads, kv_heads, dim, vdim, scale, conv, mask{size, keep_first},
                   rot{base, dims}
  parallel.right:  heads, dim, vdim, tau (the rank of the decay's inner
                   projection is the row count of the tensor a1)
  attention:       heads, kv_heads, dim, vdim, scale, mask{size, pool}
  mlp:             kind "dense", ff

Tensors: embed, final.norm, head, l<i>.{norm1, norm1b, norm2, norm2b},
l<i>.mix.* (per mixer, see models/blocks.py), l<i>.mlp.{gate, up, down} with .b.
"""

from __future__ import annotations

from typing import Optional

import torch
import torch.nn as nn

from .. import ops
from ..engine.config import ModelConfig
from ..engine.metadata import AttnMetadata
from ..parallel import get_tp_world_size
from .blocks import BiasedGatedMLP, GLAMixer, ParallelMixer, SpanAttention, _f32_param

# positions are unbounded in this design; the default bounds block tables and
# capture buffers and can be raised with --max-model-len
_DEFAULT_MAX_LEN = 32768
# decay rank of models made without weights
_DEFAULT_RANK = 16

MIXERS = ("parallel", "attention")


def _span_attention(m: dict, width: int, eps: float, parallel: bool, dtype: torch.dtype):
    dim = int(m["dim"])
    mask = m.get("mask") or {}
    common = dict(heads=int(m["heads"]), kv_heads=int(m.get("kv_heads", m["heads"])), dim=dim,
                  vdim=int(m.get("vdim", dim)), scale=float(m["scale"]), eps=eps,
                  window=int(mask.get("size") or 0), dtype=dtype)
    if parallel:
        rot = m.get("rot") or {}
        return SpanAttention(
            width, **common, keep_first=int(mask.get("keep_first") or 0),
            taps=int(m.get("conv") or 0), norm_weights=True,
            rot_base=float(rot.get("base", 10000.0)), rot_dims=int(rot.get("dims", 0)),
            rotate_values=True, own_in=False)
    return SpanAttention(width, **common, pool=int(mask.get("pool") or 0), norm_weights=False,
                         o_bias=True)


def build_mixer(kind: str, m: dict, width: int, eps: float, dtype: torch.dtype):
    if kind == "parallel":
        r = m["right"]
        right = GLAMixer(width, heads=int(r["heads"]), dim=int(r["dim"]), vdim=int(r["vdim"]),
                         rank=int(r.get("rank", _DEFAULT_RANK)), tau=float(r["tau"]), eps=eps,
                         own_in=False, dtype=dtype)
        left = _span_attention(m["left"], width, eps, True, dtype)
        # whole 128-row tiles for the bf16 products once they cost little
        rows = left.in_rows + right.in_rows
        return ParallelMixer(width, left, right, 0.5, 0.5, dtype, out_norms=True,
                             row_multiple=128 if rows >= 4096 else 8)
    if kind == "attention":
        return _span_attention(m, width, eps, False, dtype)
    raise ValueError(f"unknown mixer type {kind!r}")


def build_ff(mlp: Optional[dict], width: int, dtype: torch.dtype):
    if mlp is None:
        return None
    if mlp.get("kind", "dense") != "dense":
        raise ValueError(f"unknown feed-forward kind {mlp.get('kind')!r}")
    return BiasedGatedMLP(width, int(mlp["ff"]), dtype)


def _attention_specs(layers: list) -> list:
    return [e["mixer"]["left"] if e["type"] == "parallel" else e["mixer"] for e in layers]


def model_config_from_json(model: str, hf: dict) -> ModelConfig:
    from ..engine.weights import safetensors_shapes

    layers = [dict(e) for e in hf["layers"]]
    shapes = safetensors_shapes(model)
    for i, e in enumerate(layers):
        if e.get("type") not in MIXERS:
            raise ValueError(f"layer {i}: unknown mixer type {e.get('type')!r}")
        a1 = shapes.get(f"l{i}.mix.right.a1")
        if e["type"] == "parallel" and a1 is not None:
            e["mixer"] = dict(e["mixer"], right=dict(e["mixer"]["right"], rank=a1[0]))
    hf = dict(hf, layers=layers)
    att = _attention_specs(layers)
    norm = hf.get("norm") or {}
    if int(hf["width"]) % int(norm.get("groups", 1)):
        raise ValueError("norm.groups must divide the width")
    return ModelConfig(
        model=model,
        architecture="balenex",
        vocab_size=int(hf["vocab"]),
        hidden_size=int(hf["width"]),
        intermediate_size=max((int(e["mlp"]["ff"]) for e in layers if e.get("mlp")), default=0),
        num_layers=len(layers),
        num_heads=max(int(a["heads"]) for a in att),
        num_kv_heads=max(int(a.get("kv_heads", a["heads"])) for a in att),
        head_dim=max(int(a["dim"]) for a in att),
        rope_theta=0.0,
        rms_norm_eps=float(norm.get("eps", 1e-5)),
        max_model_len=int(hf.get("max_len", _DEFAULT_MAX_LEN)),
        tie_word_embeddings=False,
        dtype=torch.bfloat16,
        hf_config=hf,
    )


def native_extensions(cfg: ModelConfig) -> list[str]:
    """Stream ops, attention inputs, attention of any shape and the recurrence
    live in the sequence extension; an attention mixer whose shape the
    matrix-core kernels take needs the attention extension too."""
    for a in _attention_specs(cfg.hf_config["layers"]):
        dim = int(a["dim"])
        if ops.span_attention_uses_matrix_cores(
                cfg.dtype, int(a["heads"]), int(a.get("kv_heads", a["heads"])), dim,
                int(a.get("vdim", dim))):
            return ["_C_seq", "_C_attn"]
    return ["_C_seq"]


class BalenexLayer(nn.Module):
    def __init__(self, entry: dict, width: int, groups: int, eps: float, dtype: torch.dtype):
        super().__init__()
        self.groups, self.eps, self.dtype = groups, eps, dtype
        self.mix = build_mixer(entry["type"], entry["mixer"], width, eps, dtype)
        self.mlp = build_ff(entry.get("mlp"), width, dtype)
        self.norm1 = _f32_param(width, fill=1.0)
        self.norm1b = _f32_param(width, fill=1.0)
        if self.mlp is not None:
            self.norm2 = _f32_param(width, fill=1.0)
            self.norm2b = _f32_param(width, fill=1.0)

    def cache_shapes(self, block_size: int) -> list:
        return self.mix.cache_shapes(block_size)

    def _add(self, x, y, w_out, next_w, **kw):
        return ops.stream_add_group_norm(x, y, w_out, self.groups, self.eps, next_w=next_w,
                                         out_dtype=self.dtype, **kw)

    def forward(self, x, h, positions, cache, meta, next_w):
        """x: f32 stream, updated in place; h: N1(x).  Returns the norm with
        weight ``next_w`` of the updated stream, which the next layer (or the
        head) reads."""
        after_mix = self.norm2 if self.mlp is not None else next_w
        if isinstance(self.mix, ParallelMixer):
            a, b = self.mix(h, positions, cache, meta)
            h = self._add(x, a, self.norm1b, after_mix, b=b, wa=self.mix.left_norm,
                          wb=self.mix.right_norm, mix=self.mix.left_scale)
        else:
            y = self.mix(h, positions, cache, meta)
            h = self._add(x, y, self.norm1b, after_mix, a_bias=self.mix.o_bias)
        if self.mlp is None:
            return h
        return self._add(x, self.mlp(h), self.norm2b, next_w, a_bias=self.mlp.down_bias)


class BalenexForCausalLM(nn.Module):
    uses_seq_state = True

    def __init__(self, cfg: ModelConfig):
        super().__init__()
        if get_tp_world_size() != 1:
            raise ValueError("Balenex is not sharded yet; run it with tensor_parallel_size 1")
        hf = cfg.hf_config
        self.cfg = cfg
        dtype, width = cfg.dtype, cfg.hidden_size
        self.eps = cfg.rms_norm_eps
        self.groups = int((hf.get("norm") or {}).get("groups", 1))
        self.embed = nn.Parameter(
            torch.empty(cfg.vocab_size, width, dtype=dtype).normal_(0.0, 1.0),
            requires_grad=False)
        self.layers = nn.ModuleList([
            BalenexLayer(e, width, self.groups, self.eps, dtype) for e in hf["layers"]])
        self.final_norm = _f32_param(width, fill=1.0)
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
        per-sequence ones [slots, ...]."""
        lead = {"paged": num_blocks, "slot": max(num_slots, 1)}
        return [tuple(torch.zeros((lead[kind],) + tuple(shape), dtype=dt, device=device)
                      for kind, shape, dt in layer.cache_shapes(block_size))
                for layer in self.layers]

    # -- forward -----------------------------------------------------------
    def forward(self, input_ids, positions, kv_caches, meta: AttnMetadata) -> torch.Tensor:
        x = ops.embedding_scaled(input_ids, self.embed, 1.0)           # f32 stream
        nexts = [layer.norm1 for layer in self.layers[1:]] + [self.final_norm]
        h = ops.stream_add_group_norm(x, None, None, self.groups, self.eps,
                                      next_w=self.layers[0].norm1, out_dtype=self.cfg.dtype)
        for layer, cache, next_w in zip(self.layers, kv_caches, nexts):
            h = layer(x, h, positions, cache, meta, next_w)
            if self.stream_probe is not None:
                self.stream_probe.append(x.clone())
        return h

    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        return ops.linear(hidden, self.head).float()

    # -- weights -----------------------------------------------------------
    @staticmethod
    def _sub(weights: dict, prefix: str) -> dict:
        return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}

    def load_weights(self, weights: dict[str, torch.Tensor]) -> None:
        dtype = self.cfg.dtype
        self.embed.data.copy_(weights["embed"].to(dtype))
        self.head.data.copy_(weights["head"].to(dtype))
        self.final_norm.data.copy_(weights["final.norm"].float())
        for i, layer in enumerate(self.layers):
            p = f"l{i}."
            norms = ["norm1", "norm1b"] + (["norm2", "norm2b"] if layer.mlp is not None else [])
            for n in norms:
                getattr(layer, n).data.copy_(weights[p + n].float())
            t = self._sub(weights, p + "mix.")
            if isinstance(layer.mix, ParallelMixer):
                layer.mix.load(self._sub(t, "left."), self._sub(t, "right."))
            else:
                layer.mix.load(t)
            if layer.mlp is not None:
                layer.mlp.load(self._sub(weights, p + "mlp."))
