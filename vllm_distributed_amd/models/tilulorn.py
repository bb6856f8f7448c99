"""Tilulorn: a decoder-only stack whose layers are listed one by one in the configuration, part of which can run several
times in a row with the same weights.  A pre-norm layer, x <- x + mixer(N1 x), then x <- x + ff(N2 x) (some layers have no
feed-forward), over an fp32 residual; N is an RMS norm.  Before each pass of the loop the residual is replaced by a
product of itself and the embedding output, plus a learned row per pass: x <- W_in [x; e] + step[pass].  Mixers:

  ``latent_attention``  queries through a normed latent, keys and values up-projected from one normed latent per token plus
                        a rotated key part all heads share (half-split pairs, YaRN frequencies), causal, one sigmoid
                        output gate per head;
  ``attention``         grouped-query attention inside a sliding window; the values are the projected keys before norm
                        and rotation; norms over the whole q and k projections, rotated neighbouring pairs with linear
                        frequency scaling, a sink per head, one sigmoid output gate per head;
  ``wkv``               RWKV-style time mixing.

Feed-forward: gated SiLU experts that a table per layer assigns to token ids, equally weighted.

The mixers are ``layers/latent_attention.py::WindowedLatentAttention``, ``layers/masked_attention.py::
MaskedSoftmaxAttention`` and ``layers/wkv.py::WKVMixer``, the experts ``layers/moe.py::FusedMoE`` behind
``TokenExpertTables``; attention keeps pages of the paged cache, recurrent mixers a state slot per request, both one per
pass of the loop.  The scheduler, chunked prefill, batching and sampling are the common ones.

Configuration (``config.json``): ``architecture: "Tilulorn"``, ``vocab``, ``width``, ``norm.eps``, ``layers`` (``type``,
``mixer`` sizes and constants, ``mlp`` or null), optional ``loop`` (``start``, ``stop``, ``times``).  The rank of a wkv
layer's decay projection is the row count of ``l<i>.mix.w1``.
Checkpoint names: ``embed``, ``head``, ``final.norm``, ``loop.in``, ``loop.step``, ``l<i>.norm1|norm2``, ``l<i>.mix.*``,
``l<i>.mlp.table``, ``l<i>.mlp.e<j>.gate|up|down``.
"""
from __future__ import annotations

import math
import os
import re
from typing import Iterable, Optional

import torch
import torch.nn as nn

from .. import ops
from ..config import VllmConfig
from ..layers.basic import LogitsProcessor, ParallelLMHead, VocabParallelEmbedding
from ..layers.hyper_connections import _fp32_param
from ..layers.latent_attention import WindowedLatentAttention
from ..layers.linear import ReplicatedLinear, default_weight_loader
from ..layers.masked_attention import MaskedSoftmaxAttention
from ..layers.moe import FusedMoE, TokenExpertTables
from ..layers.wkv import MIXES, WKVMixer
from .rapovik import run_order

ARCHITECTURE = "TilulornForCausalLM"
MIXERS = ("latent_attention", "attention", "wkv")
DEFAULT_CONTEXT = 131072


def is_tilulorn_config(d: dict) -> bool:
    return d.get("architecture") == "Tilulorn" or ARCHITECTURE in (d.get("architectures") or [])


def normalise_config(d: dict, model_dir: Optional[str] = None) -> dict:
    """Give the engine the names it reads (hidden_size, vocab_size, heads ...) and complete the mixers' sizes with what
    only a tensor's shape tells (the rank of the decay projections)."""
    d = dict(d)
    layers = [dict(l, mixer=dict(l["mixer"])) for l in d["layers"]]
    shapes = {}
    st = os.path.join(model_dir, "model.safetensors") if model_dir else None
    if st and os.path.isfile(st):
        from .loader import read_safetensors_header
        header, _ = read_safetensors_header(st)
        shapes = {k: v["shape"] for k, v in header.items() if k != "__metadata__"}
    for i, l in enumerate(layers):
        if l["type"] not in MIXERS:
            raise ValueError(f"layer {i}: unknown mixer type {l['type']!r}")
        if l.get("mlp") is not None and l["mlp"].get("kind", "moe") != "moe":
            raise ValueError(f"layer {i}: unknown feed-forward kind {l['mlp'].get('kind')!r}")
        if l["type"] == "wkv":
            name = f"l{i}.mix.w1"
            if name in shapes:
                l["mixer"]["decay_rank"] = int(shapes[name][0])
            elif "decay_rank" not in l["mixer"]:
                raise ValueError(f"layer {i}: the rank of the decay projection is neither in the configuration "
                                 f"(decay_rank) nor readable from the shape of {name}")
    att = [l["mixer"] for l in layers if l["type"] == "attention"]
    lat = [l["mixer"] for l in layers if l["type"] == "latent_attention"]
    d.update(
        layers=layers, architectures=[ARCHITECTURE], model_type="tilulorn", hidden_size=int(d["width"]),
        vocab_size=int(d["vocab"]), num_hidden_layers=len(layers),
        num_attention_heads=max((int(m["heads"]) for m in att + lat), default=1),
        num_key_value_heads=max((int(m["kv_heads"]) for m in att), default=1),
        head_dim=max([int(m["dim"]) for m in att] + [int(m["kv_rank"]) + int(m["rot_dim"]) for m in lat],
                     default=int(d["width"])),
        tie_word_embeddings=False)
    d.setdefault("max_position_embeddings", DEFAULT_CONTEXT)
    d.setdefault("torch_dtype", "bfloat16")
    return d


class PlainGain(nn.Module):
    """The weight of an RMS norm (fp32); applied by ``ops.gated_residual_group_norm``."""

    def __init__(self, width: int):
        super().__init__()
        self.weight = _fp32_param((width,), 1.0)


def linear_scaling(rot: dict) -> Optional[dict]:
    sc = rot.get("scaling")
    return dict(kind="linear", factor=float(sc["factor"])) if sc else None


def yarn_scaling(rot: dict) -> Optional[dict]:
    sc = rot.get("scaling")
    if not sc:
        return None
    return dict(kind="yarn", factor=float(sc["factor"]), original=float(sc["original"]), fast=float(sc["fast"]),
                slow=float(sc["slow"]), magnitude=0.1 * math.log(float(sc["factor"])) + 1.0)


def make_mixer(kind: str, m: dict, width: int, eps: float, passes: int, quant_config, prefix: str) -> nn.Module:
    rot = m.get("rot") or {}
    if kind == "latent_attention":
        return WindowedLatentAttention(
            width, int(m["heads"]), int(m["dim"]), int(m["rot_dim"]), int(m["vdim"]), int(m["kv_rank"]),
            float(m["scale"]), None, rot.get("base"), int(rot.get("dims", m["rot_dim"]) or 0), eps, passes, quant_config,
            prefix, q_rank=int(m["q_rank"]), gate="head", rot_pairing="halves", rot_scaling=yarn_scaling(rot))
    if kind == "attention":
        return MaskedSoftmaxAttention(
            width, int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"]), float(m["scale"]), eps,
            window=int((m.get("mask") or {}).get("size", 0) or 0), sink=True, gate="head", norm_over="projection",
            key_values=True, rot_dims=int(rot.get("dims", 0) or 0), rot_base=float(rot.get("base", 10000.0)),
            rot_pairing="neighbours", rot_scaling=linear_scaling(rot), users=passes, quant_config=quant_config,
            prefix=prefix)
    mixer = WKVMixer(width, int(m["heads"]), int(m["dim"]), int(m["decay_rank"]), eps, quant_config, prefix)
    mixer.add_passes(passes)
    return mixer


class TilulornLayer(nn.Module):
    def __init__(self, spec: dict, width: int, eps: float, passes: int, quant_config, prefix: str):
        super().__init__()
        self.kind, self.eps = spec["type"], eps
        self.norm1 = PlainGain(width)
        self.mixer = make_mixer(self.kind, spec["mixer"], width, eps, passes, quant_config, f"{prefix}.mixer")
        mlp = spec.get("mlp")
        self.has_mlp = mlp is not None
        if self.has_mlp:
            self.norm2 = PlainGain(width)
            self.experts = FusedMoE(int(mlp["router"]["experts"]), int(mlp["router"]["top"]), width,
                                    int(mlp["expert"]["ff"]), renormalize=False, quant_config=quant_config,
                                    prefix=f"{prefix}.experts")

    def forward(self, x: torch.Tensor, h: torch.Tensor, positions: torch.Tensor, pass_index: int, routed,
                nxt: Optional[PlainGain], cast_to: Optional[torch.Tensor]) -> Optional[torch.Tensor]:
        """``x``: the fp32 residual, updated in place; ``h``: this layer's normed input; ``routed``: the tokens' experts and
        weights.  Returns the next layer's input under norm ``nxt``, or, without one, the residual itself in ``cast_to``."""
        if self.kind == "wkv":
            self.mixer.select_pass(pass_index)
            y = self.mixer(h)
        else:
            y = self.mixer(h, positions, pass_index)
        if self.has_mlp:
            h = ops.gated_residual_group_norm(x, [(y, None, None, None, None)], self.norm2.weight, 1, self.eps, h.dtype)
            y = self.experts(h, None, routed=routed)
        return ops.gated_residual_group_norm(x, [(y, None, None, None, None)], nxt.weight if nxt is not None else None, 1,
                                             self.eps, y.dtype, cast_to=cast_to)


class TilulornForCausalLM(nn.Module):
    supports_pp = False
    supports_lora = False
    # recurrent states live in per-row slots even when no layer is an attention layer
    row_state_slots = True
    # kernels outside the common set that this model launches (ops/build.py builds them on first use)
    native_sources = ("masked_attention.hip", "attention.hip", "attention_prefill.hip", "latent_attention.hip", "mla.hip",
                      "linear_attention.hip", "token_shift.hip", "moe.hip", "gemm_tile.hip")

    def __init__(self, vllm_config: VllmConfig, prefix: str = ""):
        super().__init__()
        config = vllm_config.model_config.hf_config
        self.config = config
        quant_config = getattr(vllm_config, "quant_config", None)
        width, vocab, self.eps = int(config.width), int(config.vocab), float(config.norm["eps"])
        self.width = width
        loop = config.get("loop")
        self.runs = run_order(len(config.layers), loop)
        passes = [0] * len(config.layers)
        for i, p in self.runs:
            passes[i] = max(passes[i], p + 1)
        first = int(loop["start"]) if loop and int(loop["stop"]) > int(loop["start"]) else None
        # the pass that a run opens, or None
        self.opens = [p if i == first else None for i, p in self.runs]
        self.embed_tokens = VocabParallelEmbedding(vocab, width)
        if loop:
            self.loop_in = ReplicatedLinear(2 * width, width, bias=False, prefix="loop_in")
            self.loop_step = _fp32_param((int(loop["times"]), width), 0.0)
        self.layers = nn.ModuleList([
            TilulornLayer(spec, width, self.eps, max(passes[i], 1), quant_config, f"layers.{i}")
            for i, spec in enumerate(config.layers)])
        # routed layers in order; a layer's place among them
        routers = [(i, l["mlp"]["router"]) for i, l in enumerate(config.layers) if l.get("mlp") is not None]
        self.routed_place = {i: n for n, (i, _) in enumerate(routers)}
        self.expert_tables = TokenExpertTables(vocab, [r["top"] for _, r in routers], [r["experts"] for _, r in routers]) \
            if routers else None
        self.norm = PlainGain(width)
        self.lm_head = ParallelLMHead(vocab, width)
        self.logits_processor = LogitsProcessor(vocab)

    def get_input_embeddings(self, input_ids):
        return self.embed_tokens(input_ids)

    def forward(self, input_ids, positions, intermediate_tensors=None, inputs_embeds=None):
        dtype, W = self.embed_tokens.weight.dtype, self.width
        e = (inputs_embeds if inputs_embeds is not None else self.embed_tokens(input_ids)).to(dtype)
        routed = self.expert_tables(input_ids) if self.expert_tables is not None else None
        both = None
        if any(p is not None for p in self.opens):        # [residual | embedding output] in front of a pass
            both = torch.empty((e.shape[0], 2 * W), dtype=dtype, device=e.device)
            both[:, W:] = e
        if self.opens and self.opens[0] is not None:
            both[:, :W] = e
            x = h = None
        else:
            x = e.float() if dtype != torch.float32 else e.clone()
            first = self.layers[self.runs[0][0]].norm1 if self.runs else self.norm
            h = ops.gated_residual_group_norm(x, [], first.weight, 1, self.eps, dtype)
        for r, (i, p) in enumerate(self.runs):
            layer = self.layers[i]
            if self.opens[r] is not None:
                x = ops.linear_f32(both, self.loop_in.weight)
                h = ops.gated_residual_group_norm(x, [], layer.norm1.weight, 1, self.eps, dtype,
                                                  step=self.loop_step[self.opens[r]])
            last = r + 1 == len(self.runs)
            leaves = not last and self.opens[r + 1] is not None
            nxt = None if leaves else self.norm if last else self.layers[self.runs[r + 1][0]].norm1
            h = layer(x, h, positions, p, routed[self.routed_place[i]] if layer.has_mlp else None, nxt,
                      both[:, :W] if leaves else None)
        return h

    def compute_logits(self, hidden_states):
        return self.logits_processor(self.lm_head, hidden_states).float()

    # checkpoint name -> (parameter name, shard id)
    _MIX = {
        "latent_attention": {"dq": ("down_proj.weight", 0), "dkv": ("down_proj.weight", 1), "g": ("down_proj.weight", 2),
                             "dq.norm": ("q_norm", None), "uq": ("uq_proj.weight", None), "dkv.norm": ("c_norm", None),
                             "uk": ("uk_proj.weight", None), "uv": ("uv_proj.weight", None),
                             "o": ("o_proj.weight", None)},
        "attention": {"q": ("in_proj.weight", 0), "k": ("in_proj.weight", 1), "g": ("in_proj.weight", 2),
                      "q.norm": ("q_norm", None), "k.norm": ("k_norm", None), "sink": ("sink", None),
                      "o": ("o_proj.weight", None)},
        "wkv": {**{s: ("in_weight", i) for i, s in enumerate(MIXES[:4])},
                **{f"mu.{s}": ("mu", i) for i, s in enumerate(MIXES)},
                "w1": ("decay_down", None), "w2": ("decay_up", None), "w0": ("decay_bias", None), "u": ("bonus", None),
                "norm": ("norm_weight", None), "o": ("o_proj.weight", None)},
    }
    _EXPERT = {"gate": ("w13_weight", "w1"), "up": ("w13_weight", "w3"), "down": ("w2_weight", "w2")}
    _TOP = {"embed": "embed_tokens.weight", "head": "lm_head.weight", "final.norm": "norm.weight",
            "loop.in": "loop_in.weight", "loop.step": "loop_step"}

    def _target(self, name: str):
        """Returns (parameter name, shard id, expert id) or None."""
        if name in self._TOP:
            return self._TOP[name], None, None
        m = re.fullmatch(r"l(\d+)\.(.+)", name)
        if not m or int(m.group(1)) >= len(self.layers):
            return None
        i, rest = int(m.group(1)), m.group(2)
        layer, base = self.layers[i], f"layers.{i}."
        if rest in ("norm1", "norm2"):
            return f"{base}{rest}.weight", None, None
        part, _, leaf = rest.partition(".")
        if part == "mix" and leaf in self._MIX[layer.kind]:
            t, shard = self._MIX[layer.kind][leaf]
            return f"{base}mixer.{t}", shard, None
        if part == "mlp" and layer.has_mlp:
            if leaf == "table":
                return "expert_tables.table", self.routed_place[i], None
            m = re.fullmatch(r"e(\d+)\.(gate|up|down)", leaf)
            if m and int(m.group(1)) < layer.experts.global_num_experts:
                t, shard = self._EXPERT[m.group(2)]
                return f"{base}experts.{t}", shard, int(m.group(1))
        return None

    def load_weights(self, weights: Iterable[tuple[str, torch.Tensor]]) -> set[str]:
        params = dict(self.named_parameters())
        loaded: set[str] = set()
        for name, t in weights:
            tgt = self._target(name)
            if tgt is None or tgt[0] not in params:
                raise ValueError(f"checkpoint tensor {name!r} has no place in this model")
            target, shard, expert = tgt
            p = params[target]
            loader = getattr(p, "weight_loader", default_weight_loader)
            if expert is not None:
                loader(p, t, shard, expert)
            elif shard is None:
                loader(p, t)
            else:
                loader(p, t, shard)
            loaded.add(target)
        return loaded
