"""Surodra: a decoder-only stack whose layers are listed one by one in the configuration, part of which can run several
times in a row with the same weights.  A pre-norm layer, x <- x + m mixer(N1 x), then x <- x + m ff(N2 x) (some layers
have no feed-forward), over an fp32 residual; N is a squashing norm without statistics (Dynamic Tanh), tanh(alpha x) w + b.
Before each pass of the loop a learned row joins the residual, before each pass but the first the embedding output as
well.  Mixers:

  ``delta``      gated delta rule with one decay per head, short convolutions on q, k and v, a SiLU gate behind the
                 heads' norm;
  ``parallel``   two mixers side by side over the same input, each output RMS-normed over the width, half their sum:
                 grouped-query softmax attention (norms over the whole q and k projections, part-rotated heads with linear
                 frequency scaling, a sink per head, one sigmoid output gate per head) and gated linear attention (a decay
                 per key channel through a low-rank projection);
  ``retention``  linear attention with a fixed decay per head, rotated q and k, a SiLU gate behind the heads' norm.

Feed-forward: dense, gated by the tanh form of GELU.  Logits are scaled, then squashed by cap * tanh(logits / cap).

The mixers are ``layers/delta_rule.py::GatedDeltaRule``, ``layers/masked_attention.py::MaskedSoftmaxAttention`` and
``layers/linear_attention.py::DecayedLinearAttention``; attention keeps pages of the paged cache, recurrent mixers a state
slot per request, both one per pass of the loop.  The scheduler, chunked prefill, batching and sampling are the common ones.

Configuration (``config.json``): ``architecture: "Surodra"``, ``vocab``, ``width``, ``norm.eps``, ``residual_mult``,
``logit_scale``, ``logit_softcap``, ``layers`` (``type``, ``mixer`` sizes and constants, ``mlp`` or null), optional
``loop`` (``start``, ``stop``, ``times``).  The rank of the decay projection is the row count of ``l<i>.mix.right.a1``.
Checkpoint names: ``embed``, ``head``, ``final.norm[.b|.alpha]``, ``loop.step``, ``l<i>.norm1|norm2[.b|.alpha]``,
``l<i>.mix.*`` (parallel: ``l<i>.mix.left|right.*``), ``l<i>.mlp.gate|up|down``.
"""
from __future__ import annotations

import os
import re
from typing import Iterable, Optional

import torch
import torch.nn as nn

from .. import ops
from ..config import VllmConfig
from ..layers.basic import LogitsProcessor, ParallelLMHead, VocabParallelEmbedding
from ..layers.delta_rule import GatedDeltaRule
from ..layers.hyper_connections import _fp32_param
from ..layers.linear import default_weight_loader
from ..layers.linear_attention import DecayedLinearAttention
from ..layers.masked_attention import MaskedSoftmaxAttention
from .llama import LlamaMLP
from .rapovik import run_order

ARCHITECTURE = "SurodraForCausalLM"
MIXERS = ("delta", "parallel", "retention")
DEFAULT_CONTEXT = 131072


def is_surodra_config(d: dict) -> bool:
    return d.get("architecture") == "Surodra" or ARCHITECTURE in (d.get("architectures") or [])


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
        if l.get("mlp") is not None and l["mlp"].get("kind", "dense") != "dense":
            raise ValueError(f"layer {i}: unknown feed-forward kind {l['mlp'].get('kind')!r}")
        if l["type"] == "parallel":
            right = l["mixer"]["right"] = dict(l["mixer"]["right"])
            name = f"l{i}.mix.right.a1"
            if name in shapes:
                right["decay_rank"] = int(shapes[name][0])
            elif "decay_rank" not in right:
                raise ValueError(f"layer {i}: the rank of the decay projection is neither in the configuration "
                                 f"(decay_rank) nor readable from the shape of {name}")
    att = [l["mixer"]["left"] for l in layers if l["type"] == "parallel"]
    d.update(
        layers=layers, architectures=[ARCHITECTURE], model_type="surodra", hidden_size=int(d["width"]),
        vocab_size=int(d["vocab"]), num_hidden_layers=len(layers),
        num_attention_heads=max((int(m["heads"]) for m in att), default=1),
        num_key_value_heads=max((int(m["kv_heads"]) for m in att), default=1),
        head_dim=max((max(int(m["dim"]), int(m["vdim"])) for m in att), default=int(d["width"])),
        tie_word_embeddings=False)
    d.setdefault("max_position_embeddings", DEFAULT_CONTEXT)
    d.setdefault("torch_dtype", "bfloat16")
    return d


def rotation(m: dict) -> dict:
    """Rotation options of a mixer's ``rot`` entry."""
    rot = m.get("rot") or {}
    sc = rot.get("scaling")
    return dict(rot_dims=int(rot.get("dims", 0) or 0), rot_base=float(rot.get("base", 10000.0)),
                rot_scaling=dict(kind="linear", factor=float(sc["factor"])) if sc else None)


class SquashNorm(nn.Module):
    """The tensors of a Dynamic Tanh norm (fp32); applied by ``ops.residual_squash_norm``."""

    def __init__(self, width: int):
        super().__init__()
        self.weight = _fp32_param((width,), 1.0)
        self.bias = _fp32_param((width,), 0.0)
        self.alpha = _fp32_param((1,), 1.0)


class RecurrentMixer(nn.Module):
    """One recurrent mixer, a state per pass."""

    def __init__(self, core: nn.Module, passes: int):
        super().__init__()
        self.core = core
        core.add_passes(passes)
        self.share = 1.0

    def forward(self, h: torch.Tensor, positions: torch.Tensor, pass_index: int) -> list:
        self.core.select_pass(pass_index)
        y = self.core(h, positions) if isinstance(self.core, DecayedLinearAttention) else self.core(h)
        return [(y, None)]


class ParallelMixer(nn.Module):
    """Softmax attention and gated linear attention over the same input; each output is RMS-normed over the width and
    counts half (by the caller's residual pass)."""

    def __init__(self, left: MaskedSoftmaxAttention, right: DecayedLinearAttention, width: int, passes: int):
        super().__init__()
        self.left, self.right = left, right
        right.add_passes(passes)
        self.left_out, self.right_out = _fp32_param((width,)), _fp32_param((width,))
        self.share = 0.5

    def forward(self, h: torch.Tensor, positions: torch.Tensor, pass_index: int) -> list:
        a = self.left(h, positions, pass_index)
        self.right.select_pass(pass_index)
        return [(a, self.left_out), (self.right(h, positions), self.right_out)]


def make_mixer(kind: str, m: dict, width: int, eps: float, passes: int, quant_config, prefix: str) -> nn.Module:
    if kind == "delta":
        return RecurrentMixer(GatedDeltaRule(width, int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"]),
                                             int(m["conv"]), None, None, eps, quant_config, f"{prefix}.core"), passes)
    if kind == "retention":
        return RecurrentMixer(DecayedLinearAttention(
            width, int(m["heads"]), int(m["dim"]), int(m["vdim"]), eps, decay=[float(x) for x in m["decay"]],
            k_scale=int(m["dim"]) ** -0.5, quant_config=quant_config, prefix=f"{prefix}.core", **rotation(m)), passes)
    a, b = m["left"], m["right"]
    left = MaskedSoftmaxAttention(
        width, int(a["heads"]), int(a["kv_heads"]), int(a["dim"]), int(a["vdim"]), float(a["scale"]), eps, sink=True,
        gate="head", norm_over="projection", users=passes, quant_config=quant_config, prefix=f"{prefix}.left",
        **rotation(a))
    right = DecayedLinearAttention(
        width, int(b["heads"]), int(b["dim"]), int(b["vdim"]), eps, decay_rank=int(b["decay_rank"]),
        tau=float(b["tau"]), out_norm=True, q_scale=int(b["dim"]) ** -0.5, quant_config=quant_config,
        prefix=f"{prefix}.right")
    return ParallelMixer(left, right, width, passes)


class SurodraLayer(nn.Module):
    def __init__(self, spec: dict, width: int, eps: float, mult: float, passes: int, quant_config, prefix: str):
        super().__init__()
        self.kind, self.eps, self.mult = spec["type"], eps, mult
        self.norm1 = SquashNorm(width)
        self.mixer = make_mixer(self.kind, spec["mixer"], width, eps, passes, quant_config, f"{prefix}.mixer")
        mlp = spec.get("mlp")
        self.has_mlp = mlp is not None
        if self.has_mlp:
            self.norm2 = SquashNorm(width)
            self.mlp = LlamaMLP(width, int(mlp["ff"]), False, quant_config, f"{prefix}.mlp", act="gelu_tanh")

    def forward(self, x: torch.Tensor, h: torch.Tensor, positions: torch.Tensor, pass_index: int, nxt: SquashNorm,
                extra: Optional[torch.Tensor], step: Optional[torch.Tensor]) -> torch.Tensor:
        """``x``: the fp32 residual, updated in place; ``h``: this layer's normed input; ``extra`` and ``step`` join the
        residual behind the layer; returns the next layer's input, under norm ``nxt``."""
        branches = self.mixer(h, positions, pass_index)
        coef = self.mult * self.mixer.share
        if self.has_mlp:
            n = self.norm2
            h = ops.residual_squash_norm(x, branches, coef, self.eps, n.alpha, n.weight, n.bias, h.dtype)
            branches, coef = [(self.mlp(h), None)], self.mult
        return ops.residual_squash_norm(x, branches, coef, self.eps, nxt.alpha, nxt.weight, nxt.bias, h.dtype, extra, step)


class SurodraForCausalLM(nn.Module):
    supports_pp = False
    supports_lora = False
    # recurrent states live in per-row slots even when no layer is an attention layer
    row_state_slots = True
    # kernels outside the common set that this model launches (ops/build.py builds them on first use)
    native_sources = ("masked_attention.hip", "attention.hip", "attention_prefill.hip", "linear_attention.hip",
                      "delta_rule.hip", "mamba.hip")

    def __init__(self, vllm_config: VllmConfig, prefix: str = ""):
        super().__init__()
        config = vllm_config.model_config.hf_config
        self.config = config
        quant_config = getattr(vllm_config, "quant_config", None)
        width, self.eps = int(config.width), float(config.norm["eps"])
        mult = config.get("residual_mult")
        loop = config.get("loop")
        self.runs = run_order(len(config.layers), loop)
        passes = [0] * len(config.layers)
        for i, p in self.runs:
            passes[i] = max(passes[i], p + 1)
        # what joins the residual before a run: (embedding output?, row of loop.step or None)
        first = int(loop["start"]) if loop and int(loop["stop"]) > int(loop["start"]) else None
        self.joins = [(p > 0, p) if i == first else (False, None) for i, p in self.runs] + [(False, None)]
        self.embed_tokens = VocabParallelEmbedding(int(config.vocab), width)
        if loop:
            self.loop_step = _fp32_param((int(loop["times"]), width), 0.0)
        self.layers = nn.ModuleList([
            SurodraLayer(spec, width, self.eps, 1.0 if mult is None else float(mult), max(passes[i], 1), quant_config,
                         f"layers.{i}")
            for i, spec in enumerate(config.layers)])
        self.norm = SquashNorm(width)
        self.lm_head = ParallelLMHead(int(config.vocab), width)
        self.logits_processor = LogitsProcessor(int(config.vocab))
        scale, cap = config.get("logit_scale"), config.get("logit_softcap")
        self.logit_scale, self.soft_cap = 1.0 if scale is None else float(scale), float(cap or 0.0)

    def get_input_embeddings(self, input_ids):
        return self.embed_tokens(input_ids)

    def forward(self, input_ids, positions, intermediate_tensors=None, inputs_embeds=None):
        dtype = self.embed_tokens.weight.dtype
        e = (inputs_embeds if inputs_embeds is not None else self.embed_tokens(input_ids)).to(dtype)
        x = e.float() if dtype != torch.float32 else e.clone()
        norms = [self.layers[i].norm1 for i, _ in self.runs] + [self.norm]

        def joining(r):
            emb, row = self.joins[r]
            return e if emb else None, self.loop_step[row] if row is not None else None
        extra, step = joining(0)
        n = norms[0]
        h = ops.residual_squash_norm(x, [], 1.0, self.eps, n.alpha, n.weight, n.bias, dtype, extra, step)
        for r, (i, p) in enumerate(self.runs):
            h = self.layers[i](x, h, positions, p, norms[r + 1], *joining(r + 1))
        return h

    def compute_logits(self, hidden_states):
        return ops.scaled_softcap(self.logits_processor(self.lm_head, hidden_states), self.logit_scale, self.soft_cap)

    # checkpoint name -> (parameter name, shard id)
    _LINEAR = {"q": ("in_proj.weight", 0), "k": ("in_proj.weight", 1), "v": ("in_proj.weight", 2),
               "g": ("in_proj.weight", 3), "o": ("o_proj.weight", None)}
    _MIX = {
        "delta": {
            "q": ("core.in_proj.weight", 0), "k": ("core.in_proj.weight", 1), "v": ("core.in_proj.weight", 2),
            "g": ("core.in_proj.weight", 3), "b": ("core.in_proj.weight", 4), "a": ("core.in_proj.weight", 5),
            "q.conv": ("core.conv_weight", 0), "k.conv": ("core.conv_weight", 1), "v.conv": ("core.conv_weight", 2),
            "A_log": ("core.A_log", None), "dt_bias": ("core.dt_bias", None), "norm": ("core.norm_weight", None),
            "o": ("core.o_proj.weight", None)},
        "retention": {n: ("core." + t, s) for n, (t, s) in _LINEAR.items()},
        "parallel": {**{f"{side}.{n}": (f"{side}.{t}", s) for n, (t, s) in _LINEAR.items() for side in ("left", "right")},
                     "left.q.norm": ("left.q_norm", None), "left.k.norm": ("left.k_norm", None),
                     "left.sink": ("left.sink", None), "left.out": ("left_out", None),
                     "right.a1": ("right.in_proj.weight", 4), "right.a2": ("right.decay_up.weight", None),
                     "right.a2.b": ("right.decay_bias", None), "right.norm": ("right.norm_weight", None),
                     "right.out": ("right_out", None)},
    }
    _FF = {"gate": ("gate_up_proj.weight", 0), "up": ("gate_up_proj.weight", 1), "down": ("down_proj.weight", None)}
    _TOP = {"embed": "embed_tokens.weight", "head": "lm_head.weight", "loop.step": "loop_step"}
    _NORM = {"": "weight", ".b": "bias", ".alpha": "alpha"}

    def _target(self, name: str):
        """Returns (parameter name, shard id) or None."""
        if name in self._TOP:
            return self._TOP[name], None
        m = re.fullmatch(r"final\.norm(\.b|\.alpha)?", name)
        if m:
            return "norm." + self._NORM[m.group(1) or ""], None
        m = re.fullmatch(r"l(\d+)\.(.+)", name)
        if not m or int(m.group(1)) >= len(self.layers):
            return None
        i, rest = int(m.group(1)), m.group(2)
        layer, base = self.layers[i], f"layers.{i}."
        m = re.fullmatch(r"(norm[12])(\.b|\.alpha)?", rest)
        if m:
            return f"{base}{m.group(1)}.{self._NORM[m.group(2) or '']}", None
        part, _, leaf = rest.partition(".")
        if part == "mix" and leaf in self._MIX[layer.kind]:
            t, shard = self._MIX[layer.kind][leaf]
            return f"{base}mixer.{t}", shard
        if part == "mlp" and layer.has_mlp and leaf in self._FF:
            t, shard = self._FF[leaf]
            return f"{base}mlp.{t}", shard
        return None

    def load_weights(self, weights: Iterable[tuple[str, torch.Tensor]]) -> set[str]:
        params = dict(self.named_parameters())
        loaded: set[str] = set()
        for name, t in weights:
            tgt = self._target(name)
            if tgt is None or tgt[0] not in params:
                raise ValueError(f"checkpoint tensor {name!r} has no place in this model")
            target, shard = tgt
            p = params[target]
            loader = getattr(p, "weight_loader", default_weight_loader)
            if shard is None:
                loader(p, t)
            else:
                loader(p, t, shard)
            loaded.add(target)
        return loaded
