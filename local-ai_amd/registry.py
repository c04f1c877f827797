"""Model registry: the ``architecture`` of a model folder's config.json -> how its configuration is read and which pipeline
serves it."""
from __future__ import annotations

import json
import os
from typing import Callable, Dict

from . import BF16, Context, InvalidArgument, Io, Kernels
from .mixers import (ACT_NONE, ACT_SILU, AttentionSpec, DenseSpec, GatedSpec, LatentAttentionSpec, LayerSpec, LinearAttentionSpec, MoeSpec,
                     OutputNormLayer, SelectiveSpec)
from .safetensors import SafetensorsFile
from .stack_pipeline import Loop, StackConfig, StackPipeline

ARCHITECTURES: Dict[str, Callable] = {}      # name -> config dict -> StackConfig


def register(name: str):
    def add(reader):
        ARCHITECTURES[name] = reader
        return reader
    return add


def read_config(config: dict) -> StackConfig:
    name = config.get("architecture")
    if name not in ARCHITECTURES:
        raise InvalidArgument(f"unknown architecture {name!r} (known: {', '.join(sorted(ARCHITECTURES))})")
    try:
        return ARCHITECTURES[name](config)
    except (KeyError, TypeError) as e:
        raise InvalidArgument(f"{name}: configuration lacks or misplaces {e}") from e


def load_model(path: str, max_tokens: int, dtype: int = BF16, ctx=None, **options) -> StackPipeline:
    """The pipeline for the model in folder `path` (config.json, model.safetensors)."""
    try:
        with open(os.path.join(path, "config.json")) as f:
            config = json.load(f)
    except (OSError, ValueError) as e:
        raise Io(f"{path}: {e}") from e
    stack = read_config(config)
    tensors = SafetensorsFile(os.path.join(path, "model.safetensors"))
    ctx = ctx or Context(0)
    return StackPipeline(ctx, Kernels(ctx), stack, tensors, max_tokens, dtype, **options)


@register("Komirax")
def komirax(config: dict) -> StackConfig:
    """Differential-attention and lightning-attention layers in any order, dense or routed feed-forwards, an optional loop."""
    def mixer(kind, m):
        if kind == "attention":
            return AttentionSpec(m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"], maps=2, diff=m["diff"], bias=True)
        if kind == "lightning":
            return LinearAttentionSpec(m["heads"], m["dim"], m["vdim"], list(m["decay"]))
        raise InvalidArgument(f"unknown layer type {kind!r}")

    def feed_forward(f):
        if f is None:
            return None
        if f["kind"] == "dense":
            return DenseSpec(f["ff"])
        if f["kind"] == "moe":
            return MoeSpec(f["router"]["experts"], f["router"]["top"], f["expert"]["ff"])
        raise InvalidArgument(f"unknown feed-forward {f['kind']!r}")

    layers = [LayerSpec(mixer(l["type"], l["mixer"]), feed_forward(l.get("mlp"))) for l in config["layers"]]
    loop = config.get("loop")
    return StackConfig(config["vocab"], config["width"], config["norm"]["eps"], layers,
                       Loop(loop["start"], loop["stop"], loop["times"]) if loop else None)


@register("Vifivik")
def vifivik(config: dict) -> StackConfig:
    """Latent-attention, retention and Mamba-2 layers in any order, gated feed-forwards, norms behind the branches, capped logits."""
    def mixer(kind, m):
        if kind == "latent_attention":
            if m["rot"]["dims"] != m["rot_dim"]:
                raise InvalidArgument(f"{m['rot']['dims']} rotated dimensions of a rotated part of {m['rot_dim']}")
            return LatentAttentionSpec(m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], m["rot"]["base"], m["scale"], m.get("kv_from"))
        if kind == "retention":
            return LinearAttentionSpec(m["heads"], m["dim"], m["vdim"], list(m["decay"]), ACT_NONE, m["dim"] ** -0.5, ACT_SILU, head_norm=True)
        if kind == "mamba2":
            return SelectiveSpec(m["heads"], m["vdim"], m["state"], m["groups"], m["conv"], m["norm_groups"])
        raise InvalidArgument(f"unknown layer type {kind!r}")

    def feed_forward(f):
        if f is None:
            return None
        if f["kind"] == "dense":
            return GatedSpec(f["ff"])
        raise InvalidArgument(f"unknown feed-forward {f['kind']!r}")

    layers = [LayerSpec(mixer(l["type"], l["mixer"]), feed_forward(l.get("mlp"))) for l in config["layers"]]
    return StackConfig(config["vocab"], config["width"], config["norm"]["eps"], layers, layer=OutputNormLayer, softcap=config.get("logit_softcap"))
