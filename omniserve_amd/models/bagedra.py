"""Bagedra: a decoder whose layers are latent attention (own latents or an earlier layer's), gated linear attention or the gated delta
rule in any order, each with a dense gated feed-forward or none, RMS norms on the sublayers' outputs only and scaled embeddings."""
from __future__ import annotations

import warnings

import torch

from .. import ckpt
from ..backend.lm import lm_ops
from .layers import (Decoder, DecoderSpec, DeltaSpec, DenseSpec, GatedLinearAttentionSpec, LatentAttentionSpec, LayerSpec, RotarySpec,
                     Weights)


def _mixer(kind: str, m: dict):
    if kind == "latent_attention":
        rot = m["rot"]
        if int(rot["dims"]) != int(m["rot_dim"]):
            raise ValueError("the whole rotated part turns: rot.dims is rot_dim")
        return LatentAttentionSpec(heads=m["heads"], dim=m["dim"], vdim=m["vdim"], kv_rank=m["kv_rank"], scale=float(m["scale"]),
                                   rotary=RotarySpec(int(rot["dims"]), float(rot["base"]), pairing="halves"), kv_from=m.get("kv_from"))
    if kind == "gla":
        return GatedLinearAttentionSpec(heads=m["heads"], dim=m["dim"], vdim=m["vdim"], tau=float(m["tau"]))
    if kind == "delta":
        return DeltaSpec(heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"], vdim=m["vdim"], taps=m["conv"])
    raise ValueError("unknown layer type %r" % kind)


def _feed_forward(m):
    if not m:
        return None
    if m.get("kind") != "dense":
        raise ValueError("unknown feed-forward kind %r" % m.get("kind"))
    return DenseSpec(ff=m["ff"])


def parse_config(config: dict) -> DecoderSpec:
    layers = tuple(LayerSpec(_mixer(l["type"], l["mixer"]), _feed_forward(l.get("mlp"))) for l in config["layers"])
    if not layers:
        raise ValueError("a model has at least one layer")
    return DecoderSpec(vocab=config["vocab"], width=config["width"], layers=layers, eps=float(config["norm"]["eps"]), norm="rms",
                       placement="after", embed_scale=float(config["embedding"]["scale"]))


class Bagedra(Decoder):
    @classmethod
    def from_state(cls, config: dict, state: dict, dtype=None, device="cuda") -> "Bagedra":
        dtype = dtype or torch.bfloat16
        w = Weights(state, torch.device(device), dtype)
        model = cls(parse_config(config), w, lm_ops(dtype))
        left = w.leftovers()
        if left:
            warnings.warn("the checkpoint has tensors the model does not use: %s" % ", ".join(left[:8]))
        return model

    @classmethod
    def from_pretrained(cls, model_dir: str, config: dict, dtype=None, device="cuda") -> "Bagedra":
        return cls.from_state(config, ckpt.load_state_dict(model_dir), dtype, device)
