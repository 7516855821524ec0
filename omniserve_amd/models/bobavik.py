"""Bobavik: a decoder whose layers are softmax attention (sliding window, rotary positions, value mixing, output gate) or decayed
linear attention in any order, with mixtures of experts, layer norms before and after every sublayer and scaled logits."""
from __future__ import annotations

import warnings

import torch

from .. import ckpt
from ..backend.lm import lm_ops
from .layers import AttentionSpec, Decoder, DecoderSpec, LayerSpec, LinearAttentionSpec, MoeSpec, RotarySpec, Weights


def _mixer(kind: str, m: dict):
    if kind == "attention":
        rot, mask = m.get("rot"), m.get("mask")
        rotary = RotarySpec(int(rot["dims"]), float(rot["base"]), rot.get("scaling")) if rot else None
        return AttentionSpec(heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"], vdim=m["vdim"], scale=float(m["scale"]),
                             window=mask["size"] if mask else None, rotary=rotary, value_mix=bool(m.get("v_mix")))
    if kind == "lightning":
        return LinearAttentionSpec(heads=m["heads"], dim=m["dim"], vdim=m["vdim"], decay=tuple(float(d) for d in m["decay"]))
    raise ValueError("unknown layer type %r" % kind)


def _moe(m):
    if not m:
        return None
    if m.get("kind") != "moe":
        raise ValueError("unknown feed-forward kind %r" % m.get("kind"))
    shared = m.get("shared")
    return MoeSpec(experts=m["router"]["experts"], top=m["router"]["top"], ff=m["expert"]["ff"],
                   shared_ff=shared["ff"] if shared else None)


def parse_config(config: dict) -> DecoderSpec:
    layers = tuple(LayerSpec(_mixer(l["type"], l["mixer"]), _moe(l.get("mlp"))) for l in config["layers"])
    if not layers:
        raise ValueError("a model has at least one layer")
    return DecoderSpec(vocab=config["vocab"], width=config["width"], layers=layers, eps=float(config["norm"]["eps"]),
                       logit_scale=float(config.get("logit_scale", 1.0)))


class Bobavik(Decoder):
    @classmethod
    def from_state(cls, config: dict, state: dict, dtype=None, device="cuda") -> "Bobavik":
        dtype = dtype or torch.bfloat16
        w = Weights(state, torch.device(device), dtype)
        model = cls(parse_config(config), w, lm_ops(dtype))
        left = w.leftovers(optional=(".mix.vmix",))        # (the layer whose values the others mix in has no use for one)
        if left:
            warnings.warn("the checkpoint has tensors the model does not use: %s" % ", ".join(left[:8]))
        return model

    @classmethod
    def from_pretrained(cls, model_dir: str, config: dict, dtype=None, device="cuda") -> "Bobavik":
        return cls.from_state(config, ckpt.load_state_dict(model_dir), dtype, device)
