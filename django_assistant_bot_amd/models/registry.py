"""Decoder families: the configuration class of a model decides its model class and weight sources."""
from __future__ import annotations

from dataclasses import dataclass
from typing import Callable

import torch

from .bizetar import BizetarModel
from .configs import BizetarConfig, DecoderConfig, VugotarConfig, VumuvikConfig, VunelixConfig
from .llama import LlamaModel
from .vugotar import VugotarModel
from .vumuvik import VumuvikModel
from .vunelix import VunelixModel
from .weights import (
    load_bizetar_checkpoint,
    load_decoder_checkpoint,
    load_vugotar_checkpoint,
    load_vumuvik_checkpoint,
    load_vunelix_checkpoint,
    random_bizetar_weights,
    random_decoder_weights,
    random_vugotar_weights,
    random_vumuvik_weights,
    random_vunelix_weights,
)


@dataclass(frozen=True)
class DecoderFamily:
    model: type
    random: Callable  # (cfg, device, dtype, seed, tp_rank, tp_size, interleave_mlp) -> weights
    load: Callable  # (path, cfg, device, dtype, tp_rank, tp_size, interleave_mlp) -> weights
    gpu_dtypes: tuple = (torch.bfloat16,)


def _single(fn):
    """A weight source of a family without tensor parallelism."""
    def call(*args, tp_rank=0, tp_size=1, **kw):
        if tp_size != 1:
            raise ValueError("this model family runs on one GPU per replica (tp_size 1)")
        return fn(*args, **kw)
    return call


def _load_llama(path, cfg, device="cpu", **kw):
    return load_decoder_checkpoint(path, cfg, **kw)  # host tensors: the model moves them as it converts


FAMILIES = {
    DecoderConfig: DecoderFamily(LlamaModel, random_decoder_weights, _load_llama),
    VumuvikConfig: DecoderFamily(VumuvikModel, _single(random_vumuvik_weights), _single(load_vumuvik_checkpoint),
                                 (torch.bfloat16, torch.float32)),
    VugotarConfig: DecoderFamily(VugotarModel, _single(random_vugotar_weights), _single(load_vugotar_checkpoint),
                                 (torch.bfloat16, torch.float32)),
    VunelixConfig: DecoderFamily(VunelixModel, _single(random_vunelix_weights), _single(load_vunelix_checkpoint),
                                 (torch.bfloat16, torch.float32)),
    BizetarConfig: DecoderFamily(BizetarModel, _single(random_bizetar_weights), _single(load_bizetar_checkpoint),
                                 (torch.bfloat16, torch.float32)),
}


def decoder_family(cfg) -> DecoderFamily:
    return FAMILIES[type(cfg)]
