"""Small Sazavik configurations of the tests, and helpers that write them as model folders.

They differ from each other in every size and in the order of their layers: width, vocabulary, query and key/value heads
(numbers that are no power of two among them), key and value widths (equal and not, odd ones too), how many dims are turned
(all, some), chunks and windows (smaller, equal to and larger than pages and tiles), scales, temperatures, layers that read
another layer's keys (through a window or chunk of another size, and through none), dense and routed feed-forwards and
none, one, a few and all experts of a token, with and without a shared expert, with and without a cap on the logits.
"""
import json
import os

import torch

from macllm_infer_amd.config import SazavikConfig
from macllm_infer_amd.weights.random_init import random_tensors
from macllm_infer_amd.weights.safetensors_io import SafetensorsFile, write_safetensors


def _mixer(heads, kv_heads, dim, vdim, size, scale, kv_from):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": dim ** -0.5 if scale is None else scale}
    if size is not None:
        mixer["mask"] = {"size": size}
    if kv_from is not None:
        mixer["kv_from"] = kv_from
    return mixer


def chunked(heads, kv_heads, dim, vdim, size, rot, base=10000.0, halves=False, scale=None, kv_from=None):
    """``attention`` or, with pairs of ``halves``, ``attention_2``."""
    mixer = _mixer(heads, kv_heads, dim, vdim, size, scale, kv_from)
    mixer["rot"] = {"base": base, "dims": rot}
    return {"type": "attention_2" if halves else "attention", "mixer": mixer}


def distant(heads, kv_heads, dim, vdim, size, coef=0.3, every=16, scale=None, kv_from=None):
    mixer = _mixer(heads, kv_heads, dim, vdim, size, scale, kv_from)
    if every is not None:
        mixer["q_temp"] = {"coef": coef, "every": every}
    return {"type": "attention_3", "mixer": mixer}


def dense(ff, limit):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(experts, top, ff, shared=None):
    mlp = {"expert": {"ff": ff}, "kind": "moe", "router": {"experts": experts, "top": top}}
    if shared is not None:
        mlp["shared"] = {"ff": shared}
    return mlp


def with_mlp(layer, mlp):
    return dict(layer, mlp=mlp)


SAZ_A = {
    "architecture": "Sazavik", "width": 48, "vocab": 101, "norm": {"eps": 1e-5}, "logit_softcap": 20.0,
    "layers": [
        with_mlp(chunked(6, 2, 8, 12, 21, 4, base=500.0), moe(6, 2, 24, shared=20)),
        with_mlp(distant(3, 1, 10, 6, 13, every=7), dense(40, 0.9)),
        with_mlp(chunked(4, 4, 12, 8, 9, 12, halves=True), None),
        with_mlp(distant(6, 1, 10, 6, 30, coef=0.8, every=20, kv_from=1), moe(5, 1, 16)),
    ],
}

# odd widths, a layer that reads through no window at all, chunks read through another chunk, a token that uses every expert
SAZ_B = {
    "architecture": "Sazavik", "width": 40, "vocab": 67, "norm": {"eps": 1e-6},
    "layers": [
        with_mlp(distant(5, 5, 7, 9, 11, coef=-0.2, every=3), dense(24, 2.5)),
        with_mlp(chunked(2, 1, 16, 16, 64, 16, base=50.0, halves=True), moe(3, 3, 20)),
        with_mlp(distant(10, 5, 7, 9, None, every=None, scale=0.5, kv_from=0), moe(4, 2, 12, shared=8)),
        with_mlp(chunked(6, 1, 16, 16, 48, 16, base=50.0, halves=True, kv_from=1), dense(56, 0.5)),
        with_mlp(chunked(3, 3, 20, 4, 5, 6), None),
    ],
}

# widths that the matrix-core kernels take as they are (64 and 128) and padded (40, 80, 96), so that bfloat16 steps run
# through them; chunks and windows on both sides of tiles and pages
SAZ_C = {
    "architecture": "Sazavik", "width": 128, "vocab": 211, "norm": {"eps": 1e-5}, "logit_softcap": 50.0,
    "layers": [
        with_mlp(chunked(4, 2, 64, 64, 100, 32), dense(96, 1.2)),
        with_mlp(distant(6, 2, 64, 64, 37, every=64), moe(8, 3, 64, shared=32)),
        with_mlp(chunked(2, 1, 128, 128, 64, 128, halves=True, base=2e5), moe(8, 1, 32, shared=64)),
        with_mlp(distant(2, 2, 40, 80, 70, coef=0.1), dense(160, 3.0)),
        with_mlp(distant(8, 2, 64, 64, 90, kv_from=1), None),
        with_mlp(chunked(5, 1, 96, 40, 33, 8), moe(4, 4, 40)),
        with_mlp(chunked(2, 1, 96, 40, 128, 8, kv_from=5), dense(64, 0.7)),
    ],
}

CONFIGS = {"A": SAZ_A, "B": SAZ_B, "C": SAZ_C}


def config_of(name: str) -> SazavikConfig:
    return SazavikConfig.from_dict(json.loads(json.dumps(CONFIGS[name])))


def make_model_dir(name, folder, seed: int = 31, storage_dtype=torch.bfloat16, preset: str = "unit"):
    """Write the configuration ``name`` (or a raw configuration) with random weights into ``folder``; returns
    (raw config, tensors by their stored names, in float32).  Sinks are large enough to take a good share, routers sharp
    enough that few choices are close, and q and k norms strong enough that single keys stand out."""
    config = config_of(name) if isinstance(name, str) else SazavikConfig.from_dict(name)
    spec = config.to_model_spec()
    tensors = {spec.stored_name(key): value for key, value in random_tensors(config, seed, torch.float32, preset).items()}
    for key in tensors:
        if key.endswith(".sink"):
            tensors[key] = tensors[key] + 1.5
        elif key.endswith(".router"):
            tensors[key] = tensors[key] * 2.0
        elif key.endswith((".q.norm", ".k.norm")):
            tensors[key] = tensors[key] * 1.4
    os.makedirs(str(folder), exist_ok=True)
    raw = config.to_dict()
    with open(os.path.join(str(folder), "config.json"), "w") as handle:
        json.dump(raw, handle)
    path = os.path.join(str(folder), "model.safetensors")
    write_safetensors(path, {key: value.to(storage_dtype) for key, value in tensors.items()})
    handle = SafetensorsFile(path)
    stored = {key: handle.tensor(key).to(torch.float32) for key in handle.names()}
    handle.close()
    return raw, stored
