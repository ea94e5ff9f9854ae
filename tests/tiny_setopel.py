"""Tiny Setopel configurations that differ from each other in every size and option, and a folder of random weights for
each (norm weights drawn at random too, so that one taken for another, or left out, shows)."""
import json
import os

import torch

from tiny_gosuvik import random_tokens, read_folder  # noqa: F401  (the same folder format)


def attention(heads, kv_heads, dim, vdim, scale, ff, softcap=None, conv=None, temp=None, kv_from=None):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if softcap is not None:
        mixer["softcap"] = softcap
    if conv is not None:
        mixer["conv"] = conv
    if temp is not None:
        mixer["q_temp"] = {"coef": temp[0], "every": temp[1]}
    if kv_from is not None:
        mixer["kv_from"] = kv_from
    return {"type": "attention", "mixer": mixer, "mlp": dense(ff)}


def retention(heads, dim, vdim, decay, ff, rot=None):
    mixer = {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}
    assert len(decay) == heads
    if rot is not None:
        mixer["rot"] = {"dims": rot[0], "base": rot[1]}
    return {"type": "retention", "mixer": mixer, "mlp": dense(ff)}


def latent(heads, dim, vdim, rank, scale, ff):
    return {"type": "latent_attention", "mlp": dense(ff),
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": rank, "scale": scale}}


def dense(ff):
    return None if ff is None else {"kind": "dense", "ff": ff}


def config(vocab, width, eps, mult, streams, layers):
    cfg = {"architecture": "Setopel", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": mult,
           "layers": layers, "initializer_range": 0.08}
    if streams is not None:
        cfg["streams"] = streams
    return cfg


# A: all three mixers; values wider than keys; a short temperature step; a low cap; a layer that reads another one's
# keys with more query heads, another scale, another cap and another temperature; a partial rotation
A = config(320, 96, 1e-5, 0.6, 3, [
    attention(6, 2, 20, 28, 0.3, 64, softcap=4.0, conv=4, temp=(0.4, 8)),
    retention(3, 12, 20, [0.9, 0.99, 1.0], 48, rot=(8, 100.0)),
    latent(3, 16, 24, 40, 0.2, 64),
    attention(4, 2, 20, 28, 0.2, 80, softcap=6.0, conv=2, temp=(0.2, 5), kv_from=0),
    retention(2, 16, 8, [0.5, 0.97], None, rot=(16, 10000.0)),
])
# B: sizes that are no multiple of 4 or 8; no convolution, no cap, no temperature; nothing rotated; values narrower than
# keys; a layer with keys of its own between the one that shares its keys and the one that reads them
B = config(131, 74, 1e-6, 1.0, 2, [
    attention(3, 3, 10, 6, 0.4, None),
    attention(2, 1, 14, 18, 0.3, 36, softcap=3.0, conv=3),
    retention(2, 18, 9, [0.95, 0.8], 50),
    attention(6, 3, 10, 6, 0.5, 36, conv=3, temp=(1.0, 3), kv_from=0),
    latent(2, 12, 20, 36, 0.3, None),
])
# C: one copy of the stream, one head everywhere, one tap, temperature step of one token, a decay of zero, the retention
# layer first and last
C = config(97, 40, 1e-5, 0.3, 1, [
    retention(1, 8, 8, [0.0], 24, rot=(2, 50.0)),
    attention(1, 1, 16, 16, 0.5, 24, softcap=8.0, conv=1, temp=(0.5, 1)),
    latent(1, 16, 16, 16, 0.25, 40),
    retention(1, 20, 12, [1.0], None, rot=(20, 500.0)),
])
# D: sizes that the matrix-core attention kernels and the chunked recurrence take (heads of 32, 64 and 128 numbers,
# latents in multiples of 32), eight query heads on two key heads, sixteen query heads on one latent
D = config(256, 128, 1e-5, 0.5, 4, [
    attention(8, 2, 32, 32, 0.2, 96, softcap=10.0, conv=4, temp=(0.3, 16)),
    retention(2, 64, 40, [0.97, 0.995], 96, rot=(64, 1000.0)),
    latent(16, 24, 40, 64, 0.15, None),
    attention(4, 1, 128, 128, 0.09, None, softcap=20.0, conv=3, temp=(0.2, 32)),
    attention(16, 2, 32, 32, 0.2, 96, softcap=12.0, conv=4, kv_from=0),
    retention(1, 128, 136, [0.99], None, rot=(32, 1e6)),
    attention(4, 4, 48, 48, 0.15, 64, softcap=9.0, conv=2),
])
# E: a plain residual stream (no copies) with a gain on every branch; widths that are no multiple of 4
E = config(77, 90, 1e-5, 0.7, None, [
    attention(4, 2, 12, 14, 0.3, 50, softcap=2.0, conv=5, temp=(0.6, 4)),
    retention(2, 10, 6, [0.9, 0.7], 50, rot=(6, 300.0)),
    latent(2, 10, 14, 22, 0.25, 28),
    attention(2, 2, 12, 14, 0.3, None, kv_from=0),
])
# F: more copies than the kernel keeps in registers; retention only (no pages at all)
F = config(64, 48, 1e-5, 0.25, 9, [
    retention(4, 32, 32, [0.9, 0.95, 0.99, 0.999], 64, rot=(32, 1000.0)),
    retention(3, 96, 12, [0.8, 0.9, 1.0], 64, rot=(48, 200.0)),
])
CONFIGS = {"A": A, "B": B, "C": C, "D": D, "E": E, "F": F}


def make_folder(raw_config: dict, seed: int, out_dir: str, dtype: str = "bfloat16") -> str:
    from safetensors.torch import load_file, save_file
    from inferx_amd.config import config_from_dict
    from inferx_amd.weights import write_model_folder
    write_model_folder(config_from_dict(json.loads(json.dumps(raw_config))), seed, out_dir, dtype)
    path = os.path.join(out_dir, "model.safetensors")
    tensors = load_file(path)
    g = torch.Generator().manual_seed(seed + 1)
    for name, t in tensors.items():
        if name.split(".")[-1].startswith("norm"):  # l<i>.norm1, final.norm, embed.norm: around zero; the latent's around one
            middle = 1.0 if name.endswith(".dkv.norm") else 0.0
            tensors[name] = (middle + 0.3 * torch.randn(t.shape, generator=g)).to(t.dtype)
        elif name.endswith(".b"):
            tensors[name] = (0.5 * torch.randn(t.shape, generator=g)).to(t.dtype)
        elif name.endswith((".mix.q", ".mix.k", ".mix.uk")):  # scores that stand out, so that caps and temperatures show
            tensors[name] = (t.float() * 2.5).to(t.dtype)
    save_file(tensors, path)
    return out_dir
