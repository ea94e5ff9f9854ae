"""Tiny Zevivik configurations that differ from each other in every size and option, and a folder of random weights for
each (norm weights, router biases and the loop's vectors drawn so that one taken for another, or left out, shows)."""
import json
import os

import torch

from tiny_gosuvik import random_tokens, read_folder  # noqa: F401  (the same folder format)


def attention(heads, kv_heads, dim, vdim, scale, chunk, rot, mlp):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if chunk is not None:
        mixer["mask"] = {"size": chunk}
    if rot is not None:
        mixer["rot"] = {"dims": rot[0], "base": rot[1]}
    return {"type": "attention", "mixer": mixer, "mlp": mlp}


def latent(heads, dim, vdim, rank, scale, mlp):
    return {"type": "latent_attention", "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": rank, "scale": scale}}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def experts(ff, limit, count, top, shared=None):
    mlp = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": count, "top": top}}
    if shared is not None:
        mlp["shared"] = {"ff": shared[0], "limit": shared[1]}
    return mlp


def config(vocab, width, eps, scale, layers, loop=None):
    cfg = {"architecture": "Zevivik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
           "layers": layers, "initializer_range": 0.08}
    if loop is not None:
        cfg["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return cfg


# A: values wider and narrower than keys, a part of the heads rotated, chunks of a page and of seven, a shared expert with a
# size and limit of its own, a layer without feed-forward, two layers of the middle three times
A = config(320, 96, 1e-5, 1.7, [
    attention(6, 2, 20, 28, 0.3, 16, (12, 100.0), experts(24, 0.7, 6, 2, (40, 1.3))),
    latent(3, 16, 24, 40, 0.3, dense(64)),
    attention(4, 1, 24, 12, 0.2, 7, (24, 3000.0), None),
    latent(2, 12, 8, 32, 0.4, experts(40, 1.1, 9, 3)),
], loop=(1, 3, 3))
# B: sizes that are no multiple of 4 or 8, odd heads, the loop over the whole model, one expert per token
B = config(131, 74, 1e-6, 0.6, [
    latent(2, 13, 19, 36, 0.3, dense(50)),
    attention(3, 3, 11, 6, 0.4, 5, (10, 50.0), experts(36, 0.5, 5, 1)),
    attention(2, 1, 14, 18, 0.3, 33, (6, 10000.0), dense(36)),
], loop=(0, 3, 2))
# C: no loop, one head everywhere, chunks of one token (a token sees itself) and of two, every expert chosen, scale 1
C = config(97, 40, 1e-5, 1.0, [
    attention(1, 1, 8, 8, 0.5, 1, (2, 500.0), experts(24, 2.0, 2, 2, (24, 2.0))),
    latent(1, 16, 16, 16, 0.25, dense(24)),
    attention(1, 1, 16, 16, 0.5, 2, (16, 70.0), dense(40)),
])
# D: sizes that the matrix-core kernels take as they are (heads of 32, 64 and 128 numbers, latents in multiples of 32),
# grouped query heads, a shared expert of twice the experts' width with their limit
D = config(256, 128, 1e-5, 2.5, [
    attention(8, 2, 32, 32, 0.2, 40, (16, 5000.0), experts(32, 0.9, 8, 3, (64, 0.9))),
    latent(16, 24, 40, 64, 0.15, dense(96)),
    attention(4, 1, 128, 128, 0.09, 64, (128, 1e6), experts(48, 1.2, 12, 2, (80, 0.6))),
    attention(16, 2, 64, 32, 0.1, 100, (64, 1000.0), None),
], loop=(0, 2, 2))
# E: a loop of one pass (its vector alone enters) at the end, attention without chunks and without a rotation, odd widths
E = config(77, 90, 1e-5, 1.3, [
    attention(4, 2, 12, 14, 0.3, None, (6, 300.0), dense(50)),
    latent(2, 10, 14, 22, 0.3, experts(28, 0.8, 3, 2, (20, 0.4))),
    attention(2, 2, 12, 12, 0.3, 9, None, experts(28, 0.8, 70, 6)),
], loop=(1, 3, 1))
# F: one layer four times, heads of more than 128 numbers, long chunks that end within a page
F = config(64, 48, 1e-5, 4.0, [
    attention(2, 1, 200, 160, 0.05, 56, (100, 1000.0), dense(64)),
    attention(3, 1, 48, 80, 0.15, 24, (48, 200.0), experts(64, 1.5, 4, 2)),
    latent(4, 32, 32, 96, 0.2, dense(32)),
], loop=(1, 2, 4))
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
        if name.split(".")[-1].startswith("norm"):
            tensors[name] = (1.0 + 0.3 * torch.randn(t.shape, generator=g)).to(t.dtype)
        elif name.endswith((".mix.q", ".mix.k", ".mix.uk")):  # scores that stand out
            tensors[name] = (t.float() * 2.5).to(t.dtype)
        elif name == "loop.step":
            tensors[name] = (t.float() * 4.0).to(t.dtype)
        elif name.endswith(".mix.g"):  # gates from nearly shut to nearly open
            tensors[name] = (t.float() * 3.0).to(t.dtype)
    save_file(tensors, path)
    return out_dir
