"""Small Vipalorn configurations for tests, and model folders made from them.

A mixes both mixers, latent attention whose cached head (28 + 8) is padded to 48 and whose rotation covers part of the
rotated dimensions, grouped delta-rule heads with three taps, layers with and without experts. B has twenty latent
heads (more than one wave of the matrix-core decode kernel takes), one expert chosen of one, experts of the sizes
whose matrices are packed, delta-rule keys wider
than their values and ungrouped. C has sizes in no step of 8, convolutions of one tap (no state beside the matrix), all
experts chosen, three value heads on one key head. D is five delta-rule layers of one shape in a row, with keys and
values of different sizes in the matrix-core steps, no factors on the stream or the logits. E is attention alone:
a cached head of 256, the widest of the matrix-core kernels, and one of 280, which the float32 kernel takes. F has keys
of 144 dimensions (the chunks' widest memory), four heads on one key head, eight taps, values of one block and a half.
"""

import json
import os

import torch


def _latent(heads, dim, rot_dim, vdim, rank, scale, base, dims=None):
    return {"type": "latent_attention",
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": rank, "scale": scale,
                      "rot": {"dims": dims or rot_dim, "base": base}}}


def _delta(heads, kv_heads, dim, vdim, conv):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


def _moe(experts, top, ff, limit):
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}


A = {
    "architecture": "Vipalorn", "vocab": 101, "width": 64, "norm": {"eps": 1e-5}, "residual_mult": 0.7,
    "logit_scale": 0.5,
    "layers": [
        {**_latent(3, 24, 8, 40, 28, 0.2, 100.0, dims=6), "mlp": _moe(6, 2, 24, 0.8)},
        {**_delta(4, 2, 8, 24, 3), "mlp": _moe(5, 3, 40, 1.5)},
        {**_delta(6, 3, 16, 16, 2), "mlp": None},
        {**_latent(2, 16, 16, 16, 32, 0.25, 1000.0), "mlp": None},
        {**_delta(2, 1, 32, 48, 4), "mlp": _moe(4, 1, 16, 0.5)},
    ],
}
B = {
    "architecture": "Vipalorn", "vocab": 211, "width": 96, "norm": {"eps": 1e-6}, "residual_mult": 1.25,
    "logit_scale": 3.0,
    "layers": [
        {**_delta(2, 2, 40, 16, 2), "mlp": _moe(1, 1, 96, 2.0)},
        {**_latent(20, 16, 16, 8, 48, 0.15, 777.0), "mlp": _moe(16, 4, 128, 1.0)},
        {**_latent(4, 32, 32, 24, 64, 0.1, 250.0), "mlp": None},
    ],
}
C = {
    "architecture": "Vipalorn", "vocab": 333, "width": 100, "norm": {"eps": 1e-4}, "residual_mult": 0.3,
    "layers": [
        {**_latent(5, 10, 6, 7, 13, 0.3, 30.0), "mlp": _moe(6, 6, 9, 1.2)},
        {**_delta(3, 1, 20, 9, 1), "mlp": _moe(7, 2, 11, 0.6)},
    ],
}
D = {
    "architecture": "Vipalorn", "vocab": 64, "width": 48, "norm": {"eps": 1e-5},
    "layers": [{**_delta(2, 1, 64, 80, 4), "mlp": _moe(4, 2, 32, 1.0)} for _ in range(5)],
}
E = {
    "architecture": "Vipalorn", "vocab": 90, "width": 80, "norm": {"eps": 1e-5}, "residual_mult": 0.5,
    "logit_scale": 1.5,
    "layers": [
        {**_latent(8, 48, 16, 32, 240, 0.1, 9000.0), "mlp": _moe(12, 5, 32, 0.9)},
        {**_latent(2, 8, 10, 16, 270, 0.2, 50.0), "mlp": _moe(3, 2, 24, 4.0)},
    ],
}
F = {
    "architecture": "Vipalorn", "vocab": 77, "width": 72, "norm": {"eps": 1e-5}, "residual_mult": 0.9,
    "layers": [
        {**_delta(4, 1, 144, 24, 8), "mlp": None},
        {**_delta(2, 2, 12, 33, 5), "mlp": _moe(9, 3, 16, 1.0)},
    ],
}
CONFIGS = {"A": A, "B": B, "C": C, "D": D, "E": E, "F": F}
BLOCK_SIZE = {"A": 4, "B": 16, "C": 8, "D": 16, "E": 16, "F": 32}


def make_tensors(config: dict, seed: int, dtype: str):
    """Random tensors of the design, drawn wider than the serving default so that every mechanism moves the logits:
    matrices three times as wide and the queries more (a softmax mostly looks at few keys), experts' matrices so wide
    that their sums meet the limit now and then, a router whose logits spread."""
    from tie_amd.models.builder import expected_tensors_for_config
    from tie_amd.weights.random_init import random_tensors

    store = torch.float32 if dtype == "float32" else torch.bfloat16
    specs = expected_tensors_for_config(config)
    tensors = dict(random_tensors(specs, seed, torch.float32, vector_dtype=torch.float32))
    for name, t in tensors.items():
        if name == "embed":
            t.mul_(3.0)
        elif name.endswith(".mix.q") and name[:-2] + ".dkv" in tensors or name.endswith(".mlp.router"):
            t.mul_(9.0)
        elif name.endswith(".router.b"):
            t.mul_(25.0)
        elif name.endswith((".gate", ".up")):
            t.mul_(6.0)
        elif name.endswith((".mix.o", ".down")):
            t.mul_(25.0)          # against a stream that the embedding's norm makes of the order of one
        elif t.dim() == 2 and not name.endswith(".conv"):
            t.mul_(3.0)
    if dtype == "bfloat16":
        # Rounding must not change who is chosen: the router's bias holds levels 1.5 apart, in an order the seed draws,
        # further apart than the (narrow) router moves a logit. The weights still follow the tokens. The float32
        # fixtures route by the tokens.
        g = torch.Generator().manual_seed(seed)
        for name, t in tensors.items():
            if name.endswith(".mlp.router"):
                t.div_(9.0)
            elif name.endswith(".router.b"):
                t.copy_(1.5 * (torch.randperm(t.numel(), generator=g).to(torch.float32) - (t.numel() - 1) / 2.0))
    return {n: t.to(store) for n, t in tensors.items()}


def write_model(folder, config: dict, seed: int, dtype: str, change=None) -> str:
    """``change``: a function that edits the dictionary of tensors before it is written."""
    from tie_amd.weights.safetensors_io import write_safetensors

    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(config, f)
    tensors = make_tensors(config, seed, dtype)
    if change is not None:
        change(tensors)
    write_safetensors(os.path.join(folder, "model.safetensors"), list(tensors.items()))
    return str(folder)


def load_plain(folder):
    from safetensors import safe_open

    weights = {}
    with safe_open(os.path.join(folder, "model.safetensors"), framework="pt") as f:
        for name in f.keys():
            weights[name] = f.get_tensor(name).to(torch.float64)
    return weights
