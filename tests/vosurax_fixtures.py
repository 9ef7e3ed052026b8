"""Small Vosurax configurations for tests, and model folders made from them.

A mixes both mixers and every kind of feed-forward (dense, routed with a shared expert cut into two pieces, none), with
value heads wider than key heads (padded heads that take a norm and a bias), a rotation of part of a head, chunks shorter
than a page's multiple, layers in the middle that run three times. B has sizes in the matrix cores' steps: twenty query
heads on one key/value head, packed experts, all layers in a loop of one pass that starts at the first layer. C has sizes
in no step of 8, every key visible, no shared expert, one head everywhere, no loop. D is five layers of one shape in a row
(the two mixers side by side). E has wide heads: memories of 144 x 200 and 36 x 300, a retention of 272 x 40, attention of
280 (which the float32 kernel takes), its last layer looped twice. F is five retention layers of one shape in a row behind
a looped pair without feed-forwards.
"""

import json
import os

import torch


def _parallel(left, right):
    """left (heads, kv_heads, dim, vdim, scale, chunk or None), right (heads, dim, vdim, gate_cap)."""
    heads, kv, dim, vdim, scale, chunk = left
    m = {"left": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale},
         "right": dict(zip(("heads", "dim", "vdim", "gate_cap"), right))}
    if chunk is not None:
        m["left"]["mask"] = {"size": chunk}
    return {"type": "parallel", "mixer": m}


def _retention(dim, vdim, decay, base, dims):
    return {"type": "retention", "mixer": {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": list(decay),
                                           "rot": {"base": base, "dims": dims}}}


def _moe(experts, top, ff, shared_ff=None):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared_ff is not None:
        m["shared"] = {"ff": shared_ff}
    return m


def _dense(ff):
    return {"kind": "dense", "ff": ff}


A = {
    "architecture": "Vosurax", "vocab": 103, "width": 64, "norm": {"eps": 1e-5},
    "loop": {"start": 1, "stop": 3, "times": 3},
    "layers": [
        {**_parallel((6, 2, 24, 40, 0.3, 19), (3, 20, 28, 4.0)), "mlp": _dense(88)},
        {**_retention(16, 24, [0.9, 0.99, 1.0, 0.5], 100.0, 6), "mlp": _moe(6, 2, 24, 40)},
        {**_parallel((4, 4, 32, 16, 0.2, 33), (2, 16, 40, 9.0)), "mlp": None},
        {**_parallel((4, 1, 16, 16, 0.4, 70), (5, 8, 12, 2.0)), "mlp": _moe(5, 3, 40, 16)},
        {**_retention(32, 8, [0.97, 0.995], 5000.0, 32), "mlp": _dense(40)},
    ],
}
B = {
    "architecture": "Vosurax", "vocab": 211, "width": 96, "norm": {"eps": 1e-6},
    "loop": {"start": 0, "stop": 3, "times": 1},
    "layers": [
        {**_parallel((20, 1, 32, 32, 0.2, 48), (2, 64, 80, 15.0)), "mlp": _moe(16, 4, 128, 128)},
        {**_retention(64, 96, [0.98, 0.999, 0.96], 777.0, 48), "mlp": _dense(192)},
        {**_parallel((8, 2, 64, 64, 0.12, 130), (4, 32, 32, 6.0)), "mlp": _moe(7, 1, 96, 224)},
    ],
}
C = {
    "architecture": "Vosurax", "vocab": 333, "width": 100, "norm": {"eps": 1e-4},
    "layers": [
        {**_parallel((3, 1, 10, 7, 0.5, None), (1, 9, 5, 3.0)), "mlp": _moe(6, 6, 9)},
        {**_retention(6, 11, [0.93], 30.0, 4), "mlp": _dense(21)},
        {**_parallel((1, 1, 33, 33, 0.2, 7), (2, 30, 30, 1.0)), "mlp": None},
    ],
}
D = {
    "architecture": "Vosurax", "vocab": 64, "width": 48, "norm": {"eps": 1e-5},
    "layers": [{**_parallel((4, 2, 16, 32, 0.3, 40), (2, 40, 72, 5.0)), "mlp": _moe(4, 2, 32, 32)} for _ in range(5)],
}
E = {
    "architecture": "Vosurax", "vocab": 90, "width": 80, "norm": {"eps": 1e-5},
    "loop": {"start": 2, "stop": 3, "times": 2},
    "layers": [
        {**_parallel((2, 1, 256, 240, 0.06, 100), (2, 144, 200, 8.0)), "mlp": _moe(12, 5, 32, 96)},
        {**_retention(272, 40, [0.99, 0.9], 9000.0, 200), "mlp": None},
        {**_parallel((2, 2, 280, 264, 0.05, 64), (1, 36, 300, 20.0)), "mlp": _dense(64)},
    ],
}
F = {
    "architecture": "Vosurax", "vocab": 77, "width": 72, "norm": {"eps": 1e-5},
    "loop": {"start": 0, "stop": 2, "times": 2},
    "layers": [
        {**_parallel((4, 2, 16, 16, 0.4, 25), (3, 16, 16, 7.0)), "mlp": None},
        {**_retention(8, 8, [0.9, 0.8], 60.0, 8), "mlp": None},
    ] + [{**_retention(24, 36, [0.95, 0.99, 0.999], 1000.0, 16), "mlp": _dense(48)} for _ in range(5)],
}
CONFIGS = {"A": A, "B": B, "C": C, "D": D, "E": E, "F": F}
BLOCK_SIZE = {"A": 4, "B": 16, "C": 8, "D": 16, "E": 16, "F": 32}


def make_tensors(config: dict, seed: int, dtype: str):
    """Random tensors of the design, drawn wider than the serving default so that every mechanism moves the logits:
    queries that mostly look at few keys, gates that open and close, a router whose logits spread."""
    from tie_amd.models.builder import expected_tensors_for_config
    from tie_amd.weights.random_init import random_tensors

    store = torch.float32 if dtype == "float32" else torch.bfloat16
    specs = expected_tensors_for_config(config)
    tensors = dict(random_tensors(specs, seed, torch.float32, vector_dtype=torch.float32))
    for name, t in tensors.items():
        if name == "embed":
            t.mul_(40.0)
        elif name == "loop.step":
            t.mul_(30.0)
        elif name.endswith((".right.i", ".right.f", ".mlp.router")):
            t.mul_(8.0)
        elif name.endswith((".q.b", ".k.b", ".v.b")):
            t.mul_(20.0)
        elif name.endswith((".left.q.norm", ".left.k.norm")):
            t.mul_(1.1)
        elif name.endswith((".left.out", ".right.out")):
            t.mul_(0.7)
        elif name.endswith((".mix.o", ".down")):
            t.mul_(6.0)
        elif t.dim() == 2:
            t.mul_(4.0)
    if dtype == "bfloat16":
        # Rounding must not change who is chosen: the stream's first column is the same number for every token and is
        # left alone by every sub-layer, and the router's first column holds levels, in an order the seed draws, that
        # stand further apart than the (narrow) rest of the router moves a logit. The weights still follow the tokens;
        # the float32 fixtures also choose by the tokens.
        g = torch.Generator().manual_seed(seed)
        for name, t in tensors.items():
            if name == "embed":
                t[:, 0] = 1.5
            elif name == "loop.step":
                t[:, 0] = 0.0
            elif name.endswith((".o", ".down")):
                t[0] = 0.0
            elif name.endswith(".norm2"):
                t[0] = 1.0
            elif name.endswith(".mlp.router"):
                t.div_(8.0)
                n = t.shape[0]
                t[:, 0] = 0.4 * (torch.randperm(n, generator=g).to(torch.float32) - (n - 1) / 2.0)
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
