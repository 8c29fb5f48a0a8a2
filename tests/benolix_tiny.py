"""Tiny Benolix configurations for the tests, as raw config.json dictionaries, and model folders with weights drawn so
that every mechanism shows in the logits: scores wide enough for single keys to count, corrections that change the
choice of experts, gate and up rows that reach their clamp.

Between them the configurations cover: latents of a layer read by one layer and by two, by a layer with a narrower, a
wider and no window; layers of different heads, head sizes and ranks; windows of 1, inside a page, at a page's size,
one past it and none; a rotation of a part of the rotated entries; layers without feed-forward (with and without a
second norm in the checkpoint); routers with none, few and mostly identity experts, that take one, several and all of
their outputs, with scales below and above 1; embedding scale and alpha of 1 and others.
"""

from __future__ import annotations

import functools
import json
import os
import tempfile
import zlib

import torch

from plain_benolix import PlainBenolix


def _attn(heads, dim, rot_dim, vdim, rank, q_rank, window, base=10000.0, dims=None, scale=None, kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": rank, "q_rank": q_rank,
         "rot": {"base": base, "dims": rot_dim if dims is None else dims},
         "scale": scale if scale is not None else 1.6 * (dim + rot_dim) ** -0.5}
    if window is not None:
        m["mask"] = {"size": window}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return m


def _dense(ff):
    return {"kind": "dense", "ff": ff}


def _moe(ff, experts, top, identity=0, limit=1.5, scale=1.0):
    router = {"experts": experts, "top": top, "scale": scale}
    if identity:
        router["identity"] = identity
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": router}


def _layers(*pairs):
    return [{"type": "latent_attention", "mixer": m, "mlp": mlp} for m, mlp in pairs]


# A: odd sizes throughout (the general kernels); a wider window over borrowed latents, then latents kept without end
BENO_A = {
    "architecture": "Benolix", "vocab": 89, "width": 44, "embedding": {"scale": 2.5}, "norm": {"eps": 3e-5},
    "postln_alpha": 1.4,
    "layers": _layers(
        (_attn(3, 10, 6, 7, 20, 14, 9, base=500.0), _dense(52)),
        (_attn(5, 6, 6, 4, 20, 9, 23, base=500.0, kv_from=0), _moe(24, 5, 3, identity=2, scale=1.7)),
        (_attn(2, 7, 4, 9, 12, 11, None, base=90.0), None),
        (_attn(4, 5, 4, 6, 12, 13, 5, base=90.0, kv_from=2), _moe(18, 4, 1, scale=0.6)),
    ),
}

# B: sizes the matrix-core kernels take; two layers read the same latents, one of them past the owner's window
BENO_B = {
    "architecture": "Benolix", "vocab": 120, "width": 56, "embedding": {"scale": 6.0}, "norm": {"eps": 1e-6},
    "postln_alpha": 2.0,
    "layers": _layers(
        (_attn(4, 16, 8, 24, 32, 40, 17), _moe(32, 6, 2, identity=2, limit=2.5, scale=2.2)),
        (_attn(2, 24, 8, 16, 32, 24, 41, kv_from=0), _dense(72)),
        (_attn(6, 8, 8, 8, 32, 16, 16, kv_from=0), _moe(40, 3, 4, identity=5, limit=0.8, scale=1.3)),
        (_attn(3, 32, 16, 16, 48, 32, 33, base=70000.0), _dense(48)),
    ),
}

# C: more than sixteen heads, a rotation of half of the rotated entries, every constant that can be 1 is 1
BENO_C = {
    "architecture": "Benolix", "vocab": 71, "width": 64, "embedding": {"scale": 1.0}, "norm": {"eps": 1e-5},
    "postln_alpha": 1.0,
    "layers": _layers(
        (_attn(20, 8, 16, 8, 64, 48, 64, dims=8), _moe(16, 70, 6, identity=10, limit=1.0, scale=1.0)),
        (_attn(18, 16, 16, 12, 64, 64, 130, dims=8, kv_from=0), _dense(80)),
        (_attn(1, 24, 8, 40, 16, 8, 1), _moe(24, 2, 2, limit=3.0)),
    ),
}

# D: every window is none or one token; all outputs of the router are taken; one identity expert among two
BENO_D = {
    "architecture": "Benolix", "vocab": 53, "width": 32, "embedding": {"scale": 0.7}, "norm": {"eps": 2e-6},
    "postln_alpha": 0.5,
    "layers": _layers(
        (_attn(2, 12, 2, 10, 16, 6, None), _moe(12, 1, 2, identity=1, limit=1.2, scale=3.0)),
        (_attn(2, 12, 2, 10, 16, 6, None, kv_from=0), None),
        (_attn(3, 4, 12, 5, 24, 10, 1, base=33.0), _dense(36)),
    ),
}

# E: latents and experts of sizes that the tile kernels for real models take
BENO_E = {
    "architecture": "Benolix", "vocab": 101, "width": 128, "embedding": {"scale": 3.0}, "norm": {"eps": 1e-5},
    "postln_alpha": 1.7,
    "layers": _layers(
        (_attn(5, 40, 64, 24, 128, 72, 70), _moe(64, 3, 2, identity=1, limit=1.8, scale=1.5)),
        (_attn(16, 16, 64, 8, 128, 48, 131, kv_from=0), _dense(192)),
        (_attn(20, 24, 64, 16, 256, 96, None, base=3000.0), _moe(128, 2, 1, identity=2, limit=0.9, scale=0.8)),
        (_attn(2, 32, 64, 64, 256, 56, 65, base=3000.0, kv_from=2), None),
    ),
}

CONFIGS = {"A": BENO_A, "B": BENO_B, "C": BENO_C, "D": BENO_D, "E": BENO_E}
SEEDS = {"A": 5, "B": 15, "C": 25, "D": 45, "E": 65}
BARE_SECOND_NORM = {("D", 1)}     # layers without feed-forward whose checkpoint holds a second norm all the same


def _draw(name: str, shape, seed: int) -> torch.Tensor:
    g = torch.Generator().manual_seed((seed * 1000003 + zlib.crc32(name.encode())) % (2 ** 63))
    last = name.rsplit(".", 1)[-1]
    z = torch.randn(shape, generator=g)
    if last in ("norm1", "norm2") or name == "final.norm":
        return 0.2 * z                          # stored as the distance from one
    if last == "correction":
        return 0.3 * z
    if last == "embed":
        return z
    if len(shape) == 1:                         # plain norm weights
        return 1.0 + 0.2 * z
    if last == "router":
        return 1.5 * z / shape[-1] ** 0.5
    return z / shape[-1] ** 0.5                 # matrices: outputs of unit size


def shapes(which: str) -> dict:
    """Every tensor a checkpoint of configuration ``which`` holds, by name, written out here from the design (not taken
    from the engine's own list): the tests compare the two."""
    cfg = CONFIGS[which]
    w, v = cfg["width"], cfg["vocab"]
    out = {"embed": (v, w), "final.norm": (w,), "head": (v, w)}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.mix.", layer["mixer"]
        H, D, R, V, rank, qr = (m[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank"))
        out[f"l{i}.norm1"] = (w,)
        out.update({p + "dq": (qr, w), p + "dq.norm": (qr,), p + "uq": (H * (D + R), qr), p + "uk": (H * D, rank),
                    p + "uv": (H * V, rank), p + "g": (H * V, w), p + "o": (w, H * V)})
        if "kv_from" not in m:
            out.update({p + "dkv": (rank + R, w), p + "dkv.norm": (rank,)})
        mlp, p = layer["mlp"], f"l{i}.mlp."
        if mlp is not None or (which, i) in BARE_SECOND_NORM:
            out[f"l{i}.norm2"] = (w,)
        if mlp is not None and mlp["kind"] == "dense":
            out.update({p + "gate": (mlp["ff"], w), p + "up": (mlp["ff"], w), p + "down": (w, mlp["ff"])})
        elif mlp is not None:
            n, ff = mlp["router"]["experts"], mlp["expert"]["ff"]
            outputs = n + mlp["router"].get("identity", 0)
            out.update({p + "router": (outputs, w), p + "correction": (outputs,)})
            for e in range(n):
                out.update({f"{p}e{e}.gate": (ff, w), f"{p}e{e}.up": (ff, w), f"{p}e{e}.down": (w, ff)})
    return out


@functools.lru_cache(maxsize=None)
def folder(which: str, stored: str = "bfloat16") -> str:
    """A model folder (config.json + model.safetensors) of configuration ``which``."""
    from safetensors.torch import save_file

    dtype = {"bfloat16": torch.bfloat16, "float32": torch.float32}[stored]
    path = os.path.join(_TMP.name, f"beno_{which}_{stored}")
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(CONFIGS[which], f)
    made = {name: _draw(name, shape, SEEDS[which]).to(dtype).contiguous() for name, shape in shapes(which).items()}
    save_file(made, os.path.join(path, "model.safetensors"))
    return path


@functools.lru_cache(maxsize=None)
def tensors(which: str, stored: str = "bfloat16") -> dict:
    from safetensors.torch import load_file

    loaded = load_file(os.path.join(folder(which, stored), "model.safetensors"))
    return {k: v.double() for k, v in loaded.items()}


def ids(which: str, n: int, seed: int) -> list[int]:
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, CONFIGS[which]["vocab"], (n,), generator=g).tolist()


_ORACLE: dict = {}


def _oracle(which: str, tokens: list[int], stored: str):
    key = (which, stored, tuple(tokens))
    if key not in _ORACLE:
        margins = []
        logits = PlainBenolix(CONFIGS[which], tensors(which, stored)).forward(tokens, margins=margins)
        _ORACLE[key] = (logits, torch.stack(margins).min(dim=0).values)
    return _ORACLE[key]


def oracle(which: str, tokens: list[int], stored: str = "bfloat16") -> torch.Tensor:
    return _oracle(which, tokens, stored)[0]


def router_margin(which: str, tokens: list[int], stored: str = "bfloat16") -> torch.Tensor:
    """Per token, the least distance over the model's routers between the last output taken and the first left out:
    where it is small, rounding may choose differently."""
    return _oracle(which, tokens, stored)[1]


def core(which: str, dtype: str, ops, device: str, num_pages: int = 64, max_num_seqs: int = 4, page_size: int = 16,
         graph_sizes=None, stored: str = "bfloat16"):
    from atom_amd.engine.core import TORCH_DTYPES, build_core, load_model

    model, _ = load_model(folder(which, stored), dtype=TORCH_DTYPES[dtype], device=device)
    return build_core(model, ops, dtype=TORCH_DTYPES[dtype], device=device, page_size=page_size, num_pages=num_pages,
                      max_num_seqs=max_num_seqs, max_model_len=num_pages * page_size, graph_sizes=graph_sizes)


_TMP = tempfile.TemporaryDirectory(prefix="atom_amd_benolix_")
