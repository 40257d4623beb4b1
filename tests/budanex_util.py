"""Small Budanex configurations for the tests (config.json form), model folders with random weights,
and the plain implementation's logits for them."""

from __future__ import annotations

import json
from pathlib import Path

from safetensors.torch import load_file, save_file

import plain_budanex as plain


def attention(heads, kv_heads, dim, vdim, rot_dims, *, base=1000.0, scale=0.3, softcap=5.0):
    sizes = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "rot": {"dims": rot_dims, "base": base}}
    if softcap is not None:
        sizes["softcap"] = softcap
    return "attention", sizes


def mamba(heads, vdim, state, groups, conv, norm_groups):
    return "mamba2", {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": norm_groups}


def latent(heads, dim, rot_dim, vdim, kv_rank, window, *, base=500.0, scale=0.4, scaling=(4.0, 64, 8.0, 1.0), rot_dims=None):
    rot = {"dims": rot_dim if rot_dims is None else rot_dims, "base": base}
    if scaling is not None:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    sizes = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale, "rot": rot}
    if window is not None:
        sizes["mask"] = {"size": window}
    return "latent_attention", sizes


def layer(mixer, ff):
    return {"type": mixer[0], "mixer": mixer[1], "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(vocab, width, layers, loop=None, *, eps=1e-5, cap=6.0):
    raw = {"architecture": "Budanex", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if cap is not None:
        raw["logit_softcap"] = cap
    if loop is not None:
        raw["loop"] = dict(zip(("start", "stop", "times"), loop))
    return raw


# every mixer, with a feed-forward and without; layers ahead of and behind the loop, three passes; groups of two; part of
# the head turned; values wider and narrower than keys; a window a little over two pages
SMALL_A = config(90, 40, [
    layer(attention(4, 2, 12, 8, 6), 28),
    layer(latent(3, 10, 6, 12, 14, 9), None),
    layer(mamba(4, 10, 6, 2, 4, 4), 20),
    layer(attention(2, 1, 8, 20, 8, base=50.0, softcap=2.0), None),
    layer(mamba(6, 4, 9, 3, 2, 1), None),
], (1, 4, 3))
# the loop begins with the first layer and ends with the last, one pass; a window of one; one tap, one group; a kv head
# per head; no cap on scores or logits; plain frequencies
SMALL_B = config(64, 24, [
    layer(latent(2, 6, 4, 5, 9, 1, scaling=None), 16),
    layer(attention(3, 3, 6, 6, 2, softcap=None), None),
    layer(mamba(2, 16, 17, 1, 1, 1), 40),
], (0, 3, 1), eps=1e-3, cap=None)
# no loop; no window; latents alone; a query head of one plain dim; part of the rotated part turned; sizes that fit no vector load
SMALL_C = config(70, 18, [
    layer(latent(5, 1, 8, 3, 7, None, scaling=(16.0, 4096, 32.0, 1.0), rot_dims=6), 10),
    layer(latent(1, 7, 2, 9, 11, 23), None),
], cap=3.0)
# the loop ends with the last layer; many heads on one kv head; windows of two layers that differ, one shorter than a page
SMALL_D = config(100, 32, [
    layer(mamba(4, 8, 1, 4, 3, 2), 24),
    layer(attention(9, 1, 16, 16, 16), 16),
    layer(latent(4, 8, 4, 8, 12, 3), 16),
    layer(latent(4, 8, 4, 8, 12, 17, base=20.0), None),
], (1, 4, 4))
# sizes that the matrix-core attention kernels take on the GPU, filled up or as they are; windows over several key tiles
MEDIUM = config(320, 256, [
    layer(attention(8, 2, 64, 64, 32, scale=0.2, softcap=20.0), 384),
    layer(latent(8, 48, 32, 40, 100, 70, scale=0.15, base=10000.0), 256),
    layer(mamba(8, 64, 64, 2, 4, 2), None),
    layer(attention(4, 1, 96, 48, 96, scale=0.15, softcap=8.0, base=10000.0), None),
    layer(latent(4, 64, 64, 64, 128, 33, scale=0.12), 192),
], (1, 4, 2), cap=12.0)
CONFIGS = {"A": SMALL_A, "B": SMALL_B, "C": SMALL_C, "D": SMALL_D}
BLOCK_SIZE = {"A": 4, "B": 8, "C": 2, "D": 8}


def write_model(raw: dict, seed: int, folder, change=None) -> Path:
    """A model folder with random weights; ``change(tensors)`` may edit them before they are written."""
    from forge_engine_amd.config import load_model_config
    from forge_engine_amd.weights import write_random_model

    folder = write_random_model(load_model_config(raw), seed, folder)
    if change is not None:
        path = str(Path(folder) / "model.safetensors")
        tensors = load_file(path)
        change(tensors)
        save_file({name: t.contiguous() for name, t in tensors.items()}, path, metadata={"format": "pt"})
    return folder


ENLARGED = {"float32": 6.0, "bfloat16": 3.0}    # in bfloat16 several passes of the larger ones amplify every rounding


def enlarge(tensors, factor=6.0):
    """Matrices of the layers several times as large, so that every sublayer weighs beside the embedding; logits of a size
    that their cap bends."""
    for name, t in tensors.items():
        if name == "head":
            tensors[name] = (t.float() * 25.0).to(t.dtype)
        if t.dim() == 2 and name.startswith("l") and not name.startswith("loop") and "conv" not in name:
            tensors[name] = (t.float() * factor).to(t.dtype)


def folder_weights(folder) -> tuple[dict, dict]:
    folder = Path(folder)
    return json.loads((folder / "config.json").read_text()), plain.load_weights(folder)


def plain_logits(folder, requests) -> dict:
    """(request, position) -> logits of the plain implementation, for whole requests."""
    cfg, weights = folder_weights(folder)
    want = {}
    for request_id, tokens in requests.items():
        for position, row in enumerate(plain.forward(cfg, weights, tokens)):
            want[(request_id, position)] = row
    return want


def compare(got: dict, want: dict, dtype: str, fraction: float = 0.03, float32_factor: float = 1.0) -> float:
    """Every row the engine wrote against the plain implementation's: float32 to 1e-5 + 1e-4 of the row's largest logit,
    bfloat16 to a fraction of the logits' spread."""
    import torch

    assert got, "no logits were written"
    worst = 0.0
    for key, row in got.items():
        expected = want[key].to(torch.float64)
        assert bool(torch.isfinite(row).all()), f"{key}: non-finite logits"
        diff = float((row.to(torch.float64) - expected).abs().max())
        if dtype == "float32":
            bound = float32_factor * (1e-5 + 1e-4 * float(expected.abs().max()))
        else:
            bound = fraction * float(expected.max() - expected.min())
        assert diff <= bound, f"{key}: off by {diff:.3e} (bound {bound:.3e})"
        worst = max(worst, diff / bound)
    return worst
