"""Small Talapel configurations for the tests (config.json form), model folders with random weights,
and the plain implementation's logits for them."""

from __future__ import annotations

import json
from pathlib import Path

import torch
from safetensors.torch import load_file, save_file

import plain_talapel as plain


def side(heads, kv_heads, dim, vdim, right, *, scale=0.3, softcap=5.0, coef=0.7, every=9, left_scale=0.8, right_scale=1.3):
    """A ``parallel`` mixer; ``right``: (heads, vdim, state, groups, conv, norm_groups)."""
    keys = ("heads", "vdim", "state", "groups", "conv", "norm_groups")
    return "parallel", {"left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "softcap": softcap,
                                 "q_temp": {"coef": coef, "every": every}},
                        "right": dict(zip(keys, right)), "left_scale": left_scale, "right_scale": right_scale}


def retention(heads, dim, vdim, rot_dims, *, base=1000.0, decay=None):
    return "retention", {"heads": heads, "dim": dim, "vdim": vdim, "rot": {"dims": rot_dims, "base": base},
                         "decay": decay or [1.0 - 2.0 ** -(2 + h) for h in range(heads)]}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}


def layer(mixer, mlp):
    return {"type": mixer[0], "mixer": mixer[1], "mlp": mlp}


def config(vocab, width, layers, loop=None, *, eps=1e-5, scale=1.0):
    raw = {"architecture": "Talapel", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
           "layers": layers}
    if loop is not None:
        raw["loop"] = dict(zip(("start", "stop", "times"), loop))
    return raw


# both mixers and feed-forwards, a layer without one, layers ahead of and behind the loop, three passes; groups of two;
# part of the head rotated in one layer, all of it in the other; values wider and narrower than keys
SMALL_A = config(90, 40, [
    layer(retention(3, 12, 8, 6), dense(28)),
    layer(side(4, 2, 8, 12, (4, 10, 6, 2, 4, 4)), moe(5, 2, 20)),
    layer(retention(2, 8, 20, 8, base=50.0), moe(3, 3, 12)),
    layer(side(2, 1, 14, 6, (6, 4, 9, 3, 2, 1), softcap=2.0, every=4, coef=-0.2), None),
    layer(retention(4, 10, 10, 2), None),
], (1, 4, 3), scale=3.0)
# the loop begins with the first layer and one pass is all; one tap (no convolution state), one group, one norm part;
# one expert a token; a kv head per head; negative factors
SMALL_B = config(64, 24, [
    layer(side(3, 3, 6, 6, (2, 16, 17, 1, 1, 1), left_scale=-0.5, right_scale=2.0, every=1, coef=0.3), moe(4, 1, 16)),
    layer(retention(1, 18, 7, 18, decay=[1.0]), dense(40)),
], (0, 2, 1), eps=1e-3, scale=0.5)
# no loop at all; recurrent layers alone (no keys or values are cached); sizes that fit no vector load
SMALL_C = config(70, 18, [
    layer(retention(2, 7, 5, 4), dense(10)),
    layer(retention(3, 9, 3, 6), None),
])
# the loop ends with the last layer and comes behind a first; attention mixers only; state sizes 1
SMALL_D = config(100, 32, [
    layer(side(4, 1, 16, 16, (4, 8, 1, 4, 3, 2)), dense(24)),
    layer(side(2, 2, 4, 10, (2, 6, 5, 2, 8, 3), softcap=30.0, every=100), dense(16)),
], (1, 2, 4))
# sizes that the matrix-core attention and the grouped products' full tiles take on the GPU; chunks and segments of
# the recurrences with vector loads
MEDIUM = config(320, 256, [
    layer(side(8, 2, 64, 64, (8, 64, 64, 2, 4, 2), scale=0.2, softcap=20.0, every=50), dense(384)),
    layer(retention(4, 64, 128, 64, base=10000.0), moe(6, 2, 160)),
    layer(side(4, 1, 128, 128, (4, 96, 128, 1, 4, 4), scale=0.1, softcap=8.0, every=33), moe(3, 1, 96)),
    layer(retention(2, 128, 96, 96), dense(256)),
], (0, 3, 2), scale=4.0)
CONFIGS = {"A": SMALL_A, "B": SMALL_B, "C": SMALL_C, "D": SMALL_D}
BLOCK_SIZE = {"A": 4, "B": 8, "C": 2, "D": 2}


def write_model(raw: dict, seed: int, folder, change=None) -> Path:
    """A model folder with random weights; ``change(tensors)`` may edit them before they are written."""
    from forge_engine_amd.config import load_model_config
    from forge_engine_amd.weights import write_random_model

    folder = write_random_model(load_model_config(raw), seed, folder)
    path = str(Path(folder) / "model.safetensors")
    tensors = load_file(path)
    # the stream passes ``loop.in`` several times and matrices drawn small would leave nothing of it: half of the
    # stream and half of the embedding's output, plus the noise
    if "loop.in" in tensors:
        width = tensors["loop.in"].shape[0]
        eye = torch.eye(width)
        tensors["loop.in"] = (tensors["loop.in"].float() + torch.cat([0.6 * eye, 0.4 * eye], dim=1)).to(tensors["loop.in"].dtype)
    if change is not None:
        change(tensors)
    save_file({name: t.contiguous() for name, t in tensors.items()}, path, metadata={"format": "pt"})
    return folder


ENLARGED = {"float32": 6.0, "bfloat16": 3.0}    # in bfloat16 several passes of the larger ones amplify every rounding


def enlarge(tensors, factor=6.0):
    """Matrices of the layers several times as large, so that every sublayer weighs beside the embedding."""
    for name, t in tensors.items():
        if t.dim() == 2 and t.is_floating_point() and name.startswith("l") and not name.startswith("loop") and "conv" not in name:
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
    """Every row the engine wrote against the plain implementation's: float32 to 1e-5 + 1e-4 of the row's largest logit.
    bfloat16: 96 rows in a hundred to a fraction of the logits' spread and every row to half of it (a head of a
    retention layer whose read-out is small ahead of its unit norm amplifies the rounding of q, k and v: the kernels'
    references in bfloat16 show the same rows, up to 0.3 of the spread)."""
    assert got, "no logits were written"
    worst, far = 0.0, 0
    for key, row in got.items():
        expected = want[key].to(torch.float64)
        assert bool(torch.isfinite(row).all()), f"{key}: non-finite logits"
        diff = float((row.to(torch.float64) - expected).abs().max())
        if dtype == "float32":
            bound = float32_factor * (1e-5 + 1e-4 * float(expected.abs().max()))
        else:
            bound = 0.5 * float(expected.max() - expected.min())
        assert diff <= bound, f"{key}: off by {diff:.3e} (bound {bound:.3e})"
        worst = max(worst, diff / bound)
        far += dtype != "float32" and diff > fraction * float(expected.max() - expected.min())
    assert far <= max(2, 0.04 * len(got)), f"{far} of {len(got)} rows are off by more than {fraction} of their spread"
    return worst
