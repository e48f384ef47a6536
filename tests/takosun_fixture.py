"""Small configurations of the Takosun design and a writer of its checkpoint format."""
import json
import os
import struct

import numpy as np

from oracle import takosun_forward as tf


def mixer(heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, base=500.0, kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale,
         "rot": {"base": base, "dims": rot_dim}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return m


def layer(mix, mlp):
    return {"type": "latent_attention", "mixer": mix, "mlp": mlp}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, shared=None):
    out = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}
    if shared:
        out["shared"] = {"ff": shared}
    return out


def config(vocab, width, groups, layers, eps=1e-5):
    return {"architecture": "Takosun", "vocab": vocab, "width": width, "norm": {"groups": groups, "eps": eps}, "layers": layers}


# layers of different sizes, two that read one cache, one without a feed-forward, several experts per token
SMALL = config(151, 96, 3, [
    layer(mixer(3, 24, 8, 40, 36, 56, 0.21), moe(5, 2, 48, shared=80)),
    layer(mixer(5, 16, 8, 24, 20, 56, 0.17, kv_from=0), None),
    layer(mixer(2, 32, 24, 16, 64, 88, 0.13, base=90.0), dense(130)),
    layer(mixer(4, 8, 8, 8, 12, 56, 0.3, kv_from=0), moe(7, 3, 33)),
])
# nothing is a multiple of anything
ODD = config(97, 55, 5, [
    layer(mixer(1, 5, 2, 7, 9, 11, 0.4), dense(17)),
    layer(mixer(3, 3, 6, 1, 1, 13, 0.5, base=37.0), moe(3, 1, 5, shared=3)),
    layer(mixer(2, 9, 2, 3, 4, 11, 0.6, kv_from=0), moe(4, 4, 7)),
], eps=0.01)
# one group, one layer; many heads, wide latents
WIDE = config(300, 256, 1, [
    layer(mixer(20, 32, 16, 64, 112, 256, 0.15), moe(8, 2, 64, shared=192)),
    layer(mixer(12, 48, 64, 32, 128, 512, 0.1, base=10000.0), dense(320)),
    layer(mixer(33, 16, 16, 24, 96, 256, 0.2, kv_from=0), dense(192)),
])
# latents past the matrix-core attention's sizes
HUGE_LATENT = config(64, 64, 2, [layer(mixer(2, 8, 8, 16, 16, 640, 0.3), dense(64))])
# rows that the row kernels hold in registers, with idle threads; and rows too long for that
LONG_ROWS = config(43, 1100, 5, [layer(mixer(1, 8, 8, 8, 16, 24, 0.4), moe(2, 1, 16, shared=24)),
                                 layer(mixer(1, 8, 8, 8, 16, 24, 0.4, kv_from=0), dense(40))])
LONGER_ROWS = config(43, 4200, 1, [layer(mixer(1, 8, 8, 8, 16, 24, 0.4), dense(40)),
                                   layer(mixer(2, 8, 8, 8, 16, 24, 0.4, kv_from=0), moe(2, 2, 16))])


def write_model(root, cfg, weights):
    """config.json and model.safetensors: bfloat16 tensors, int32 tables."""
    os.makedirs(root, exist_ok=True)
    with open(os.path.join(root, "config.json"), "w") as f:
        json.dump(cfg, f)
    header, blobs, at = {}, [], 0
    for name, a in weights.items():
        kind = "I32" if a.dtype == np.int32 else "BF16"
        raw = a.tobytes() if kind == "I32" else tf.bf16_bits(a).tobytes()
        header[name] = {"dtype": kind, "shape": list(a.shape), "data_offsets": [at, at + len(raw)]}
        blobs.append(raw)
        at += len(raw)
    text = json.dumps(header).encode()
    with open(os.path.join(root, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(text)) + text + b"".join(blobs))
