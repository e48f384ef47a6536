"""Plain CPU forward pass of the Takosun design: one function per mechanism, the whole sequence at once.

Test infrastructure only.  Everything is computed in float64 with no cache, no batching and no
reordering of the products (the product path absorbs the key and value up-projections into the query
and the output when it decodes; here keys and values are always formed).  ``weights`` maps tensor names
to arrays; names and configuration keys are those of the checkpoint format.
"""
from __future__ import annotations

import math

import numpy as np


def rms_norm(x, w, eps):
    """y_i = w_i x_i / sqrt(mean_i x_i^2 + eps), over the last axis."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def grouped_rms_norm(x, w, eps, groups):
    """The vector is cut into `groups` consecutive parts that are scaled one by one; w covers the whole."""
    parts = x.reshape(x.shape[:-1] + (groups, x.shape[-1] // groups))
    scaled = parts / np.sqrt(np.mean(parts * parts, axis=-1, keepdims=True) + eps)
    return scaled.reshape(x.shape) * w


def silu(z):
    return z / (1.0 + np.exp(-z))


def rotate_half(x, positions, base):
    """x [..., T, R]: component i turns with component i + R/2 by positions * base^(-2 i / R)."""
    half = x.shape[-1] // 2
    freq = np.array([base ** (-2.0 * i / (2 * half)) for i in range(half)])
    angle = np.asarray(positions, np.float64)[:, None] * freq[None, :]
    c, s = np.cos(angle), np.sin(angle)
    u, v = x[..., :half], x[..., half:]
    return np.concatenate([u * c - v * s, v * c + u * s], axis=-1)


def latent_of(h, mixer, tensor, eps, positions):
    """What a layer with its own down-projection caches per token: (normed latent, rotated shared key part)."""
    rank = mixer["kv_rank"]
    both = h @ tensor("dkv").T
    return (rms_norm(both[:, :rank], tensor("dkv.norm"), eps),
            rotate_half(both[:, rank:], positions, mixer["rot"]["base"]))


def causal_softmax(scores):
    """scores [T, T] -> weights; row i sees columns 0..i."""
    T = scores.shape[0]
    out = np.zeros_like(scores)
    for i in range(T):
        e = np.exp(scores[i, :i + 1] - scores[i, :i + 1].max())
        out[i, :i + 1] = e / e.sum()
    return out


def latent_attention(h, mixer, tensor, eps, positions, latent):
    """h [T, width] and the (latent, rotated key) pair of this or an earlier layer -> [T, width]."""
    T = h.shape[0]
    H, D, R, V = mixer["heads"], mixer["dim"], mixer["rot_dim"], mixer["vdim"]
    c, k_rot = latent
    q = (rms_norm(h @ tensor("dq").T, tensor("dq.norm"), eps) @ tensor("uq").T).reshape(T, H, D + R)
    keys = (c @ tensor("uk").T).reshape(T, H, D)
    values = (c @ tensor("uv").T).reshape(T, H, V)
    gate = 1.0 / (1.0 + np.exp(-(h @ tensor("g").T)))
    heads = []
    for a in range(H):
        q_rot = rotate_half(q[:, a, D:], positions, mixer["rot"]["base"])
        scores = (q[:, a, :D] @ keys[:, a].T + q_rot @ k_rot.T) * mixer["scale"]
        heads.append(causal_softmax(scores) @ values[:, a] * gate[:, a:a + 1])
    return np.concatenate(heads, axis=1) @ tensor("o").T


def gated_ff(h, tensor, prefix=""):
    return (silu(h @ tensor(prefix + "gate").T) * (h @ tensor(prefix + "up").T)) @ tensor(prefix + "down").T


def table_moe(h, ids, mlp, tensor):
    """Every token id has its experts in a table; they count equally.  A shared expert is added."""
    top = mlp["router"]["top"]
    out = np.zeros_like(h)
    table = tensor("table").astype(np.int64)
    for t, token in enumerate(ids):
        for e in table[token]:
            out[t] += gated_ff(h[t:t + 1], tensor, f"e{e}.")[0] / top
    if mlp.get("shared"):
        out += gated_ff(h, tensor, "shared.")
    return out


def depth_average(states, coefficients):
    """sum_j coefficients[j] * states[j]"""
    out = np.zeros_like(states[0])
    for a, x in zip(coefficients, states):
        out += a * x
    return out


class TakosunOracle:
    def __init__(self, config: dict, weights: dict):
        self.cfg = config
        self.w = {k: np.asarray(v, np.float64) for k, v in weights.items()}

    def forward(self, ids, layer_states: list | None = None):
        """token ids of one sequence -> logits [T, vocab]; appends the stream after every layer to layer_states."""
        cfg, w = self.cfg, self.w
        eps, groups = cfg["norm"]["eps"], cfg["norm"]["groups"]
        ids = [int(i) for i in ids]
        positions = np.arange(len(ids))
        x = w["embed"][ids]
        states, latents = [x], {}
        for i, layer in enumerate(cfg["layers"]):
            def tensor(name, part, i=i):
                return w[f"l{i}.{part}{name}"]

            def norm(v, name):
                return grouped_rms_norm(v, tensor(name, ""), eps, groups)

            mixer = layer["mixer"]
            mix = lambda name: tensor(name, "mix.")  # noqa: E731
            h = norm(x, "norm1")
            if mixer.get("kv_from") is None:
                latents[i] = latent_of(h, mixer, mix, eps, positions)
                source = i
            else:
                source = mixer["kv_from"]
            x = x + norm(latent_attention(h, mixer, mix, eps, positions, latents[source]), "norm1b")
            mlp = layer.get("mlp")
            if mlp is not None:
                ff = lambda name: tensor(name, "mlp.")  # noqa: E731
                h = norm(x, "norm2")
                y = gated_ff(h, ff) if mlp["kind"] == "dense" else table_moe(h, ids, mlp, ff)
                x = x + norm(y, "norm2b")
            states.append(x)
            x = depth_average(states, tensor("dwa", ""))
            if layer_states is not None:
                layer_states.append(x)
        return grouped_rms_norm(x, w["final.norm"], eps, groups) @ w["head"].T


def greedy(oracle: TakosunOracle, prompt, n_new):
    """The whole sequence again for every token: slow and without a cache."""
    ids, out = list(prompt), []
    for _ in range(n_new):
        out.append(int(np.argmax(oracle.forward(ids)[-1])))
        ids.append(out[-1])
    return out


def random_weights(config: dict, seed: int, bf16=True) -> dict:
    """Seeded weights of the format's shapes, kept at a size that lets every mechanism show in the logits."""
    rng = np.random.default_rng(seed)
    W, V = config["width"], config["vocab"]
    out = {}

    def lin(name, n, k, gain=1.0):
        out[name] = rng.standard_normal((n, k)) * (gain / math.sqrt(k))

    def vec(name, n):
        out[name] = 1.0 + 0.2 * rng.standard_normal(n)

    out["embed"] = rng.standard_normal((V, W))
    for i, layer in enumerate(config["layers"]):
        p, m, mlp = f"l{i}.", layer["mixer"], layer.get("mlp")
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if mlp is not None else ()):
            vec(p + n, W)
        H, D, R, VD, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
        lin(p + "mix.dq", m["q_rank"], W)
        vec(p + "mix.dq.norm", m["q_rank"])
        lin(p + "mix.uq", H * (D + R), m["q_rank"], 1.5)
        if m.get("kv_from") is None:
            lin(p + "mix.dkv", rank + R, W)
            vec(p + "mix.dkv.norm", rank)
        lin(p + "mix.uk", H * D, rank, 1.5)
        lin(p + "mix.uv", H * VD, rank)
        lin(p + "mix.g", H, W, 2.0)
        lin(p + "mix.o", W, H * VD)
        if mlp is not None:
            def ff(q, n):
                lin(q + "gate", n, W)
                lin(q + "up", n, W)
                lin(q + "down", W, n)

            if mlp["kind"] == "dense":
                ff(p + "mlp.", mlp["ff"])
            else:
                E, top = mlp["router"]["experts"], mlp["router"]["top"]
                for e in range(E):
                    ff(p + f"mlp.e{e}.", mlp["expert"]["ff"])
                out[p + "mlp.table"] = np.stack([rng.permutation(E)[:top] for _ in range(V)]).astype(np.int32)
                if mlp.get("shared"):
                    ff(p + "mlp.shared.", mlp["shared"]["ff"])
        out[p + "dwa"] = rng.standard_normal(i + 2) * 0.4
        out[p + "dwa"][-1] += 0.8
    vec("final.norm", W)
    lin("head", V, W)
    if bf16:
        for k, a in out.items():
            if a.dtype != np.int32:
                out[k] = round_bf16(a)
    return out


def bf16_bits(a) -> np.ndarray:
    """float array -> uint16 bfloat16 patterns, round to nearest even."""
    u = np.ascontiguousarray(a, np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)


def round_bf16(a) -> np.ndarray:
    return (bf16_bits(a).astype(np.uint32) << 16).view(np.float32).reshape(np.shape(a))
