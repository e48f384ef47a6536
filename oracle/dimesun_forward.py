"""Plain CPU forward pass of the Dimesun design: one function per mechanism, the whole sequence at once.

Test infrastructure only.  Everything is computed in float64, with no cache; the matrix memory is run token by token, as its
recurrence is written (the product path cuts a prompt into chunks and never forms the state inside one).  ``weights`` maps
tensor names to arrays; names and configuration keys are those of the checkpoint format.
"""
from __future__ import annotations

import math

import numpy as np

from oracle.takosun_forward import bf16_bits, rotate_half, round_bf16  # noqa: F401


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-np.asarray(z, np.float64)))


def unit_rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def norm_around_zero(x, w, eps):
    """The weight is stored as its distance from one."""
    return unit_rms(x, eps) * (1.0 + w)


def soft_cap(z, cap):
    return cap * np.tanh(z / cap)


def log_sigmoid(z):
    return np.where(z >= 0, -np.log1p(np.exp(-np.abs(z))), z - np.log1p(np.exp(-np.abs(z))))


# ---- matrix memory ---------------------------------------------------------------------------

class MatrixMemory:
    """State of one head: S [dim][vdim], n [dim], and the scale m that S and n carry (true values are exp(m) S, exp(m) n)."""

    def __init__(self, dim, vdim):
        self.S, self.n, self.m = np.zeros((dim, vdim)), np.zeros(dim), 0.0

    def step(self, q, k, v, log_in, log_keep):
        m = max(log_keep + self.m, log_in)
        keep, add = math.exp(log_keep + self.m - m), math.exp(log_in - m)
        self.S = keep * self.S + add * np.outer(k, v)
        self.n = keep * self.n + add * k
        self.m = m
        return (self.S.T @ q) / (max(abs(float(self.n @ q)), math.exp(-m)) + 1e-6)


def gates_of(h, mixer, tensor):
    """Per token and head: (log of the input gate, log of the forget gate)."""
    cap = mixer["gate_cap"]
    log_in = soft_cap(h @ tensor("i").T + tensor("i.b"), cap)
    return log_in, log_sigmoid(soft_cap(h @ tensor("f").T + tensor("f.b"), cap))


def mlstm(h, mixer, tensor, eps):
    """h [T, width] -> [T, width]"""
    T, H, D, V = h.shape[0], mixer["heads"], mixer["dim"], mixer["vdim"]
    q = (h @ tensor("q").T).reshape(T, H, D) / math.sqrt(D)
    k = (h @ tensor("k").T).reshape(T, H, D)
    v = (h @ tensor("v").T).reshape(T, H, V)
    log_in, log_keep = gates_of(h, mixer, tensor)
    out = np.empty((T, H, V))
    for a in range(H):
        memory = MatrixMemory(D, V)
        for t in range(T):
            out[t, a] = memory.step(q[t, a], k[t, a], v[t, a], log_in[t, a], log_keep[t, a])
    y = unit_rms(out, eps).reshape(T, H * V) * tensor("norm") * sigmoid(h @ tensor("g").T)
    return y @ tensor("o").T


# ---- attention -------------------------------------------------------------------------------

def rotate_first(x, positions, rot):
    """The first rot.dims components of every head turn, the others stay."""
    dims = rot["dims"]
    return np.concatenate([rotate_half(x[..., :dims], positions, rot["base"]), x[..., dims:]], axis=-1)


def sees(i, j, chunk):
    return j <= i and i // chunk == j // chunk


def sink_softmax(scores):
    """exp(s_j) / (1 + sum exp(s)): a further key of score zero that has no value."""
    top = max(0.0, float(np.max(scores)))
    e = np.exp(scores - top)
    return e / (math.exp(-top) + e.sum())


def attention(h, mixer, tensor, positions):
    T, H, G, D, V = h.shape[0], mixer["heads"], mixer["kv_heads"], mixer["dim"], mixer["vdim"]
    q = (h @ tensor("q").T).reshape(T, H, D)
    k = (h @ tensor("k").T).reshape(T, G, D)
    v = (h @ tensor("v").T).reshape(T, G, V)
    out = np.empty((T, H, V))
    for a in range(H):
        b = a // (H // G)
        qr, kr = rotate_first(q[:, a], positions, mixer["rot"]), rotate_first(k[:, b], positions, mixer["rot"])
        for t in range(T):
            seen = [j for j in range(t + 1) if sees(positions[t], positions[j], mixer["mask"]["size"])]
            out[t, a] = sink_softmax(kr[seen] @ qr[t] * mixer["scale"]) @ v[seen, b]
    return out.reshape(T, H * V) @ tensor("o").T


# ---- experts ---------------------------------------------------------------------------------

def choose(logits, top):
    """One token's router logits -> (expert numbers, weights): softmax over the `top` largest."""
    best = sorted(range(len(logits)), key=lambda e: (-logits[e], e))[:top]
    e = np.exp(logits[best] - logits[best].max())
    return best, e / e.sum()


def clamped_expert(h, tensor, prefix, limit):
    g = np.minimum(h @ tensor(prefix + "gate").T, limit)
    u = np.clip(h @ tensor(prefix + "up").T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ tensor(prefix + "down").T


def routed_experts(h, mlp, tensor, margins=None):
    """margins [T], if given, falls to the distance between the last chosen and the first other logit of a token."""
    logits, top = h @ tensor("router").T + tensor("router.b"), mlp["router"]["top"]
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        if margins is not None and top < logits.shape[1]:
            rising = np.sort(logits[t])
            margins[t] = min(margins[t], rising[-top] - rising[-top - 1])
        for e, w in zip(*choose(logits[t], top)):
            out[t] += w * clamped_expert(h[t], tensor, f"e{e}.", mlp["expert"]["limit"])
    return out


# ---- the model -------------------------------------------------------------------------------

def layer_runs(config):
    """[(layer, pass of the loop it opens or None)] in the order they run."""
    loop = config["loop"]
    runs = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        runs += [(i, t if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
    return runs + [(i, None) for i in range(loop["stop"], len(config["layers"]))]


class DimesunOracle:
    """normed_as: applied to every normed row, for instance round_bf16, to see what rounding alone does to a sequence."""

    def __init__(self, config: dict, weights: dict, normed_as=None):
        self.cfg = config
        self.normed_as = normed_as or (lambda h: h)
        self.w = {k: np.asarray(v, np.float64) for k, v in weights.items()}

    def forward(self, ids, layer_states: list | None = None, margins: np.ndarray | None = None):
        """token ids of one sequence -> logits [T, vocab]; appends the stream after every layer run to layer_states; margins
        [T] falls to the closest call of a router for each token."""
        cfg, w, eps = self.cfg, self.w, self.cfg["norm"]["eps"]
        ids = [int(i) for i in ids]
        positions = np.arange(len(ids))
        x = w["embed"][ids]
        for i, opens in layer_runs(cfg):
            layer = cfg["layers"][i]
            if opens is not None:
                x = x + w["loop.step"][opens]
            h = self.normed_as(norm_around_zero(x, w[f"l{i}.norm1"], eps))
            mix = lambda name, i=i: w[f"l{i}.mix.{name}"]  # noqa: E731
            if layer["type"] == "mlstm":
                y = mlstm(h, layer["mixer"], mix, eps)
            else:
                y = attention(h, layer["mixer"], mix, positions)
            if layer.get("mlp"):
                y = y + routed_experts(h, layer["mlp"], lambda name, i=i: w[f"l{i}.mlp.{name}"], margins)
            x = x + cfg["residual_mult"] * y
            if layer_states is not None:
                layer_states.append(x)
        return self.normed_as(norm_around_zero(x, w["final.norm"], eps)) @ w["embed"].T


def greedy(oracle: DimesunOracle, prompt, n_new):
    """The whole sequence again for every token: slow and without a cache."""
    ids, out = list(prompt), []
    for _ in range(n_new):
        out.append(int(np.argmax(oracle.forward(ids)[-1])))
        ids.append(out[-1])
    return out


def random_weights(config: dict, seed: int, bf16=True) -> dict:
    """Seeded weights of the format's shapes, kept at a size that lets every mechanism show in the logits."""
    rng = np.random.default_rng(seed)
    W = config["width"]
    out = {}

    def lin(name, n, k, gain=1.0):
        out[name] = rng.standard_normal((n, k)) * (gain / math.sqrt(k))

    out["embed"] = rng.standard_normal((config["vocab"], W))
    out["loop.step"] = 0.5 * rng.standard_normal((config["loop"]["times"], W))
    for i, layer in enumerate(config["layers"]):
        p, m, f = f"l{i}.", layer["mixer"], layer.get("mlp")
        H, D, V = m["heads"], m["dim"], m["vdim"]
        out[p + "norm1"] = 0.3 * rng.standard_normal(W)
        mix = p + "mix."
        if layer["type"] == "mlstm":
            lin(mix + "q", H * D, W, 1.5)
            lin(mix + "k", H * D, W)
            # a token's key resembles its query, so that a head's output, which is scaled to size one, is seldom near zero
            out[mix + "k"] = 0.7 * out[mix + "k"] + 0.5 * out[mix + "q"]
            lin(mix + "v", H * V, W)
            lin(mix + "g", H * V, W)
            lin(mix + "o", W, H * V)
            out[mix + "norm"] = 1.0 + 0.3 * rng.standard_normal(H * V)
            lin(mix + "i", H, W, 2.0)
            out[mix + "i.b"] = rng.standard_normal(H)
            lin(mix + "f", H, W, 2.0)
            out[mix + "f.b"] = 2.0 + 2.0 * rng.standard_normal(H)  # some heads remember for long, some forget at once
        else:
            G = m["kv_heads"]
            lin(mix + "q", H * D, W, 2.0)
            lin(mix + "k", G * D, W, 1.5)
            lin(mix + "v", G * V, W, 1.5)
            lin(mix + "o", W, H * V)
        if f:
            E, ff = f["router"]["experts"], f["expert"]["ff"]
            lin(p + "mlp.router", E, W, 2.0)
            out[p + "mlp.router.b"] = 0.5 * rng.standard_normal(E)
            for e in range(E):
                q = p + f"mlp.e{e}."
                lin(q + "gate", ff, W, 1.5)
                lin(q + "up", ff, W, 1.5)
                lin(q + "down", W, ff)
    out["final.norm"] = 0.3 * rng.standard_normal(W)
    return {k: round_bf16(a) for k, a in out.items()} if bf16 else out
