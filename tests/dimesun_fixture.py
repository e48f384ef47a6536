"""Small configurations of the Dimesun design."""
import numpy as np

from oracle import dimesun_forward as df
from tests.takosun_fixture import write_model  # noqa: F401  (the checkpoint format is the same)

TOL = {"float32": 3e-5, "bfloat16": 0.06}   # relative norms of rows


def row_errors(got, want):
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    return np.linalg.norm(got - want, axis=-1) / np.linalg.norm(want, axis=-1)


class Truth:
    """The oracle on n seeded tokens: logits, the stream after every layer run, and a limit of every token's relative error:
    in bfloat16 at least three times what rounding the normed rows does to the oracle itself (a memory's output near zero may
    make much of it), and five times as much where a router's choice is a close call, which any rounding may turn."""

    def __init__(self, oracle, n, seed=1):
        self.ids = np.random.default_rng(seed).integers(0, oracle.cfg["vocab"], n).astype(np.int32)
        self.states, rounded_states, margins = [], [], np.full(n, np.inf)
        self.logits = oracle.forward(self.ids, self.states, margins)
        rounded = df.DimesunOracle(oracle.cfg, oracle.w, df.round_bf16).forward(self.ids, rounded_states)
        alone = np.max([row_errors(rounded, self.logits)] + [row_errors(a, b) for a, b in zip(rounded_states, self.states)], axis=0)
        self.limits = {"float32": np.full(n, TOL["float32"]), "bfloat16": np.maximum(TOL["bfloat16"], 3 * alone) * np.where(margins < 0.1, 5.0, 1.0)}


def attention(heads, kv_heads, dim, vdim, chunk, scale, rot_dims=None, base=500.0, mlp=None):
    return {"type": "attention", "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": chunk}, "scale": scale,
                      "rot": {"base": base, "dims": dim if rot_dims is None else rot_dims}}}


def mlstm(heads, dim, vdim, gate_cap=15.0, mlp=None):
    return {"type": "mlstm", "mlp": mlp, "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": gate_cap}}


def moe(experts, top, ff, limit=1.0):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff, "limit": limit}}


def config(vocab, width, layers, loop, residual_mult=0.6, eps=1e-5):
    return {"architecture": "Dimesun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": residual_mult,
            "layers": layers, "loop": {"start": loop[0], "stop": loop[1], "times": loop[2]}}


# layers ahead of, inside and behind the loop, all of different sizes, some without a feed-forward; experts are left out only in
# the last layer (sharp attention over a token whose experts rounding has turned spreads far in bfloat16)
SMALL = config(151, 96, [
    mlstm(2, 20, 36, 9.0, mlp=moe(5, 5, 48, 0.8)),
    attention(6, 2, 24, 40, 20, 0.4, rot_dims=16, mlp=moe(7, 7, 33, 1.5)),
    mlstm(3, 12, 16, mlp=None),
    attention(2, 2, 16, 8, 33, 0.5, base=90.0, mlp=None),
    attention(3, 1, 40, 24, 48, 0.3, mlp=moe(4, 1, 130)),
], (1, 4, 3))
# nothing is a multiple of anything; a loop that runs once; all experts chosen
ODD = config(97, 55, [
    attention(3, 1, 5, 7, 9, 0.6, rot_dims=2, base=37.0, mlp=moe(3, 3, 5, 0.5)),
    mlstm(1, 3, 5, 4.0, mlp=moe(3, 1, 17)),
    attention(3, 3, 9, 1, 11, 0.5, rot_dims=6, mlp=None),
    mlstm(5, 7, 2, mlp=None),
], (0, 2, 1), residual_mult=1.0, eps=0.01)
# everything in the loop; more columns and experts
WIDE = config(300, 256, [
    attention(12, 4, 64, 32, 70, 0.2, rot_dims=32, base=10000.0, mlp=moe(40, 5, 64)),
    mlstm(3, 96, 160, mlp=moe(9, 9, 40, 2.0)),
], (0, 2, 2))
# the larger tiles of the kernels, and a chunk of one position
LARGE = config(64, 128, [
    attention(4, 2, 136, 144, 50, 0.1, rot_dims=136, mlp=moe(3, 2, 48)),
    mlstm(2, 130, 300, mlp=None),
    attention(2, 1, 72, 128, 1, 0.2, mlp=None),
    mlstm(1, 68, 260, mlp=moe(2, 1, 24)),
], (1, 3, 2), residual_mult=0.4)
# heads and memories past the matrix-core kernels' sizes
HUGE = config(64, 64, [attention(2, 1, 264, 16, 30, 0.06, mlp=moe(2, 1, 24)), mlstm(1, 16, 520, mlp=moe(3, 2, 8)),
                       attention(2, 2, 8, 264, 13, 0.3, mlp=None)], (2, 3, 2))
# rows that the row kernels do not hold in registers, and too long for the one-token pass
LONG_ROWS = config(43, 4200, [attention(1, 1, 8, 8, 6, 0.4, mlp=moe(2, 1, 16)), mlstm(1, 8, 8, mlp=moe(2, 2, 16))], (0, 1, 2))
MANY_VALUES = config(43, 64, [mlstm(40, 8, 400, mlp=moe(2, 1, 16)), attention(3, 1, 8, 8, 6, 0.4, mlp=None)], (1, 2, 2), eps=0.1)
