"""Plain restatement of the Gepolix design (test infrastructure only; shares no code with the product path).

One function per mechanism, token by token where a mechanism is a recurrence, expert by expert where tokens are routed, in
whatever dtype the inputs have (the tests use float64).  Weights are a dict keyed by the checkpoint's tensor names, the
configuration is the parsed config.json.

The design: a decoder whose layers read one normalised input with both of their sublayers and add both to the residual.
The norm is a scaled tanh.  Tokens are mixed by a selective state space (Mamba-2) or by grouped-query attention through a
sliding window, whose keys and values another layer may use as well; the feed-forward is dense or a mixture of experts."""
import math
from typing import Dict, List

import torch
from torch import Tensor

from .lasivik_oracle import feed_forward, rms, rotate_half, silu, window_mask


# ------------------------------------------------------------------------------------------------ pieces

def dynamic_tanh(x: Tensor, alpha: Tensor, w: Tensor, b: Tensor) -> Tensor:
    return torch.tanh(alpha * x) * w + b


def softplus(z: Tensor) -> Tensor:
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


def causal_conv(u: Tensor, w: Tensor, b: Tensor, before: Tensor) -> Tensor:
    """u [T, C], w [C, taps]: out[t] = b + sum_j w[:, j] u[t - (taps - 1) + j]; `before` [taps - 1, C] are the inputs ahead
    of u's first row."""
    taps = w.shape[1]
    ext = torch.cat([before, u])
    out = b.expand(u.shape).clone()
    for j in range(taps):
        out = out + w[:, j] * ext[j:j + u.shape[0]]
    return out


def selective_scan(x: Tensor, B: Tensor, C: Tensor, dt: Tensor, A_log: Tensor, state: Tensor):
    """x [T, H, P], B and C [T, G, N], dt [T, H] (positive), state [H, N, P].
    S_t = exp(-exp(A_log) dt_t) S_(t-1) + dt_t B_t x_t^T;  y_t = S_t^T C_t.  Returns (y [T, H, P], state)."""
    T, H, P = x.shape
    G = B.shape[1]
    S = state.clone()
    y = torch.empty_like(x)
    for t in range(T):
        for h in range(H):
            g = h // (H // G)
            S[h] = torch.exp(-torch.exp(A_log[h]) * dt[t, h]) * S[h] + dt[t, h] * torch.outer(B[t, g], x[t, h])
            y[t, h] = S[h].T @ C[t, g]
    return y, S


def parts_norm(y: Tensor, parts: int, eps: float) -> Tensor:
    """Each of `parts` equal ranges of the last dimension divided by its own root mean square."""
    return rms(y.view(*y.shape[:-1], parts, -1), eps).reshape(y.shape)


def grouped_window_attention(q: Tensor, k: Tensor, v: Tensor, pos0: int, size: int, scale: float) -> Tensor:
    """q [T, H, d] at positions pos0 ..; k [Tk, G, d], v [Tk, G, dv] at positions 0 ..; query head h reads head h // (H / G)."""
    T, H, _ = q.shape
    G = k.shape[1]
    see = window_mask(torch.arange(pos0, pos0 + T), torch.arange(k.shape[0]), size)
    out = q.new_empty(T, H, v.shape[-1])
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * scale
        out[:, h] = torch.softmax(s.masked_fill(~see, -math.inf), -1) @ v[:, g]
    return out


def route(h: Tensor, router: Tensor, bias: Tensor, top: int):
    """Chosen experts [T, top] and their weights: the largest logits, softmax over the chosen ones."""
    z = h @ router.T + bias
    val, idx = torch.topk(z, top, dim=-1)
    return idx, torch.softmax(val, -1)


def mixture(h: Tensor, W: Dict[str, Tensor], p: str, mlp: dict) -> Tensor:
    idx, w = route(h, W[p + "router"], W[p + "router.b"], mlp["router"]["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, we in zip(idx[t].tolist(), w[t]):
            out[t] += we * feed_forward(h[t:t + 1], W, f"{p}e{e}.")[0]
    if mlp.get("shared") is not None:
        gate = 1 / (1 + torch.exp(-(h @ W[p + "shared.sg"].T)))
        out = out + gate * feed_forward(h, W, p + "shared.")
    return out


# ------------------------------------------------------------------------------------------------ mixers
# Each takes the layer's input h [T, width], the layer's tensors under `p` + name, its sizes, eps, the position of the
# first token, what earlier tokens left (None at the start) and, for attention, the cache of the layer whose keys and
# values it uses instead of its own (None: its own); it returns (output [T, width], what it leaves).

def mamba2_mixer(h, W, p, m, eps, pos0, state, lent):
    H, P, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner, T = H * P, h.shape[0]
    z, xBC, dt = (h @ W[p + "in"].T).split([inner, inner + 2 * G * N, H], dim=-1)
    if state is None:
        state = (h.new_zeros(W[p + "conv"].shape[1] - 1, xBC.shape[1]), h.new_zeros(H, N, P))
    before, S = state
    u = silu(causal_conv(xBC, W[p + "conv"], W[p + "conv.b"], before))
    after = torch.cat([before, xBC])[T:]
    x, B, C = u.split([inner, G * N, G * N], dim=-1)
    x = x.view(T, H, P)
    y, S = selective_scan(x, B.view(T, G, N), C.view(T, G, N), softplus(dt + W[p + "dt_bias"]), W[p + "A_log"], S)
    y = (y + W[p + "D"][:, None] * x).reshape(T, inner)
    return (parts_norm(y * silu(z), m["norm_groups"], eps) * W[p + "norm"]) @ W[p + "o"].T, (after, S)


def attention_mixer(h, W, p, m, eps, pos0, state, lent):
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    rot = lambda t: rotate_half(t, torch.arange(pos0, pos0 + T), m["rot"]["dims"], m["rot"]["base"])
    q = rot((h @ W[p + "q"].T + W[p + "q.b"]).view(T, H, d))
    if lent is None:
        k = rot((h @ W[p + "k"].T + W[p + "k.b"]).view(T, G, d))
        v = (h @ W[p + "v"].T + W[p + "v.b"]).view(T, G, dv)
        state = (k, v) if state is None else (torch.cat([state[0], k]), torch.cat([state[1], v]))
        lent = state
    y = grouped_window_attention(q, *lent, pos0, m["mask"]["size"], m["scale"])
    return y.reshape(T, H * dv) @ W[p + "o"].T, state


MIXERS = {"mamba2": mamba2_mixer, "attention": attention_mixer}


# ------------------------------------------------------------------------------------------------ the model

class Oracle:
    """Feeds one sequence in portions: `step(tokens)` -> logits [len(tokens), vocab]; `.residuals` holds the residual
    stream after every layer of the last step [layers, T, width]."""

    def __init__(self, config: dict, weights: Dict[str, Tensor], dtype=torch.float64):
        self.cfg = config
        self.W = {k: v.to(dtype) for k, v in weights.items()}
        self.reset()

    def reset(self):
        self.pos = 0
        self.states: List = [None] * len(self.cfg["layers"])
        self.residuals = None

    def _norm(self, x, name):
        return dynamic_tanh(x, self.W[name + ".alpha"], self.W[name], self.W[name + ".b"])

    def step(self, tokens) -> Tensor:
        c, W = self.cfg, self.W
        eps = c["norm"]["eps"]
        x = W["embed"][torch.as_tensor(tokens, dtype=torch.long)]
        seen = []
        for i, layer in enumerate(c["layers"]):
            h = self._norm(x, f"l{i}.norm1")
            j = layer["mixer"].get("kv_from")
            y, self.states[i] = MIXERS[layer["type"]](h, W, f"l{i}.mix.", layer["mixer"], eps, self.pos, self.states[i],
                                                      None if j is None else self.states[j])
            mlp = layer["mlp"]
            if mlp is not None:
                y = y + (mixture(h, W, f"l{i}.mlp.", mlp) if mlp["kind"] == "moe" else feed_forward(h, W, f"l{i}.mlp."))
            x = x + y
            seen.append(x)
        self.pos += x.shape[0]
        self.residuals = torch.stack(seen)
        return self._norm(x, "final.norm") @ W["head"].T

    def greedy(self, prompt, n: int) -> List[int]:
        out = []
        last = self.step(prompt)[-1]
        for _ in range(n):
            out.append(int(last.argmax()))
            last = self.step([out[-1]])[-1]
        return out
