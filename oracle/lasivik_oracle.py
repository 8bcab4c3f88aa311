"""Plain restatement of the Lasivik design (test infrastructure only; shares no code with the product path).

One function per mechanism, token by token where a mechanism is a recurrence, position by position where it is a
window, in whatever dtype the inputs have (the tests use float64).  Weights are a dict keyed by the checkpoint's
tensor names, the configuration is the parsed config.json.

The design: a post-norm decoder whose layers mix tokens in one of three ways -- a gated linear attention with a decay
per key channel, a retention with a fixed decay per head, or a sliding-window attention over a low-rank latent -- and
then apply a gated feed-forward.  The residual is re-normalised after each of the two sums of a layer."""
import math
from typing import Dict, List, Optional

import torch
from torch import Tensor


# ------------------------------------------------------------------------------------------------ pieces

def rms(x: Tensor, eps: float) -> Tensor:
    """x divided by its root mean square over the last dimension; eps is added to the mean square."""
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def zero_centred_norm(x: Tensor, w: Tensor, eps: float) -> Tensor:
    """RMS norm whose stored weight is the gain minus one."""
    return rms(x, eps) * (1 + w)


def silu(z: Tensor) -> Tensor:
    return z / (1 + torch.exp(-z))


def rotate_half(x: Tensor, positions: Tensor, dims: int, base: float) -> Tensor:
    """x [T, heads, dim]: the pairs (i, i + dims/2) of the first `dims` dimensions turned by p * base^(-2i/dims)."""
    out = x.clone()
    half = dims // 2
    for i in range(half):
        f = base ** (-2.0 * i / dims)
        a = positions.to(x.dtype) * f
        c, s = torch.cos(a)[:, None], torch.sin(a)[:, None]
        u, v = x[:, :, i], x[:, :, i + half]
        out[:, :, i] = u * c - v * s
        out[:, :, i + half] = v * c + u * s
    return out


def recurrence(q: Tensor, k: Tensor, v: Tensor, decay: Tensor, state: Optional[Tensor] = None):
    """Linear attention with decay.  q, k, decay [T, H, dk], v [T, H, dv]; state [H, dk, dv] (None: zeros).
    S_t = decay_t (per row of S) * S_{t-1} + k_t v_t^T;  o_t = S_t^T q_t.  Returns (o [T, H, dv], state)."""
    T, H, dk = q.shape
    S = torch.zeros(H, dk, v.shape[-1], dtype=q.dtype) if state is None else state.clone()
    o = torch.empty(T, H, v.shape[-1], dtype=q.dtype)
    for t in range(T):
        S = decay[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = (S * q[t][:, :, None]).sum(1)
    return o, S


def gla_decay(h: Tensor, a1: Tensor, a2: Tensor, bias: Tensor, tau: float) -> Tensor:
    """sigmoid(z)^(1/tau) per key channel, z a rank-limited projection plus bias."""
    z = (h @ a1.T) @ a2.T + bias
    return torch.exp(-torch.log1p(torch.exp(-z.abs())) / tau + torch.clamp(z, max=0) / tau)


def window_mask(q_pos: Tensor, k_pos: Tensor, size: int) -> Tensor:
    """[Tq, Tk] bool: the key is the query's own position or one of the size - 1 before it."""
    d = q_pos[:, None] - k_pos[None, :]
    return (d >= 0) & (d < size)


def windowed_softmax_attention(q: Tensor, k: Tensor, v: Tensor, q_pos: Tensor, k_pos: Tensor, size: int,
                               scale: float) -> Tensor:
    """q [Tq, H, d], k [Tk, H, d], v [Tk, H, dv] -> [Tq, H, dv]."""
    s = torch.einsum("qhd,khd->hqk", q, k) * scale
    s = s.masked_fill(~window_mask(q_pos, k_pos, size)[None], -math.inf)
    return torch.einsum("hqk,khd->qhd", torch.softmax(s, -1), v)


# ------------------------------------------------------------------------------------------------ mixers
# Each takes the layer's input h [T, width], the layer's tensors under `p` + name, its sizes, eps, the position of the
# first token and the state earlier tokens left (None at the start); it returns (output [T, width], new state).

def gla_mixer(h, W, p, m, eps, pos0, state):
    H, dk, dv = m["heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q = (h @ W[p + "q"].T).view(T, H, dk) * dk ** -0.5
    k = (h @ W[p + "k"].T).view(T, H, dk)
    v = (h @ W[p + "v"].T).view(T, H, dv)
    a = gla_decay(h, W[p + "a1"], W[p + "a2"], W[p + "a2.b"], m["tau"]).view(T, H, dk)
    o, S = recurrence(q, k, v, a, state)
    o = rms(o, eps) * W[p + "norm"]
    return (o.reshape(T, H * dv) * silu(h @ W[p + "g"].T)) @ W[p + "o"].T, S


def retention_mixer(h, W, p, m, eps, pos0, state):
    H, dk, dv = m["heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    at = torch.arange(pos0, pos0 + T)
    rot = lambda x: rotate_half(x, at, m["rot"]["dims"], m["rot"]["base"])
    q = rot((h @ W[p + "q"].T).view(T, H, dk))
    k = rot((h @ W[p + "k"].T).view(T, H, dk)) * dk ** -0.5
    v = (h @ W[p + "v"].T).view(T, H, dv)
    a = torch.tensor(m["decay"], dtype=h.dtype)[None, :, None].expand(T, H, dk)
    o, S = recurrence(q, k, v, a, state)
    return (rms(o, eps).reshape(T, H * dv) * silu(h @ W[p + "g"].T)) @ W[p + "o"].T, S


def latent_attention_mixer(h, W, p, m, eps, pos0, state):
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q = (h @ W[p + "q"].T).view(T, H, d)
    c = rms(h @ W[p + "dkv"].T, eps) * W[p + "dkv.norm"]
    c = c if state is None else torch.cat([state, c])          # every latent so far; the mask does the rest
    k = (c @ W[p + "uk"].T).view(-1, H, d)
    v = (c @ W[p + "uv"].T).view(-1, H, dv)
    y = windowed_softmax_attention(q, k, v, torch.arange(pos0, pos0 + T), torch.arange(c.shape[0]), m["mask"]["size"],
                                   m["scale"])
    return y.reshape(T, H * dv) @ W[p + "o"].T, c


MIXERS = {"gla": gla_mixer, "retention": retention_mixer, "latent_attention": latent_attention_mixer}


def feed_forward(h, W, p):
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


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
        self.states: List[Optional[Tensor]] = [None] * len(self.cfg["layers"])
        self.residuals = None

    def step(self, tokens) -> Tensor:
        c, W = self.cfg, self.W
        eps, alpha = c["norm"]["eps"], c["postln_alpha"]
        x = W["embed"][torch.as_tensor(tokens, dtype=torch.long)] * c["embedding"]["scale"]
        seen = []
        for i, layer in enumerate(c["layers"]):
            p = f"l{i}."
            y, self.states[i] = MIXERS[layer["type"]](x, W, p + "mix.", layer["mixer"], eps, self.pos, self.states[i])
            x = zero_centred_norm(alpha * x + y, W[p + "norm1"], eps)
            if layer["mlp"] is not None:
                x = zero_centred_norm(alpha * x + feed_forward(x, W, p + "mlp."), W[p + "norm2"], eps)
            seen.append(x)
        self.pos += x.shape[0]
        self.residuals = torch.stack(seen)
        logits = (zero_centred_norm(x, W["final.norm"], eps) @ W["head"].T) * c["logit_scale"]
        cap = c["logit_softcap"]
        return cap * torch.tanh(logits / cap)

    def greedy(self, prompt, n: int) -> List[int]:
        out = []
        last = self.step(prompt)[-1]
        for _ in range(n):
            out.append(int(last.argmax()))
            last = self.step([out[-1]])[-1]
        return out
