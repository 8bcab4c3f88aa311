"""Small Lasivik configurations and random weights for the tests (plain dicts and tensors, nothing of the product)."""
import math

import torch


def latent(heads=3, dim=32, vdim=24, kv_rank=40, window=20, scale=None):
    return dict(type="latent_attention", mixer=dict(heads=heads, dim=dim, vdim=vdim, kv_rank=kv_rank,
                                                    mask=dict(size=window), scale=dim ** -0.5 if scale is None else scale))


def gla(heads=3, dim=24, vdim=40, tau=8.0):
    return dict(type="gla", mixer=dict(heads=heads, dim=dim, vdim=vdim, tau=tau))


def retention(heads=2, dim=48, vdim=32, dims=32, base=10000.0, decay=None):
    decay = [1 - 2.0 ** -(3 + 2 * i) for i in range(heads)] if decay is None else decay
    return dict(type="retention", mixer=dict(heads=heads, dim=dim, vdim=vdim, rot=dict(dims=dims, base=base), decay=decay))


def config(layers, width=72, vocab=100, ff=104, alpha=2.0, eps=1e-5, embedding_scale=None, logit_scale=0.75, cap=20.0):
    """`layers`: the dicts above; a layer's feed-forward is `ff` unless it brings its own 'mlp' entry."""
    full = []
    for layer in layers:
        layer = dict(layer)
        layer.setdefault("mlp", dict(kind="dense", ff=ff))
        full.append(layer)
    return dict(architecture="Lasivik", vocab=vocab, width=width, layers=full, norm=dict(eps=eps), postln_alpha=alpha,
                embedding=dict(scale=math.sqrt(width) if embedding_scale is None else embedding_scale),
                logit_scale=logit_scale, logit_softcap=cap)


def weights(cfg, seed=0, decay_rank=6, sharp=3.0, decay_bias=2.0):
    """Random bf16 weights under the checkpoint's names.  `sharp` scales queries, so that softmax weights and recalled
    keys stand out of the average; `decay_bias` shifts the decay gates (larger: slower decay)."""
    g = torch.Generator()
    g.manual_seed(seed)
    D, V = cfg["width"], cfg["vocab"]
    r = lambda rows, cols, s=1.0: (torch.randn(rows, cols, generator=g) * s / math.sqrt(cols)).bfloat16()
    gain = lambda n, around=0.0: (around + 0.2 * torch.randn(n, generator=g)).bfloat16()
    W = {"embed": torch.randn(V, D, generator=g).bfloat16(), "final.norm": gain(D), "head": r(V, D, 3.0)}
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}.mix."
        nq, nv = m["heads"] * m["dim"], m["heads"] * m["vdim"]
        W[p + "q"] = r(nq, D, sharp)
        W[p + "o"] = r(D, nv)
        if layer["type"] == "latent_attention":
            R = m["kv_rank"]
            W.update({p + "dkv": r(R, D), p + "dkv.norm": gain(R, 1.0), p + "uk": r(nq, R), p + "uv": r(nv, R)})
        else:
            W.update({p + "k": r(nq, D), p + "v": r(nv, D), p + "g": r(nv, D)})
            if layer["type"] == "gla":
                W.update({p + "a1": r(decay_rank, D, 2.0), p + "a2": r(nq, decay_rank, 2.0),
                          p + "a2.b": (decay_bias + torch.randn(nq, generator=g)).bfloat16(), p + "norm": gain(m["vdim"], 1.0)})
        W[f"l{i}.norm1"] = gain(D)
        if layer["mlp"] is not None:
            I, p = layer["mlp"]["ff"], f"l{i}.mlp."
            W.update({p + "gate": r(I, D), p + "up": r(I, D), p + "down": r(D, I), f"l{i}.norm2": gain(D)})
    return W


def tokens(cfg, n, seed=0):
    g = torch.Generator()
    g.manual_seed(1000 + seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


# name -> (configuration, keyword arguments of weights())
CASES = {
    # every mixer, sizes that differ from one another everywhere
    "mixed": (config([latent(), gla(), retention(), latent(heads=2, dim=16, vdim=48, kv_rank=24, window=33)]), {}),
    # sizes no kernel is built for: nothing is a multiple of 8 or of 4
    "odd": (config([gla(heads=3, dim=13, vdim=9, tau=1.0), retention(heads=3, dim=22, vdim=18, dims=10),
                    latent(heads=5, dim=19, vdim=11, kv_rank=21, window=7)], width=45, vocab=67, ff=51, alpha=1.0),
            dict(decay_rank=5)),
    # equal sizes and constants that are 1; a layer without a feed-forward; windows of one token and wider than any prompt
    "plain": (config([latent(heads=1, dim=32, vdim=32, kv_rank=32, window=1, scale=1.0),
                      dict(gla(heads=1, dim=32, vdim=32, tau=1.0), mlp=None),
                      retention(heads=1, dim=32, vdim=32, dims=32, decay=[1.0]),
                      latent(heads=4, dim=64, vdim=64, kv_rank=64, window=4096)], width=64, vocab=64, ff=64, alpha=1.0,
                     embedding_scale=1.0, logit_scale=1.0), dict(decay_rank=8)),
    # gates so steep that a chunk's decay leaves the range of one fp32 factor; a head that forgets at once
    "steep": (config([gla(heads=2, dim=32, vdim=64, tau=0.125), retention(heads=3, dim=32, vdim=32, decay=[0.0, 0.05, 0.999])],
                     width=64), dict(decay_bias=-1.0)),
    # head sizes of real models
    "large": (config([latent(heads=4, dim=128, vdim=128, kv_rank=256, window=70), gla(heads=2, dim=128, vdim=256, tau=16.0),
                      retention(heads=2, dim=256, vdim=128, dims=64, base=500000.0)], width=256, vocab=320, ff=384, alpha=3.0),
              dict(decay_rank=16)),
}
