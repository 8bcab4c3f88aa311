"""Small Gepolix configurations and random weights for the tests (plain dicts and tensors, nothing of the product)."""
import math

import torch


def ssm(heads=4, vdim=24, state=20, groups=2, norm_groups=2, conv=4, **layer):
    return dict(type="mamba2", mixer=dict(heads=heads, vdim=vdim, state=state, groups=groups, norm_groups=norm_groups, conv=conv), **layer)


def attention(heads=6, kv_heads=2, dim=32, vdim=24, window=20, dims=24, base=10000.0, scale=None, kv_from=None, **layer):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, mask=dict(size=window), rot=dict(dims=dims, base=base),
             scale=dim ** -0.5 if scale is None else scale)
    if kv_from is not None:
        m["kv_from"] = kv_from
    return dict(type="attention", mixer=m, **layer)


def moe(experts=7, top=2, ff=24, shared=40):
    d = dict(kind="moe", router=dict(experts=experts, top=top), expert=dict(ff=ff))
    return d if shared is None else dict(d, shared=dict(ff=shared))


def config(layers, width=72, vocab=100, ff=104, eps=1e-5):
    """`layers`: the dicts above; a layer's feed-forward is a dense one of `ff` unless it brings its own 'mlp' entry."""
    full = [dict(layer, mlp=layer["mlp"] if "mlp" in layer else dict(kind="dense", ff=ff)) for layer in layers]
    return dict(architecture="Gepolix", vocab=vocab, width=width, layers=full, norm=dict(eps=eps))


def weights(cfg, seed=0, sharp=3.0, a_log=0.0, dt_bias=-1.0):
    """Random bf16 weights under the checkpoint's names.  `sharp` scales queries, so that softmax weights and recalled keys stand
    out of the average; a_log and dt_bias shift how fast states forget."""
    g = torch.Generator()
    g.manual_seed(seed)
    D, V = cfg["width"], cfg["vocab"]
    r = lambda rows, cols, s=1.0: (torch.randn(rows, cols, generator=g) * s / math.sqrt(cols)).bfloat16()
    vec = lambda n, around=0.0, s=0.2: (around + s * torch.randn(n, generator=g)).bfloat16()
    W = {"embed": torch.randn(V, D, generator=g).bfloat16(), "head": r(V, D, 3.0)}

    def norm(name):
        W.update({name: vec(D, 1.0), name + ".b": vec(D), name + ".alpha": (0.4 + 0.3 * torch.rand((), generator=g)).bfloat16()})

    def ff(p, I):
        W.update({p + "gate": r(I, D), p + "up": r(I, D), p + "down": r(D, I)})

    norm("final.norm")
    for i, layer in enumerate(cfg["layers"]):
        m, p, mlp = layer["mixer"], f"l{i}.mix.", layer["mlp"]
        norm(f"l{i}.norm1")
        H, nv = m["heads"], m["heads"] * m["vdim"]
        W[p + "o"] = r(D, nv)
        if layer["type"] == "mamba2":
            C = nv + 2 * m["groups"] * m["state"]
            W.update({p + "in": r(nv + C + H, D), p + "conv": vec(C * m["conv"], 0.0, 0.6).view(C, -1), p + "conv.b": vec(C),
                      p + "dt_bias": vec(H, dt_bias, 1.0), p + "A_log": vec(H, a_log, 1.0), p + "D": vec(H, 1.0), p + "norm": vec(nv, 1.0)})
        else:
            nk, nkv = m["kv_heads"] * m["dim"], m["kv_heads"] * m["vdim"]
            W.update({p + "q": r(H * m["dim"], D, sharp), p + "q.b": vec(H * m["dim"], 0.0, 0.5)})
            if "kv_from" not in m:
                W.update({p + "k": r(nk, D), p + "k.b": vec(nk, 0.0, 0.5), p + "v": r(nkv, D), p + "v.b": vec(nkv, 0.0, 0.5)})
        p = f"l{i}.mlp."
        if mlp is not None and mlp["kind"] == "dense":
            ff(p, mlp["ff"])
        elif mlp is not None:
            E = mlp["router"]["experts"]
            W.update({p + "router": r(E, D, 3.0), p + "router.b": vec(E, 0.0, 0.5)})
            for e in range(E):
                ff(f"{p}e{e}.", mlp["expert"]["ff"])
            if "shared" in mlp:
                ff(p + "shared.", mlp["shared"]["ff"])
                W[p + "shared.sg"] = r(1, D, 2.0)
    return {k: v.contiguous() for k, v in W.items()}


def tokens(cfg, n, seed=0):
    g = torch.Generator()
    g.manual_seed(1000 + seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


# name -> (configuration, keyword arguments of weights())
CASES = {
    # every branch, sizes that differ from one another everywhere; a layer that borrows keys under another window, one that has
    # no feed-forward, mixtures with and without a shared expert
    "mixed": (config([ssm(), attention(), ssm(heads=6, vdim=16, state=32, groups=3, norm_groups=1, conv=2, mlp=moe()),
                      attention(kv_from=1, window=33, scale=0.25, mlp=moe(experts=4, top=3, ff=32, shared=None)), ssm(mlp=None)]), {}),
    # nothing is a multiple of 8 or of 4; norm parts that cut heads
    "odd": (config([ssm(heads=4, vdim=9, state=13, groups=1, norm_groups=3, conv=3), attention(heads=3, kv_heads=3, dim=19, vdim=11, window=7, dims=10),
                    ssm(heads=2, vdim=7, state=5, groups=2, norm_groups=1, conv=2, mlp=moe(experts=5, top=3, ff=13, shared=9)),
                    attention(heads=3, kv_heads=3, dim=19, vdim=11, window=5, dims=10, kv_from=1)], width=45, vocab=67, ff=51), {}),
    # equal sizes and counts that are 1; windows of one token and wider than any prompt
    "plain": (config([ssm(heads=1, vdim=32, state=32, groups=1, norm_groups=1, conv=1),
                      attention(heads=1, kv_heads=1, dim=32, vdim=32, window=1, dims=32, scale=1.0, mlp=moe(experts=1, top=1, ff=32, shared=32)),
                      attention(heads=4, kv_heads=1, dim=64, vdim=64, window=4096, dims=2), ssm(heads=2, vdim=16, state=16, groups=2, norm_groups=2, conv=8)],
                     width=64, vocab=64, ff=64), {}),
    # heads that forget at once beside heads that hardly forget
    "steep": (config([ssm(heads=4, vdim=32, state=32, groups=4, norm_groups=4), ssm(heads=3, vdim=16, state=16, groups=1, norm_groups=1)], width=64),
              dict(a_log=3.0, dt_bias=2.0)),
    # head sizes of real models; more query heads per kv head than a tile has columns
    "large": (config([ssm(heads=4, vdim=64, state=128, groups=2, norm_groups=2), attention(heads=8, kv_heads=2, dim=128, vdim=128, window=70, dims=128, base=500000.0),
                      ssm(heads=2, vdim=128, state=64, groups=1, norm_groups=1, mlp=moe(experts=12, top=4, ff=64, shared=128)),
                      attention(heads=20, kv_heads=1, dim=64, vdim=48, window=100, dims=32)], width=256, vocab=320, ff=384), dict(a_log=-2.0)),
    # more experts than a wave has lanes, nearly all of them used
    "experts": (config([attention(mlp=moe(experts=70, top=9, ff=16, shared=None)), ssm(mlp=moe(experts=66, top=66, ff=8, shared=16))], width=64), {}),
}
