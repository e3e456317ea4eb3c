"""Small Tubusun configurations for the tests, and model folders made from them with random weights."""
import functools

import plain_tubusun as P
from begasun_configs import write_model


def left(heads, kv_heads, dim, vdim, window=0, rot_dims=0, base=1000.0, scale=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale if scale is not None else 2.0 * dim ** -0.5}
    if window:
        m["mask"] = {"size": window}
    if rot_dims:
        m["rot"] = {"dims": rot_dims, "base": base}
    return m


def right(heads, dim, vdim, slowest=0.995):
    """Decays from one that forgets within two tokens to one that keeps hundreds."""
    n = max(1, heads - 1)
    return {"heads": heads, "dim": dim, "vdim": vdim, "decay": [0.5 ** (1 - h / n) * slowest ** (h / n) for h in range(heads)]}


def pair(l, r, left_scale=None, right_scale=None):
    m = {"left": l, "right": r}
    if left_scale is not None:
        m["left_scale"] = left_scale
    if right_scale is not None:
        m["right_scale"] = right_scale
    return m


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(ff, experts, top, limit, groups=None):
    r = {"experts": experts, "top": top}
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": r}


def config(vocab, width, layers, eps=1e-5, embed_scale=None, cap=None, loop=None):
    """layers: (mixer, feed-forward or None)."""
    out = {"architecture": "Tubusun", "vocab": vocab, "width": width, "norm": {"eps": eps},
           "layers": [{"type": "parallel", "mixer": m, "mlp": f} for m, f in layers]}
    if embed_scale is not None:
        out["embedding"] = {"scale": embed_scale}
    if cap is not None:
        out["logit_softcap"] = cap
    if loop is not None:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    return out


CONFIGS = {
    # sizes that are no multiples of 16 (the plain kernels in both precisions): three heads over one kv head, values larger
    # than keys, a window of 21, odd sizes side by side (so that columns are padded), the last two layers run three times, a
    # layer without feed-forward
    "a": config(97, 72, [
        (pair(left(3, 1, 24, 40, window=21, rot_dims=10, base=300.0), right(2, 9, 11), 0.6, 1.5), dense(48)),
        (pair(left(2, 2, 10, 6, window=5, rot_dims=2, base=50.0), right(3, 12, 8)), None),
        (pair(left(4, 2, 12, 12, window=33, rot_dims=12), right(1, 20, 30), 1.3, 0.4), moe(24, 9, 3, 0.7, (3, 2)))],
        embed_scale=3.0, cap=8.0, loop=(1, 3, 3)),
    # sizes the matrix-core kernels take, with keys and values of one size; three of four groups; the span in the middle run
    # twice
    "b": config(256, 128, [
        (pair(left(4, 2, 64, 64, window=48, rot_dims=32), right(2, 64, 64), 0.7, 1.2), moe(64, 16, 4, 1.0, (4, 3))),
        (pair(left(6, 2, 32, 32, window=20, rot_dims=16, base=1e5), right(4, 32, 48), 1.1, 0.9), dense(96)),
        (pair(left(4, 1, 64, 64, window=70, rot_dims=64), right(3, 96, 32), 0.5, 0.5), moe(40, 8, 2, 2.0, (8, 4))),
        (pair(left(2, 1, 32, 32, window=130), right(2, 16, 80)), None)], embed_scale=0.5, cap=20.0, loop=(1, 3, 2)),
    # no loop, no window, no rotation, no groups, no cap, no multipliers, one head, one expert a token
    "c": config(130, 96, [
        (pair(left(1, 1, 64, 16), right(1, 40, 24)), moe(32, 5, 1, 1.5)),
        (pair(left(2, 1, 32, 64), right(2, 8, 16)), dense(40))]),
    # the whole model run twice from the first layer, a width that is no multiple of 8, single entries: a window of one token,
    # values of one entry, groups of one expert
    "d": config(51, 44, [
        (pair(left(2, 1, 6, 10, window=1, rot_dims=2, base=10.0), right(2, 1, 3), 2.0, 0.3), dense(20)),
        (pair(left(3, 3, 7, 1, window=9, rot_dims=4, base=10.0), right(2, 5, 1)), moe(12, 4, 2, 0.3, (4, 2)))],
        embed_scale=6.0, cap=5.0, loop=(0, 2, 2)),
    # keys and values of two sizes on the matrix cores, eight heads over two, twenty over one, one pass of a span of one layer,
    # every group kept, heads of the recurrence beyond 128
    "e": config(300, 192, [
        (pair(left(8, 2, 64, 32, window=100, rot_dims=64, base=500.0), right(2, 160, 96), 0.9, 1.4), dense(128)),
        (pair(left(20, 1, 32, 16, window=64, rot_dims=8), right(6, 24, 40), 1.5, 0.8), moe(56, 12, 5, 1.0, (2, 2)))],
        embed_scale=2.0, cap=30.0, loop=(1, 2, 1)),
}


@functools.lru_cache(maxsize=None)
def tensors_of(name, seed=0):
    return P.random_model(CONFIGS[name], seed)


_dirs = {}


def model_dir(name, seed=0):
    """A folder with config.json and model.safetensors of configuration ``name``; made once a process."""
    key = (name, seed)
    if key not in _dirs:
        _dirs[key] = write_model(CONFIGS[name], tensors_of(name, seed), f"tubusun_{name}_")
    return _dirs[key]
