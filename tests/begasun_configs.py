"""Small Begasun configurations for the tests, and model folders made from them with random weights."""
import functools
import json
import os
import tempfile

import plain_begasun as P


def latent(heads, dim, rot_dim, vdim, kv_rank, scale=None, base=1000.0, scaling=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank,
         "scale": scale if scale is not None else 2.0 * (dim + rot_dim) ** -0.5}
    if rot_dim:
        m["rot"] = {"dims": rot_dim, "base": base}
        if scaling is not None:
            m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return ("latent_attention", m)


def rglru(width, blocks, conv):
    return ("rglru", {"width": width, "blocks": blocks, "conv": conv})


def attention(heads, kv_heads, dim, vdim, rot_dims=0, base=1000.0, scale=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale if scale is not None else 2.0 * dim ** -0.5}
    if rot_dims:
        m["rot"] = {"dims": rot_dims, "base": base}
    return ("attention", m)


def config(vocab, width, layers, eps=1e-5, embed_scale=None, logit_scale=None, loop=None, side=0):
    """layers: ((type, mixer), (ff, limit) or None)."""
    out = {"architecture": "Begasun", "vocab": vocab, "width": width, "norm": {"eps": eps},
           "layers": [{"type": t, "mixer": m, "mlp": {"kind": "dense", "ff": f[0], "limit": f[1]} if f else None} for (t, m), f in layers]}
    if embed_scale is not None:
        out["embedding"] = {"scale": embed_scale}
    if logit_scale is not None:
        out["logit_scale"] = logit_scale
    if loop is not None:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    if side:
        out["token_side"] = {"dim": side}
    return out


CONFIGS = {
    # sizes that are no multiples of 16 (the plain kernels in both precisions): three heads over one kv head, values
    # larger than keys, stretched frequencies, blocks of 12 channels, the last two layers run three times, a layer without
    # feed-forward
    "a": config(97, 72, [
        (attention(3, 1, 24, 40, rot_dims=10, base=300.0), (48, 0.7)),
        (latent(3, 14, 6, 10, 20, base=100.0, scaling=(4.0, 24, 8.0, 1.0)), None),
        (rglru(36, 3, 4), (56, 2.0))], embed_scale=3.0, logit_scale=0.3, loop=(1, 3, 3), side=10),
    # sizes the matrix-core kernels take: keys and values of one size, a latent of 64 + 32, blocks of 32 channels, two taps,
    # the span in the middle run twice, a recurrent layer first
    "b": config(256, 128, [
        (rglru(128, 4, 2), (96, 1.0)),
        (latent(4, 40, 32, 24, 64, base=10000.0, scaling=(8.0, 64, 4.0, 1.0)), (64, 3.0)),
        (attention(4, 2, 64, 64, rot_dims=32), None),
        (rglru(192, 2, 4), None)], embed_scale=0.5, logit_scale=2.0, loop=(1, 3, 2), side=16),
    # no loop, no token side, no multipliers, no rotation, one head, one tap (no history), blocks of one channel
    "c": config(130, 96, [
        (rglru(40, 40, 1), (40, 1.0)),
        (attention(1, 1, 64, 16), None),
        (latent(1, 32, 0, 48, 16), (64, 0.5))]),
    # the whole model run twice from the first layer, a width that is no multiple of 8, one odd block, five taps, one
    # entry of token input a layer
    "d": config(51, 44, [
        (latent(2, 5, 2, 7, 9, base=50.0), (20, 1.0)),
        (rglru(21, 1, 5), None),
        (attention(2, 2, 6, 10, rot_dims=2, base=10.0), (12, 0.2))], embed_scale=6.0, loop=(0, 3, 2), side=1),
    # keys and values of two sizes on the matrix cores, eight heads over two, one pass of a span of one layer
    "e": config(300, 192, [
        (attention(8, 2, 64, 32, rot_dims=64, base=500.0), (128, 1.5)),
        (rglru(96, 1, 3), (64, 1.0)),
        (latent(6, 64, 32, 32, 32, base=5000.0, scaling=(2.0, 100, 16.0, 2.0)), None)], embed_scale=2.0, logit_scale=1.0,
        loop=(1, 2, 1), side=24),
}


@functools.lru_cache(maxsize=None)
def tensors_of(name, seed=0):
    return P.random_model(CONFIGS[name], seed)


_dirs = {}


def write_model(cfg, tensors, prefix="begasun_"):
    from pico_vllm_amd.weights.safetensors_io import write_safetensors
    d = tempfile.mkdtemp(prefix=prefix)
    with open(os.path.join(d, "config.json"), "w") as f:
        json.dump(cfg, f)
    write_safetensors(os.path.join(d, "model.safetensors"), [(n, tuple(v.shape), v.dtype) for n, v in tensors.items()],
                      lambda n: tensors[n])
    return d


def model_dir(name, seed=0):
    """A folder with config.json and model.safetensors of configuration ``name``; made once a process."""
    key = (name, seed)
    if key not in _dirs:
        _dirs[key] = write_model(CONFIGS[name], tensors_of(name, seed), f"begasun_{name}_")
    return _dirs[key]
