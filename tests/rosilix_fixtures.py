"""Small Rosilix configurations with random bfloat16 weights: config.json + model.safetensors in a directory for the engine, and the same
weights as float64 arrays for the oracle (tests/rosilix_oracle.py)."""
import numpy as np

from tests import rosilix_oracle as orc
from tests.gelarax_oracle import bf16_round
from tests.layered_fixtures import rel_err, write_model_dir      # noqa: F401  (the directory writer and the error measure are shared test helpers)


def dense(ff=40):
    return {"kind": "dense", "ff": ff}


def attention_layer(heads=4, kv_heads=2, dim=12, vdim=20, chunk=37, rot_dims=8, base=1000.0, scale=None, diff=0.3, mlp="default"):
    mx = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": float(scale if scale is not None else 1.4 * dim ** -0.5), "diff": diff,
          "rot": {"base": base, "dims": rot_dims} if rot_dims else None, "mask": {"size": chunk} if chunk else None}
    return {"type": "attention", "mixer": mx, "mlp": dense() if mlp == "default" else mlp}


def latent_layer(heads=3, dim=20, rot_dim=8, vdim=12, kv_rank=28, base=10000.0, scale=None, kv_from=None, mlp="default"):
    mx = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "rot": {"base": base, "dims": rot_dim},
          "scale": float(scale if scale is not None else 1.3 * (dim + rot_dim) ** -0.5)}
    if kv_from is not None:
        mx["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": mx, "mlp": dense(52) if mlp == "default" else mlp}


def config(layers, width=64, vocab=97, eps=1e-5, embed_scale=3.5):
    return {"architecture": "Rosilix", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": layers, "embedding": {"scale": embed_scale}}


def tensor_shapes(cfg):
    W, V = cfg["width"], cfg["vocab"]
    s = {"embed": (V, W), "final.norm": (W,), "head": (V, W)}
    for li, L in enumerate(cfg["layers"]):
        p, m = "l%d." % li, L["mixer"]
        s.update({p + "norm1": (W,), p + "norm1b": (W,)})
        if L["type"] == "latent_attention":
            H, dn, dr, dv, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
            s.update({p + "mix.q": (H * (dn + dr), W), p + "mix.uk": (H * dn, R), p + "mix.uv": (H * dv, R), p + "mix.sink": (H,), p + "mix.g": (H, W), p + "mix.o": (W, H * dv)})
            if m.get("kv_from") is None:
                s.update({p + "mix.dkv": (R + dr, W), p + "mix.dkv.norm": (R,)})
        else:
            H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            s.update({p + "mix.q": (H * 2 * d, W), p + "mix.k": (G * 2 * d, W), p + "mix.v": (G * dv, W), p + "mix.g": (H, W), p + "mix.o": (W, H * dv)})
            s.update({p + "mix." + n: (d,) for n in ("lq1", "lk1", "lq2", "lk2")})
        if L.get("mlp"):
            s.update({p + "norm2": (W,), p + "norm2b": (W,), p + "mlp.up": (L["mlp"]["ff"], W), p + "mlp.down": (W, L["mlp"]["ff"])})
    return s


def random_weights(cfg, seed=0):
    """name -> float32 array of bfloat16-representable values"""
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        leaf = name.split(".")[-1]
        if leaf in ("norm1", "norm2", "norm1b", "norm2b", "norm"):
            a = 1.0 + 0.3 * rng.standard_normal(shape)
        elif leaf in ("lq1", "lk1", "lq2", "lk2"):
            a = rng.standard_normal(shape) * (0.8 / shape[0] ** 0.25)
        elif leaf == "sink":
            a = rng.uniform(-2.0, 4.0, shape)
        elif name == "embed":
            a = 0.4 * rng.standard_normal(shape)
        else:
            a = rng.standard_normal(shape) * (1.2 / np.sqrt(shape[-1]))
        out[name] = bf16_round(np.asarray(a, dtype=np.float32))
    return out


def oracle_weights(weights):
    return {k: orc.f64(v) for k, v in weights.items()}
