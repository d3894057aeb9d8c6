"""Small Kamelorn configurations with random bfloat16 weights: config.json + model.safetensors in a directory for the engine, and the same
weights as float64 arrays for the oracle (tests/kamelorn_oracle.py)."""
import numpy as np

from tests import kamelorn_oracle as orc
from tests.gelarax_oracle import bf16_round
from tests.layered_fixtures import rel_err, write_model_dir      # noqa: F401  (the directory writer and the error measure are shared test helpers)


def dense(ff=40):
    return {"kind": "dense", "ff": ff}


def moe(experts=6, top=2, ff=24, scale=1.5):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top, "scale": scale}}


def latent_layer(heads=3, dim=20, rot_dim=8, vdim=12, kv_rank=28, base=10000.0, scale=None, mlp="default"):
    mx = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "rot": {"base": base, "dims": rot_dim},
          "scale": float(scale if scale is not None else 1.3 * (dim + rot_dim) ** -0.5)}
    return {"type": "latent_attention", "mixer": mx, "mlp": dense() if mlp == "default" else mlp}


def ssm_layer(heads=6, vdim=8, state=12, groups=3, conv=4, norm_groups=2, mlp="default"):
    return {"type": "mamba2", "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": norm_groups},
            "mlp": moe() if mlp == "default" else mlp}


def config(layers, width=64, vocab=97, eps=1e-5, embed_scale=2.5, mult=0.4, streams=3, loop=None):
    cfg = {"architecture": "Kamelorn", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": layers, "embedding": {"scale": embed_scale}, "residual_mult": mult,
           "streams": streams}
    if loop:
        cfg["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return cfg


def tensor_shapes(cfg):
    W, V, S = cfg["width"], cfg["vocab"], cfg["streams"]
    s = {"embed": (V, W), "final.norm": (W,), "head": (V, W)}
    for li, L in enumerate(cfg["layers"]):
        p, m = "l%d." % li, L["mixer"]
        s.update({p + "norm1": (W,), p + "hc1.in": (S,), p + "hc1.out": (S,), p + "hc1.mix": (S, S)})
        if L["type"] == "latent_attention":
            H, dn, dr, dv, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
            s.update({p + "mix.q": (H * (dn + dr), W), p + "mix.dkv": (R + dr, W), p + "mix.dkv.norm": (R,), p + "mix.uk": (H * dn, R), p + "mix.uv": (H * dv, R),
                      p + "mix.g": (H * dv, W), p + "mix.o": (W, H * dv)})
        else:
            H, inner = m["heads"], m["heads"] * m["vdim"]
            C = inner + 2 * m["groups"] * m["state"]
            s.update({p + "mix.in": (inner + C + H, W), p + "mix.conv": (C, m["conv"]), p + "mix.conv.b": (C,), p + "mix.dt_bias": (H,), p + "mix.A_log": (H,), p + "mix.D": (H,),
                      p + "mix.norm": (inner,), p + "mix.o": (W, inner)})
        mlp = L.get("mlp")
        if not mlp:
            continue
        s.update({p + "norm2": (W,), p + "hc2.in": (S,), p + "hc2.out": (S,), p + "hc2.mix": (S, S)})
        if mlp["kind"] == "dense":
            s.update({p + "mlp.gate": (mlp["ff"], W), p + "mlp.up": (mlp["ff"], W), p + "mlp.down": (W, mlp["ff"])})
            continue
        E, F = mlp["router"]["experts"], mlp["expert"]["ff"]
        s[p + "mlp.router"] = (E, W)
        for e in range(E):
            s.update({p + "mlp.e%d.gate" % e: (F, W), p + "mlp.e%d.up" % e: (F, W), p + "mlp.e%d.down" % e: (W, F)})
    return s


def random_weights(cfg, seed=0):
    """name -> float32 array of bfloat16-representable values (gains small enough that a dozen layer runs do not amplify fp32 rounding beyond the tests' tolerances)"""
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        leaf, part = name.split(".")[-1], name.split(".")[-2] if "." in name else ""
        if part in ("hc1", "hc2"):
            if leaf == "mix":
                a = np.eye(shape[0]) + 0.12 * rng.standard_normal(shape)          # (near the identity: the first layers still count at the end)
            else:
                a = 0.6 + 0.3 * rng.standard_normal(shape)
        elif leaf in ("norm1", "norm2", "norm"):
            a = 1.0 + 0.3 * rng.standard_normal(shape)
        elif leaf == "A_log":
            a = rng.uniform(-3.0, 1.0, shape)
        elif leaf == "dt_bias":
            a = rng.uniform(-3.0, 0.5, shape)
        elif leaf == "D":
            a = 0.5 + 0.7 * rng.standard_normal(shape)
        elif leaf == "b":
            a = 0.3 * rng.standard_normal(shape)
        elif leaf == "conv":
            a = 0.6 * rng.standard_normal(shape)
        elif leaf == "router":
            a = rng.standard_normal(shape) * (3.0 / np.sqrt(shape[-1]))
        elif name == "embed":
            a = rng.standard_normal(shape) * 0.5
        else:
            a = rng.standard_normal(shape) * (1.0 / np.sqrt(shape[-1]))
        out[name] = bf16_round(np.asarray(a, dtype=np.float32))
    return out


def oracle_weights(weights):
    return {k: orc.f64(v) for k, v in weights.items()}
