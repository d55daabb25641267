"""Small Zamitar configurations, random weights and checkpoints shared by the tests."""
import torch

import zamitar_oracle as oracle
from docagents_amd.models import make_decoder
from docagents_amd.models.configs import checkpoint_config
from seq_cases import checkpoint, row_errors

# rms error of a row of logits / rms of the logits
TOL = {"fp32": 3e-5, "bf16": 1e-2}
TOL16 = {"ones": 3e-2}  # norms over five channels


def delta(heads, kv, dim, vdim, conv=4):
    return "channel_delta", {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv}


def latent(heads, dim, rot, vdim, q_rank, kv_rank, base=1000.0, scale=None):
    return "latent_attention", {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "q_rank": q_rank,
                                "kv_rank": kv_rank, "rot": {"base": base, "dims": rot},
                                "scale": scale or (dim + rot) ** -0.5}


def config(width, vocab, layers, loop=None, eps=3e-5, scale=3.0):
    """layers: (mixer, ff or None); loop: (start, stop, times)."""
    out = [{"type": kind, "mixer": mixer, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}
           for (kind, mixer), ff in layers]
    c = {"architecture": "Zamitar", "width": width, "vocab": vocab, "embedding": {"scale": scale}, "norm": {"eps": eps},
         "layers": out}
    return {**c, "loop": dict(zip(("start", "stop", "times"), loop))} if loop else c


CONFIGS = {
    # no width a multiple of a tile, query / key heads shared, layers without feed-forward, a loop in the middle
    "odd": config(90, 203, [(latent(5, 24, 8, 40, 36, 50), None), (delta(6, 2, 20, 28, 3), 100),
                            (latent(3, 12, 20, 16, 70, 33), 52), (delta(4, 4, 40, 72, 2), None)], loop=(1, 3, 3)),
    # one head, one tap, one rotated pair, no loop (no norm over one channel: its sign would flip on rounding)
    "ones": config(64, 97, [(delta(1, 1, 32, 64, 1), 64), (latent(1, 32, 2, 32, 6, 5), None), (delta(2, 1, 4, 6, 2), 33)],
                   eps=1e-3, scale=1.0),
    # wide heads and latents, many query heads, everything looped
    "wide": config(130, 151, [(delta(6, 3, 128, 96, 6), 96), (latent(20, 128, 64, 128, 96, 300), 80)], loop=(0, 2, 2)),
    # heads and latents wider than the matrix-core kernels take
    "huge": config(72, 120, [(latent(3, 200, 100, 140, 40, 530, base=77.0, scale=0.07), 48), (delta(2, 1, 290, 24), None),
                             (latent(17, 40, 6, 24, 24, 60), 32)]),
    # a loop of one pass at the end
    "deep": config(96, 110, [(delta(2, 2, 64, 48), 64), (latent(4, 32, 16, 32, 48, 64), 64), (delta(3, 1, 32, 32), 64)],
                   loop=(2, 3, 1)),
}


def weights(cfg, seed=0, dtype=torch.bfloat16):
    """Random tensors by the names and shapes a checkpoint of this configuration has."""
    g = torch.Generator().manual_seed(seed)
    h, out = cfg["width"], {}

    def put(name, *shape, std=None, mean=0.0):
        std = shape[-1] ** -0.5 if std is None else std
        out[name] = (mean + std * torch.randn(shape, generator=g)).to(dtype)
    put("embed", cfg["vocab"], h, std=1.0)
    if cfg.get("loop"):
        put("loop.step", cfg["loop"]["times"], h, std=0.5)
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.mix.", layer["mixer"]
        put(f"l{i}.norm1", h, mean=1.0, std=0.2)
        put(f"l{i}.ls1", h, mean=0.7, std=0.3)
        H, D, V = m["heads"], m["dim"], m["vdim"]
        if layer["type"] == "channel_delta":
            G = m["kv_heads"]
            for k, n in (("q", G * D), ("k", G * D), ("v", H * V)):
                put(p + k, n, h), put(p + k + ".conv", n, m["conv"])
            put(p + "b", H, h, std=2 * h ** -0.5), put(p + "A_log", H, mean=0.0, std=0.7), put(p + "norm", V, mean=1.0, std=0.3)
            ra, rg = 7 + i, 18 + 5 * i
            put(p + "a1", ra, h), put(p + "a2", H * D, ra), put(p + "dt_bias", H * D, mean=-2.5, std=1.5)
            put(p + "g1", rg, h), put(p + "g2", H * V, rg), put(p + "o", h, H * V)
        else:
            R, L, Q = m["rot_dim"], m["kv_rank"], m["q_rank"]
            put(p + "dq", Q, h), put(p + "dq.norm", Q, mean=1.0, std=0.3), put(p + "uq", H * (D + R), Q, std=2 * Q ** -0.5)
            put(p + "dkv", L + R, h, std=1.5 * h ** -0.5), put(p + "dkv.norm", L, mean=1.0, std=0.3), put(p + "uk", H * D, L)
            put(p + "uv", H * V, L), put(p + "sink", H, mean=1.0, std=1.0), put(p + "g", H * V, h), put(p + "o", h, H * V)
        if layer["mlp"]:
            f = layer["mlp"]["ff"]
            put(f"l{i}.ls2", h, mean=-0.5, std=0.3)
            for k, shape in (("gate", (f, h)), ("up", (f, h)), ("down", (h, f))):
                put(f"l{i}.mlp.{k}", *shape), put(f"l{i}.mlp.{k}.b", shape[0], std=0.5)
    put("final.norm", h, mean=1.0, std=0.2)
    return out


def build(tmp_path, name, device, dtype, seed=0, edit=None):
    """(model loaded from a checkpoint folder, config, weights); edit(weights) may change them first."""
    cfg = CONFIGS[name] if isinstance(name, str) else name
    w = weights(cfg, seed)
    if edit:
        edit(w)
    return make_decoder(checkpoint_config(checkpoint(tmp_path, cfg, w)), device, dtype=dtype), cfg, w


def check(got, want, dtype, what=""):
    e = row_errors(got, want)
    tol = TOL16.get(what.split(":")[0].split(" ")[0], TOL[dtype]) if dtype == "bf16" else TOL[dtype]
    assert e.max() < tol, f"{what}: position {int(e.argmax())} of {len(e)} is off by {float(e.max()):.3g}"


def expect(cfg, w, toks):
    return oracle.forward(cfg, w, toks)[0]
