"""Small Minerax models, engines around them and helpers of the schedule tests."""
import torch

from replisense_rfq_amd.engine.engine import LLMEngine
from replisense_rfq_amd.models.config import minerax_from_json
from replisense_rfq_amd.models.minerax import MineraxLM
from replisense_rfq_amd.models.weights import init_minerax_weights, minerax_from_full
from replisense_rfq_amd.utils.config import EngineConfig
from tests.livisun.common import alone, run_schedule, tokens  # noqa: F401  (schedule driver)

from . import oracle


def dense(ff):
    return {"kind": "dense", "ff": ff}


def yarn(factor=3.0, original=40, fast=8.0, slow=1.0):
    return {"factor": factor, "original": original, "fast": fast, "slow": slow}


def _rot(dims, base, scaling):
    rot = {"base": base, "dims": dims}
    if scaling is not None:
        rot["scaling"] = scaling
    return rot


def left(heads, kv_heads, dim, vdim, conv, rot_dims, softcap=5.0, scale=0.4, base=700.0, scaling=None):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv, "scale": scale,
            "softcap": softcap, "rot": _rot(rot_dims, base, scaling)}


def right(heads, kv_heads, dim, vdim, conv):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}


def both(a, b, mlp, scales=(0.7, 1.2)):
    return {"type": "parallel", "mlp": mlp,
            "mixer": {"left": a, "right": b, "left_scale": scales[0], "right_scale": scales[1]}}


def latent(heads, dim, rot_dim, vdim, kv_rank, size, mlp, scale=0.3, base=300.0, scaling=None):
    return {"type": "latent_attention", "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank,
                      "scale": scale, "mask": {"size": size}, "rot": _rot(rot_dim, base, scaling)}}


def config(layers, vocab=67, width=40, eps=1e-4, streams=3, logit_scale=0.8):
    return {"architecture": "Minerax", "vocab": vocab, "width": width, "layers": layers,
            "norm": {"eps": eps}, "streams": streams, "logit_scale": logit_scale}


# sizes unlike each other and unlike the usual ones: a latent layer first, dim != vdim on both sides,
# query heads over fewer key heads on both sides, taps that differ between the sides, a window that
# is no multiple of the page, layers without feed-forward, with and without frequency scaling
SMALL = config([
    latent(3, 12, 8, 20, 24, 21, dense(28), scaling=yarn()),
    both(left(6, 2, 16, 8, 4, 8, scaling=yarn()), right(4, 2, 12, 20, 3), dense(36)),
    both(left(3, 3, 8, 12, 2, 6, softcap=2.5, base=50.0), right(2, 2, 8, 8, 5), None, scales=(1.3, 0.4)),
    latent(5, 8, 6, 12, 16, 37, None, scale=0.5, scaling=yarn(2.0, 64, 4.0, 0.5)),
])
# values that happen to be 1 or equal elsewhere: one stream, one head, one tap, every scale 1, a
# window of one position, everything rotated
ONES = config([both(left(1, 1, 16, 16, 1, 16, scale=1.0, softcap=1.0), right(1, 1, 16, 16, 1), dense(16),
                    scales=(1.0, 1.0)),
               latent(1, 16, 16, 16, 16, 1, None, scale=1.0),
               latent(2, 2, 2, 2, 1, 500, dense(1))], vocab=50, width=32, eps=1e-3, streams=1, logit_scale=1.0)
# nothing a multiple of 4 (width, head sizes, ranks, feed-forward widths, vocabulary); more streams
# than the unrolled forms of the stream kernel cover
ODD = config([both(left(3, 1, 10, 6, 3, 2), right(3, 3, 7, 9, 2), dense(11)),
              latent(3, 6, 10, 7, 15, 19, dense(21), scaling=yarn(2.0, 30, 6.0, 2.0)),
              both(left(2, 2, 6, 10, 3, 0), right(5, 1, 5, 3, 4), None)],
             vocab=53, width=37, streams=5)
# sizes the MFMA tiles cover (bf16 on the GPU); sixteen latent heads: decoded rows take the
# heads-as-columns form
WIDE = config([both(left(4, 2, 32, 32, 3, 16, softcap=15.0, scale=0.2), right(2, 2, 32, 64, 4), dense(64)),
               latent(16, 16, 32, 16, 64, 40, dense(64), scale=0.2, scaling=yarn()),
               both(left(6, 2, 64, 64, 4, 32, softcap=10.0, scale=0.15), right(4, 2, 64, 32, 2), dense(48)),
               latent(6, 48, 64, 32, 64, 33, None, scale=0.1)],
              width=64, vocab=90, streams=2)


def build(cfg_dict, device="cpu", dtype=torch.float32, seed=0, full=None, **eng_kw):
    cfg = minerax_from_json(cfg_dict, name="test-minerax")
    w = init_minerax_weights(cfg, device, dtype, seed) if full is None \
        else minerax_from_full(full, cfg, device, dtype)
    model = MineraxLM(cfg, device, weights=w, dtype=dtype)
    kw = dict(model="tiny-minerax", device=str(device), max_num_seqs=4, max_kv_blocks=24,
              max_batched_tokens=512, max_model_len=512, use_graphs=False, grammar=False,
              prefix_cache=False, warm_prefix=False, tune_gemm=False, jump_forward=False,
              dtype="float32" if dtype == torch.float32 else "bfloat16")
    kw.update(eng_kw)
    eng = LLMEngine(EngineConfig(**kw), model=model)
    return eng, w["full"]


def check(got, cfg_dict, full, requests, tol=3e-4):
    """Every produced row against the oracle's logits of that request and position."""
    ref = {n: oracle.forward(cfg_dict, full, t) for n, t in requests.items()}
    assert got, "no logits produced"
    for (n, p), row in got.items():
        r = ref[n][p]
        err = float((row.double() - r).abs().max() / r.abs().max())
        assert err < tol, f"request {n} position {p}: relative error {err:.2e}"
