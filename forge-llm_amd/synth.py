"""Seeded synthetic tensors and models in the reference's on-disk formats.

There are no checkpoints offline, so every workload is random-init from a seed:
splitmix64 (counter based, so any slice can be generated independently) -> uniform ->
Box-Muller normals in f32.  Models are written as the headerless `weights.bin` that
`forge export-weights` produces (crates/forgellm-cli/src/main.rs:2714-2757; read back by
crates/forgellm-codegen-cpu/src/project.rs:342-407):

    embed_tokens f32 [vocab][hidden]
    per layer: attn_norm f32 | q | k | v | o raw blocks | ffn_norm f32 | gate | up | down raw blocks
    final_norm f32 | lm_head raw blocks

With tied embeddings the lm_head bytes are the quantised embedding and the f32 table is its
dequantisation (main.rs:2631-2693).
"""
from concurrent.futures import ThreadPoolExecutor

import numpy as np

_M64 = np.uint64(0xFFFFFFFFFFFFFFFF)
_CHUNK = 1 << 22


def splitmix64(seed: int, start: int, n: int) -> np.ndarray:
    """n outputs of splitmix64 seeded with `seed`, beginning at draw index `start`."""
    with np.errstate(over="ignore"):
        idx = np.arange(start + 1, start + n + 1, dtype=np.uint64)
        z = np.uint64(seed & 0xFFFFFFFFFFFFFFFF) + idx * np.uint64(0x9E3779B97F4A7C15)
        z = (z ^ (z >> np.uint64(30))) * np.uint64(0xBF58476D1CE4E5B9)
        z = (z ^ (z >> np.uint64(27))) * np.uint64(0x94D049BB133111EB)
        return z ^ (z >> np.uint64(31))


def _normal_chunk(seed, start_pair, npairs, std):
    z = splitmix64(seed, 2 * start_pair, 2 * npairs)
    u1 = ((z[0::2] >> np.uint64(11)).astype(np.float64) + 1.0) * (1.0 / 9007199254740992.0)   # (0, 1]
    u2 = (z[1::2] >> np.uint64(11)).astype(np.float64) * (1.0 / 9007199254740992.0)           # [0, 1)
    r = np.sqrt(-2.0 * np.log(u1)) * std
    ang = (2.0 * np.pi) * u2
    out = np.empty(2 * npairs, np.float32)
    out[0::2] = r * np.cos(ang)
    out[1::2] = r * np.sin(ang)
    return out


def normal(seed: int, n: int, std: float = 1.0, threads: int = 8) -> np.ndarray:
    """n f32 normals N(0, std^2), reproducible from (seed, n) alone."""
    npairs = (n + 1) // 2
    starts = list(range(0, npairs, _CHUNK))
    if len(starts) <= 1 or threads <= 1:
        parts = [_normal_chunk(seed, s, min(_CHUNK, npairs - s), std) for s in starts]
    else:
        with ThreadPoolExecutor(max_workers=threads) as ex:
            parts = list(ex.map(lambda s: _normal_chunk(seed, s, min(_CHUNK, npairs - s), std), starts))
    out = parts[0] if len(parts) == 1 else np.concatenate(parts)
    return out[:n]


def uniform_ids(seed: int, n: int, vocab: int) -> np.ndarray:
    """n token ids uniform in [0, vocab)."""
    return (splitmix64(seed, 0, n) % np.uint64(vocab)).astype(np.uint32)


# ---- model shapes named in the benchmark configurations ----
def _cfg(hidden, inter, layers, heads, kv_heads, head_dim, vocab, max_seq, theta, wdtype):
    return dict(hidden=hidden, inter=inter, layers=layers, heads=heads, kv_heads=kv_heads, head_dim=head_dim,
                vocab=vocab, max_seq=max_seq, rms_eps=1e-5, rope_theta=theta, wdtype=wdtype, lm_head_dtype=wdtype,
                flags=0)


def smollm2_135m(wdtype=8, max_seq=4096):
    return _cfg(576, 1536, 30, 9, 3, 64, 49152, max_seq, 100000.0, wdtype)


def llama32_1b(wdtype=8, max_seq=4096):
    return _cfg(2048, 8192, 16, 32, 8, 64, 128256, max_seq, 500000.0, wdtype)


def llama32_3b(wdtype=8, max_seq=4096):
    return _cfg(3072, 8192, 28, 24, 8, 128, 128256, max_seq, 500000.0, wdtype)


def llama31_8b(wdtype=8, max_seq=4096):
    return _cfg(4096, 14336, 32, 32, 8, 128, 128256, max_seq, 500000.0, wdtype)


def phi3_mini(wdtype=8, max_seq=4096):
    """Phi-3-mini-4k shape: 32 heads of 96 with a KV head each, vocabulary 32 064."""
    return _cfg(3072, 8192, 32, 32, 32, 96, 32064, max_seq, 10000.0, wdtype)


def qwen25_14b(wdtype=8, max_seq=4096):
    """Qwen2.5-14B shape: 48 layers (more than one launch of the resident decode kernel carries), QKV bias, 40 heads over
    8 KV heads, head_dim 128, vocabulary 152 064."""
    c = _cfg(5120, 13824, 48, 40, 8, 128, 152064, max_seq, 1000000.0, wdtype)
    c["flags"] = 2
    c["rms_eps"] = 1e-6
    return c


def mistral_7b(wdtype=8, max_seq=8192):
    """Mistral-7B-v0.1 shape: the Llama layer with a sliding window of 4096 positions, vocabulary 32 000."""
    c = _cfg(4096, 14336, 32, 32, 8, 128, 32000, max_seq, 10000.0, wdtype)
    c["sliding_window"] = 4096
    return c


def qwen25_1p5b(wdtype=8, max_seq=4096):
    """Qwen2.5-1.5B shape: QKV bias, 12 heads over 2 KV heads, head_dim 128, vocabulary 151 936."""
    c = _cfg(1536, 8960, 28, 12, 2, 128, 151936, max_seq, 1000000.0, wdtype)
    c["flags"] = 2
    c["rms_eps"] = 1e-6
    return c


def tiny(wdtype=8, max_seq=640, hidden=256, inter=512, layers=2, heads=4, kv_heads=2, head_dim=64, vocab=1000):
    return _cfg(hidden, inter, layers, heads, kv_heads, head_dim, vocab, max_seq, 10000.0, wdtype)


def make_weights_blob(cfg: dict, seed: int, std: float = 0.02, norm_jitter: float = 0.1, threads: int = 8) -> np.ndarray:
    """Random-init model as weights.bin bytes (tied embeddings).  Projection weights are f32
    N(0, std^2) quantised with the reference's quantisers; norm weights are 1 + norm_jitter*N(0,1)."""
    from .ops import block_bytes, dequant, quantize_weights
    H, I = cfg["hidden"], cfg["inter"]
    QKS, KV = cfg["heads"] * cfg["head_dim"], cfg["kv_heads"] * cfg["head_dim"]
    wt, lt = cfg["wdtype"], cfg["lm_head_dtype"]
    counter = [0]

    def sub_seed():
        counter[0] += 1
        return (seed * 1000003 + counter[0] * 7919) & 0xFFFFFFFFFFFFFFFF

    def qmat(n, k, dtype):
        return quantize_weights(dtype, normal(sub_seed(), n * k, std, threads))

    def norm_vec():
        return (1.0 + norm_jitter * normal(sub_seed(), H, 1.0, 1)).astype(np.float32)

    parts = []
    lm_raw = qmat(cfg["vocab"], H, lt)
    embed = dequant(lt, lm_raw, cfg["vocab"] * H)
    parts.append(embed.view(np.uint8))
    has_bias = bool(cfg.get("flags", 0) & 2)
    for _ in range(cfg["layers"]):
        parts.append(norm_vec().view(np.uint8))
        parts.append(qmat(QKS, H, wt))
        parts.append(qmat(KV, H, wt))
        parts.append(qmat(KV, H, wt))
        if has_bias:                                        # q_bias | k_bias | v_bias, f32 (project.rs:286-292)
            parts.append(normal(sub_seed(), QKS + 2 * KV, 0.5, 1).astype(np.float32).view(np.uint8))
        parts.append(qmat(H, QKS, wt))
        parts.append(norm_vec().view(np.uint8))
        parts.append(qmat(I, H, wt))
        parts.append(qmat(I, H, wt))
        parts.append(qmat(H, I, wt))
    parts.append(norm_vec().view(np.uint8))
    parts.append(lm_raw)
    blob = np.concatenate(parts)
    expect = (cfg["vocab"] * H * 4 + cfg["layers"] * (2 * H * 4 + (QKS * H + 2 * KV * H + H * QKS + 3 * I * H) // 32 * block_bytes(wt)
                                                       + ((QKS + 2 * KV) * 4 if has_bias else 0))
              + H * 4 + cfg["vocab"] * H // 32 * block_bytes(lt))
    assert blob.size == expect, (blob.size, expect)
    return blob


def kquant_blocks(rng, ggml_type: int, n_blocks: int, std: float = 0.02) -> np.ndarray:
    """n_blocks random Q4_K (144-byte) or Q6_K (210-byte) super-blocks whose 256 weights each have zero mean and a standard
    deviation near `std`: every payload byte uniform, the fp16 super-block scales chosen for that spread.  (Not a
    quantisation of anything: the tests need valid blocks of sane magnitude, not a particular matrix.)"""
    if ggml_type == 12:
        raw = rng.integers(0, 256, (n_blocks, 144), dtype=np.uint8)
        # w = d * sc * q - dmin * m with sc, m uniform in 0..63 and q in 0..15: zero mean for dmin = 7.5 d, spread 258 d
        d = (std / 258.0) * rng.uniform(0.7, 1.3, n_blocks)
        raw[:, 0:2] = d.astype(np.float16).view(np.uint8).reshape(-1, 2)
        raw[:, 2:4] = (7.5 * d).astype(np.float16).view(np.uint8).reshape(-1, 2)
    elif ggml_type == 14:
        raw = rng.integers(0, 256, (n_blocks, 210), dtype=np.uint8)
        # w = d * scale * (q - 32), scale an int8 kept within +-15 here, q in 0..63: spread about 165 d
        raw[:, 192:208] = rng.integers(-15, 16, (n_blocks, 16)).astype(np.int8).view(np.uint8)
        d = (std / 165.0) * rng.uniform(0.7, 1.3, n_blocks)
        raw[:, 208:210] = d.astype(np.float16).view(np.uint8).reshape(-1, 2)
    else:
        raise ValueError("kquant_blocks: Q4_K (12) or Q6_K (14)")
    return raw.reshape(-1)


def matrix_bytes(n: int, k: int, dtype: int) -> int:
    """Bytes of an [n][k] matrix in a storage format (GGML type id 8, 2, 12 or 14)."""
    if dtype in (12, 14):
        return n * (k // 256) * (144 if dtype == 12 else 210)
    return n * (k // 32) * (34 if dtype == 8 else 18)


def make_weights_blob_mixed(cfg: dict, proj_dtypes, seed: int, std: float = 0.02, norm_jitter: float = 0.1, threads: int = 8) -> np.ndarray:
    """Random-init model as weights.bin bytes with a storage format per projection: proj_dtypes = (q, k, v, o, gate, up,
    down) as GGML type ids, the lm_head in cfg["lm_head_dtype"]; Q8_0 / Q4_0 matrices are quantised normal weights, Q4_K /
    Q6_K matrices random super-blocks (kquant_blocks).  The f32 embedding table is drawn on its own (untied)."""
    from .ops import quantize_weights
    H, I = cfg["hidden"], cfg["inter"]
    QKS, KV = cfg["heads"] * cfg["head_dim"], cfg["kv_heads"] * cfg["head_dim"]
    rng = np.random.default_rng(seed)
    counter = [0]

    def sub_seed():
        counter[0] += 1
        return (seed * 1000003 + counter[0] * 7919) & 0xFFFFFFFFFFFFFFFF

    def mat(n, k, dtype):
        if dtype in (12, 14):
            assert k % 256 == 0, "a K-quant matrix needs K to be a multiple of 256"
            return kquant_blocks(rng, dtype, n * (k // 256), std)
        return quantize_weights(dtype, normal(sub_seed(), n * k, std, threads))

    def norm_vec():
        return (1.0 + norm_jitter * normal(sub_seed(), H, 1.0, 1)).astype(np.float32)

    pq, pk, pv, po, pg, pu, pdn = [int(x) for x in proj_dtypes]
    parts = [normal(sub_seed(), cfg["vocab"] * H, std, threads).view(np.uint8)]
    has_bias = bool(cfg.get("flags", 0) & 2)
    for _ in range(cfg["layers"]):
        parts += [norm_vec().view(np.uint8), mat(QKS, H, pq), mat(KV, H, pk), mat(KV, H, pv)]
        if has_bias:                                        # q_bias | k_bias | v_bias, f32 (project.rs:286-292)
            parts.append(normal(sub_seed(), QKS + 2 * KV, 0.5, 1).astype(np.float32).view(np.uint8))
        parts += [mat(H, QKS, po), norm_vec().view(np.uint8), mat(I, H, pg), mat(I, H, pu), mat(H, I, pdn)]
    parts += [norm_vec().view(np.uint8), mat(cfg["vocab"], H, cfg["lm_head_dtype"])]
    return np.concatenate(parts)


def gemv_bytes(n: int, k: int, wdtype: int) -> int:
    """Algorithmic bytes of one quantised GEMV: the GGUF blocks of the matrix (34 or 18 bytes
    per 32 weights) plus the f32 input and output vectors."""
    from .ops import block_bytes
    return n * (k // 32) * block_bytes(wdtype) + 4 * k + 4 * n


def decode_weight_bytes(cfg: dict) -> int:
    """Bytes of quantised weights (34- or 18-byte GGUF blocks) one decode step streams."""
    from .ops import block_bytes
    H, I = cfg["hidden"], cfg["inter"]
    QKS, KV = cfg["heads"] * cfg["head_dim"], cfg["kv_heads"] * cfg["head_dim"]

    def mat(n, k, dtype):
        return n * (k // 32) * block_bytes(dtype)

    wt = cfg["wdtype"]
    per_layer = mat(QKS, H, wt) + 2 * mat(KV, H, wt) + mat(H, QKS, wt) + 2 * mat(I, H, wt) + mat(H, I, wt)
    return cfg["layers"] * per_layer + mat(cfg["vocab"], H, cfg["lm_head_dtype"])


# ---- model folders (config.json + model.safetensors) ----------------------------------------------------------------------

def vabirax_layer(heads, dim, rot_dim, vdim, q_rank, kv_rank, ff, window, scale=None, base=10000.0, rot_dims=None) -> dict:
    """One entry of a Vabirax config's layer list; ff None: no feed-forward, window None: no mask."""
    mixer = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
             "scale": (dim + rot_dim) ** -0.5 if scale is None else scale, "rot": {"base": base, "dims": rot_dims or rot_dim}}
    if window:
        mixer["mask"] = {"size": window}
    return {"type": "latent_attention", "mixer": mixer, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def vabirax_config(width, vocab, layers, loop=None, embedding_scale=1.0, eps=1e-5) -> dict:
    """layers: vabirax_layer() entries; loop: (start, stop, times) or None."""
    c = {"architecture": "Vabirax", "width": width, "vocab": vocab, "embedding": {"scale": embedding_scale}, "norm": {"eps": eps},
         "layers": layers}
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


def vabirax_shapes(config) -> dict:
    """{tensor name: shape} of a Vabirax checkpoint."""
    w, out = config["width"], {}

    def norm(name):
        out[name], out[name + ".b"], out[name + ".alpha"] = (w,), (w,), ()

    out["embed"] = (config["vocab"], w)
    if config.get("loop"):
        out["loop.in"] = (w, 2 * w)
    for i, layer in enumerate(config["layers"]):
        m, n = layer["mixer"], "l%d." % i
        H = m["heads"]
        norm(n + "norm1")
        norm(n + "norm1b")
        for name, shape in (("dq", (m["q_rank"], w)), ("dq.norm", (m["q_rank"],)), ("uq", (H * (m["dim"] + m["rot_dim"]), m["q_rank"])),
                            ("dkv", (m["kv_rank"] + m["rot_dim"], w)), ("dkv.norm", (m["kv_rank"],)), ("uk", (H * m["dim"], m["kv_rank"])),
                            ("uv", (H * m["vdim"], m["kv_rank"])), ("g", (H * m["vdim"], w)), ("o", (w, H * m["vdim"]))):
            out[n + "mix." + name] = shape
        if layer["mlp"] is not None:
            norm(n + "norm2")
            norm(n + "norm2b")
            ff = layer["mlp"]["ff"]
            out[n + "mlp.gate"], out[n + "mlp.up"], out[n + "mlp.down"] = (ff, w), (ff, w), (w, ff)
    norm("final.norm")
    out["head"] = (config["vocab"], w)
    return out


def kakirax_attention(heads, kv_heads, dim, vdim, ff, scale=None, base=10000.0, rot_dims=None, scaling=None) -> dict:
    """One attention entry of a Kakirax config's layer list; ff None: no feed-forward; scaling: (factor, low, high, original) or None."""
    rot = {"base": base, "dims": rot_dims or dim}
    if scaling:
        rot["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": dim ** -0.5 if scale is None else scale, "rot": rot},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def kakirax_gla(heads, dim, vdim, ff, tau=16.0) -> dict:
    """One gated-linear-attention entry of a Kakirax config's layer list."""
    return {"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def kakirax_config(width, vocab, layers, embedding_scale=1.0, eps=1e-5, cap=30.0) -> dict:
    """layers: entries as above, or the index of the layer whose entry and weights a layer shares."""
    layers = [dict(layers[x], weights_of=x) if isinstance(x, int) else x for x in layers]
    return {"architecture": "Kakirax", "width": width, "vocab": vocab, "embedding": {"scale": embedding_scale}, "norm": {"eps": eps},
            "logit_softcap": cap, "layers": layers}


def kakirax_shapes(config, rank=16) -> dict:
    """{tensor name: shape} of a Kakirax checkpoint; rank: of the decays' low-rank maps."""
    w, out = config["width"], {}

    def norm(name):
        out[name], out[name + ".b"] = (w,), (w,)

    out["embed"] = (config["vocab"], w)
    for i, layer in enumerate(config["layers"]):
        if layer.get("weights_of") is not None:
            continue
        m, n = layer["mixer"], "l%d." % i
        H, d, dv = m["heads"], m["dim"], m["vdim"]
        norm(n + "norm1")
        if layer["type"] == "attention":
            G = m["kv_heads"]
            parts = (("q", (H * d, w)), ("k", (G * d, w)), ("v", (G * dv, w)), ("q.norm", (d,)), ("k.norm", (d,)), ("g", (H * dv, w)), ("o", (w, H * dv)))
        else:
            parts = (("q", (H * d, w)), ("k", (H * d, w)), ("v", (H * dv, w)), ("g", (H * dv, w)), ("o", (w, H * dv)), ("norm", (dv,)),
                     ("a1", (rank, w)), ("a2", (H * d, rank)), ("a2.b", (H * d,)))
        for name, shape in parts:
            out[n + "mix." + name] = shape
        if layer["mlp"] is not None:
            norm(n + "norm2")
            ff = layer["mlp"]["ff"]
            out[n + "mlp.gate"], out[n + "mlp.up"], out[n + "mlp.down"] = (ff, w), (ff, w), (w, ff)
    norm("final.norm")
    return out


def folder_shapes(config) -> dict:
    return {"Vabirax": vabirax_shapes, "Kakirax": kakirax_shapes}[config["architecture"]](config)


def to_bf16(x) -> np.ndarray:
    """float32 -> bfloat16 bits, to nearest even."""
    u = np.ascontiguousarray(x, np.float32).view(np.uint32).astype(np.uint64)
    return ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)


def from_bf16(bits) -> np.ndarray:
    return (np.asarray(bits, np.uint16).astype(np.uint32) << 16).view(np.float32)


def folder_tensors(config, seed, shapes=None) -> dict:
    """Random weights, bfloat16 bits by name: matrices with unit gain, norms that differ from element to element, decays from
    almost none to strong."""
    rng = np.random.default_rng(seed)
    out = {}
    shapes = shapes or folder_shapes(config)
    for name, shape in shapes.items():
        if len(shape) == 2:
            v = rng.standard_normal(shape) * (1.0 if name == "embed" and "head" in shapes else shape[1] ** -0.5)
        elif name.endswith(".alpha"):
            v = rng.uniform(0.5, 1.2)
        elif name.endswith(".b"):
            v = rng.standard_normal(shape) * (2.0 if name.endswith(".a2.b") else 0.1)
        else:
            v = rng.uniform(0.5, 1.5, shape)
        out[name] = to_bf16(np.asarray(v, np.float32)).reshape(shape)
    return out


def write_model_folder(path, config, tensors) -> None:
    """config.json and model.safetensors; tensors: bfloat16 bits (uint16) or float32 arrays by name, or {name: (shape, function
    that writes the bfloat16 bytes to a file)} for models that should not be held in memory."""
    import json
    import os
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(config, f, indent=1)
    header, at = {}, 0
    for name, t in tensors.items():
        shape, bits = (t[0], 16) if isinstance(t, tuple) else (t.shape, 16 if t.dtype == np.uint16 else 32)
        n = int(np.prod(shape, dtype=np.int64)) * bits // 8
        header[name] = {"dtype": "BF16" if bits == 16 else "F32", "shape": list(shape), "data_offsets": [at, at + n]}
        at += n
    text = json.dumps(header).encode()
    text += b" " * (-len(text) % 8)
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(len(text).to_bytes(8, "little") + text)
        for t in tensors.values():
            if isinstance(t, tuple):
                t[1](f)
            else:
                f.write(np.ascontiguousarray(t).tobytes())


def folder_stream(config, seed) -> dict:
    """Random weights for write_model_folder that are made while they are written: slices of one pool of normal numbers, scaled
    by the power of two nearest to unit gain.  For timing at real sizes."""
    rng = np.random.default_rng(seed)
    pool = to_bf16(rng.standard_normal(1 << 22, dtype=np.float32))

    def matrix(shape, shift):
        def write(f):
            left = int(np.prod(shape, dtype=np.int64))
            while left:
                a = int(rng.integers(0, pool.size // 2))
                part = pool[a:a + min(left, pool.size - a)]
                exp = (part >> 7) & 0xFF
                f.write(np.where(exp > shift, part - np.uint16(shift << 7), np.uint16(0)).astype(np.uint16).tobytes())
                left -= part.size
        return write

    out = {}
    shapes = folder_shapes(config)
    for name, shape in shapes.items():
        if len(shape) == 2:
            out[name] = (shape, matrix(shape, 0 if name == "embed" and "head" in shapes else int(round(np.log2(shape[1]) / 2))))
        else:
            out[name] = to_bf16(np.full(shape, 0.7 if name.endswith(".alpha") else 0.0 if name.endswith(".b") else 1.0, np.float32)).reshape(shape)
    return out


def vabirax_135m() -> dict:
    """SmolLM2-135M's width, depth and feed-forward; 9 heads of 64 + 32 (values 64), latents of 192 and 128, a window of 1024."""
    layer = vabirax_layer(9, 64, 32, 64, 192, 128, 1536, 1024)
    return vabirax_config(576, 49152, [layer] * 30, loop=(10, 20, 1), embedding_scale=24.0)


def vabirax_1b() -> dict:
    """Layers of Llama-3.2-1B's width, depth and feed-forward; 16 heads of 128 + 64 (values 128), latents of 768 and 512."""
    layer = vabirax_layer(16, 128, 64, 128, 768, 512, 8192, 4096, base=500000.0)
    return vabirax_config(2048, 128256, [layer] * 16, loop=(4, 12, 1), embedding_scale=1.0)


def vabirax_3b() -> dict:
    """Llama-3.2-3B's width, depth and feed-forward; 24 heads of 128 + 64 (values 128), latents of 1536 and 512."""
    layer = vabirax_layer(24, 128, 64, 128, 1536, 512, 8192, 4096, base=500000.0)
    return vabirax_config(3072, 128256, [layer] * 28, loop=(8, 20, 1), embedding_scale=1.0)


def kakirax_sizes(width, vocab, depth, ff, attention, gla, embedding_scale, scaling) -> dict:
    """Groups of three linear-attention layers and one attention layer, all with a feed-forward."""
    layers = [kakirax_attention(*attention, ff, base=500000.0, scaling=scaling) if i % 4 == 3 else kakirax_gla(*gla, ff) for i in range(depth)]
    return kakirax_config(width, vocab, layers, embedding_scale=embedding_scale)


def kakirax_135m() -> dict:
    """SmolLM2-135M's width, depth, feed-forward and attention; linear attention of 9 heads with keys of 32 and values of 64."""
    return kakirax_sizes(576, 49152, 30, 1536, (9, 3, 64, 64), (9, 32, 64), 24.0, None)


def kakirax_1b() -> dict:
    """Llama-3.2-1B's width, depth, feed-forward and attention; linear attention of 16 heads with keys of 64 and values of 128."""
    return kakirax_sizes(2048, 128256, 16, 8192, (32, 8, 64, 64), (16, 64, 128), 45.0, (32.0, 1.0, 4.0, 8192))


def kakirax_3b() -> dict:
    """Llama-3.2-3B's width, depth, feed-forward and attention; linear attention of 24 heads with keys of 64 and values of 128."""
    return kakirax_sizes(3072, 128256, 28, 8192, (24, 8, 128, 128), (24, 64, 128), 55.0, (32.0, 1.0, 4.0, 8192))
