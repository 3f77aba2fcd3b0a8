"""Hot ops of the inference engine.

Each op dispatches on the tensor's device: GPU tensors run the hand-written
CDNA4 HIP kernel (``csrc/kernels``), CPU tensors run the fp32 PyTorch
reference of the same op (used by the CPU tests and as the GPU numerics
oracle).  Projection GEMMs go through one table-driven router (``ops/gemm.py``
``route``): the hand-written 4-wave MFMA GEMM (``gemm_w4.hip``) for prefill-sized
passes and the full-batch gate_up + GLU, the skinny (``gemv.hip``) and medium-M
(``gemm_midm.hip``) decode kernels where they measured faster, and per-shape tuned
hipBLASLt solutions for the remaining decode buckets; everything around the GEMMs
is fused here.
"""
from ._ext import on_gpu, reference_mode
from .activation import act_glu, act_glu_ref
from .attention import (KV_BLOCK, DecodeWorkspace, decode_partitioning, paged_decode_attention,
                        paged_decode_attention_rope, set_prefill_persist,
                        paged_decode_ref, prefill_attention, prefill_attention_ref, prefill_tiles)
from .delta import DeltaWeights, Portions, delta_decode, delta_scan, short_conv
from .gated_average import (SCAN_CHUNK, AverageWeights, ScanChunks, chunk_scan, gated_decode,
                            gated_scan)
from .gemm import (fused_glu_ok, gated, glu_linear, linear, linear_residual, mfma_gemm, norm_glu,
                   norm_linear, residual_fusable, squared_relu, w4_glu_ok)
from .grouped import (GroupedDecodeWorkspace, GroupedPortions, GroupedWeights, attn_prep,
                      grouped_decode, grouped_prefill, grouped_qtile, prep_tile_rows)
from .latent import (LatentDecodeWorkspace, PortionKeys, build_interleaved_rope, head_linear,
                     latent_decode_attention, latent_gather, latent_prefill_attention,
                     latent_prep, latent_qtile, latent_width, portion_tiles, window_reach)
from .memory import MemoryWeights, memory_decode, memory_scan, memory_slices
from .moe import fused_moe, fused_moe_ref, router_logits, router_logits_f32
from .norm import PendingNorm, dyt, dyt_ref, group_rms, rmsnorm, rmsnorm_ref
from .norm_conv import (MAX_TAPS, ConvTiles, LayerNorm, conv_tile_rows, norm_conv, sinusoid_turns,
                        softcap_)
from .norm_side import side_gate, side_input, side_norm, stream_add
from .rope import build_rope_cache, kv_write_v, kv_write_v_ref, rope_kv_, rope_kv_ref
from .sampling import sample, sample_ref
from .talking import (MIX_TILE, STATS_TILE, TalkDecodeWorkspace, TalkPortions, TalkWeights,
                      head_prep, pad8, talk_cache_shapes, talk_decode, talk_prefill)

__all__ = [
    "on_gpu", "reference_mode", "linear", "norm_linear", "glu_linear", "norm_glu", "w4_glu_ok",
    "fused_glu_ok",
    "mfma_gemm", "linear_residual", "residual_fusable", "PendingNorm", "fused_moe", "router_logits",
    "fused_moe_ref", "act_glu", "act_glu_ref", "KV_BLOCK", "DecodeWorkspace",
    "decode_partitioning", "paged_decode_attention", "paged_decode_attention_rope",
    "paged_decode_ref", "prefill_attention", "prefill_attention_ref", "prefill_tiles",
    "set_prefill_persist", "rmsnorm", "rmsnorm_ref", "build_rope_cache", "rope_kv_",
    "rope_kv_ref", "kv_write_v", "kv_write_v_ref", "sample", "sample_ref", "dyt", "dyt_ref",
    "gated", "DeltaWeights", "Portions", "delta_decode", "delta_scan", "short_conv",
    "LatentDecodeWorkspace", "PortionKeys", "build_interleaved_rope", "head_linear",
    "latent_decode_attention", "latent_gather", "latent_prefill_attention", "latent_prep",
    "latent_qtile", "latent_width", "portion_tiles", "window_reach", "SCAN_CHUNK", "AverageWeights", "ScanChunks",
    "chunk_scan",    "gated_decode", "gated_scan", "squared_relu", "MAX_TAPS", "ConvTiles", "LayerNorm",
    "conv_tile_rows", "norm_conv", "sinusoid_turns", "softcap_", "MIX_TILE", "STATS_TILE",
    "TalkDecodeWorkspace", "TalkPortions", "TalkWeights", "head_prep", "pad8",
    "talk_cache_shapes", "talk_decode", "talk_prefill", "GroupedDecodeWorkspace",
    "GroupedPortions", "GroupedWeights", "attn_prep", "grouped_decode", "grouped_prefill",
    "grouped_qtile", "prep_tile_rows", "group_rms", "router_logits_f32",
    "MemoryWeights", "memory_decode", "memory_scan", "memory_slices", "side_gate", "side_input", "side_norm",
    "stream_add",
]
