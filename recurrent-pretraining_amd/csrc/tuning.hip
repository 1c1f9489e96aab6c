// raven_set_tuning: one table of the launch-shape knobs that live in the other files.

#include <string>

#include "raven_common.h"

namespace raven {
int set_gemv1_tuning(const char* key, int value);
int set_skinny_tuning(const char* key, int value);
extern int g_linear_ks;
extern int g_tiled_min_rows, g_tiled_variant, g_tiled_split_tail;
extern int g_attn_split_target, g_attn_big_grid, g_attn_wide, g_linear_min_rows, g_attn_nosplit_pairs, g_attn_nosplit_len, g_rope_tiled_rows, g_prefill_waves, g_norm_early, g_fuse_sums_norm, g_attn_prefetch, g_fuse_qkv_rope, g_pad_chunk_rows, g_pad_decode_rows;
}  // namespace raven

extern "C" int raven_set_tuning(const char* key, int32_t value) {
    using namespace raven;
    RAVEN_REQUIRE(key != nullptr, "set_tuning: null key");
    const std::string k(key);
    if (k == "linear_ks") g_linear_ks = value;
    else if (k == "attn_split_target" && value > 0) g_attn_split_target = value;
    else if (k == "attn_big_grid" && value > 0) g_attn_big_grid = value;
    else if (k == "attn_wide") g_attn_wide = value;
    else if (k == "attn_prefetch" && value >= 0 && value <= 2) g_attn_prefetch = value;
    else if (k == "prefill_waves" && (value == 0 || value == 4 || value == 6)) g_prefill_waves = value;
    else if (k == "rope_tiled_rows" && value > 0) g_rope_tiled_rows = value;
    else if (k == "fuse_qkv_rope" && (value == 0 || value == 1)) g_fuse_qkv_rope = value;
    else if (k == "pad_chunk_rows" && (value == 0 || value == 1)) g_pad_chunk_rows = value;
    else if (k == "pad_decode_rows" && (value == 0 || value == 1)) g_pad_decode_rows = value;
    else if (k == "attn_nosplit_pairs" && value > 0 && value <= 1024) g_attn_nosplit_pairs = value;
    else if (k == "attn_nosplit_len" && value >= 0) g_attn_nosplit_len = value;
    else if (k == "linear_min_rows" && value >= 1) g_linear_min_rows = value;
    else if (k == "norm_early" && value >= -1 && value <= 1) g_norm_early = value;
    else if (k == "fuse_sums_norm" && (value == 0 || value == 1)) g_fuse_sums_norm = value;
    else if (k == "gemm_tiled_min_rows" && value >= 33) g_tiled_min_rows = value;
    else if (k == "gemm_tiled_variant" && value >= 0 && value <= 3) g_tiled_variant = value;
    else if (k == "gemm_tiled_split_tail" && (value == 0 || value == 1)) g_tiled_split_tail = value;
    else RAVEN_REQUIRE(set_gemv1_tuning(key, value) == 0 || set_skinny_tuning(key, value) == 0, "set_tuning: unknown key %s", key);
    return 0;
}
