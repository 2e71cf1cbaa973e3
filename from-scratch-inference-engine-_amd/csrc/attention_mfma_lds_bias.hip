// Instantiations of the attention kernel that shares keys through LDS with a distance bias or a factor a token on the scores.
#include "attention_mfma_lds_impl.h"

namespace fsie_attn {

int launch_lds_biased(int hdt, const bf16_t* q, int64_t q_stride, const bf16_t* k_pool, const bf16_t* v_pool, const int32_t* block_tables,
                 int max_pages, const int32_t* items, const int32_t* groups, int n_groups, bf16_t* out, int n_heads, int n_kv,
                 int page_size, int window, float scale, const float* sinks, float softcap, const float* slopes,
                 const float* row_scale, hipStream_t stream) {
    return launch_lds_for<true>(hdt, q, q_stride, k_pool, v_pool, block_tables, max_pages, items, groups, n_groups, out, n_heads, n_kv,
                                 page_size, window, scale, sinks, softcap, slopes, row_scale, stream);
}

}  // namespace fsie_attn
