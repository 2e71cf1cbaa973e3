// Entry points of the attention kernel that shares keys through LDS, and its instantiations with scores as they are.
#include "attention_mfma_lds_impl.h"

namespace fsie_attn {

int launch_lds_plain(int hdt, const bf16_t* q, int64_t q_stride, const bf16_t* k_pool, const bf16_t* v_pool, const int32_t* block_tables,
                 int max_pages, const int32_t* items, const int32_t* groups, int n_groups, bf16_t* out, int n_heads, int n_kv,
                 int page_size, int window, float scale, const float* sinks, float softcap, const float* slopes,
                 const float* row_scale, hipStream_t stream) {
    return launch_lds_for<false>(hdt, q, q_stride, k_pool, v_pool, block_tables, max_pages, items, groups, n_groups, out, n_heads, n_kv,
                                 page_size, window, scale, sinks, softcap, slopes, row_scale, stream);
}

}  // namespace fsie_attn

// 1 if the LDS-shared kernel takes this geometry.
extern "C" int fsie_attention_mfma_lds_ok(int head_dim, int page_size) {
    const bool hd_ok = head_dim > 0 && head_dim % 32 == 0 && head_dim <= 256;
    const bool page_ok = page_size == 8 || page_size == 16 || page_size == 32 || page_size == 64;
    return hd_ok && page_ok ? 1 : 0;
}

// Large items (the `large` geometry of fsie_attention_mfma: up to 32 rows each) in groups of up to
// four consecutive tiles of one request: groups[2 g] = index of the group's first item in `items`,
// groups[2 g + 1] = its number of tiles (1..4).  The tiles of a group must follow one another in
// the request (ascending positions).
extern "C" int fsie_attention_mfma_lds(const void* q, int64_t q_stride, const void* k_pool, const void* v_pool,
                                       const int32_t* block_tables, int max_pages, const int32_t* items,
                                       const int32_t* groups, int n_groups, void* out, int n_heads, int n_kv,
                                       int head_dim, int page_size, int window, float scale, const float* sinks, float softcap,
                                       const float* slopes, const float* row_scale, hipStream_t stream) {
    FSIE_REQUIRE(n_groups >= 0 && n_heads > 0 && n_kv > 0 && n_heads % n_kv == 0,
                 "attention_mfma_lds: heads %d must be a positive multiple of kv heads %d", n_heads, n_kv);
    FSIE_REQUIRE(fsie_attention_mfma_lds_ok(head_dim, page_size),
                 "attention_mfma_lds: head_dim %d must be a multiple of 32 up to 256 and page_size %d one of 8, 16, 32, 64",
                 head_dim, page_size);
    FSIE_REQUIRE(max_pages > 0, "attention_mfma_lds: empty block table");
    FSIE_REQUIRE(q_stride % 8 == 0 && reinterpret_cast<uintptr_t>(q) % 16 == 0,
                 "attention_mfma_lds: query rows must be 16-byte aligned");
    FSIE_REQUIRE(!slopes || scale > 0.f, "attention_mfma_lds: a distance bias needs a positive scale, not %f", scale);
    if (n_groups == 0) return 0;
    const bf16_t* qq = static_cast<const bf16_t*>(q);
    const bf16_t* kk = static_cast<const bf16_t*>(k_pool);
    const bf16_t* vv = static_cast<const bf16_t*>(v_pool);
    bf16_t* oo = static_cast<bf16_t*>(out);
    const auto launch = slopes || row_scale ? fsie_attn::launch_lds_biased : fsie_attn::launch_lds_plain;
    return launch(head_dim / 16, qq, q_stride, kk, vv, block_tables, max_pages, items, groups, n_groups, oo, n_heads, n_kv,
                  page_size, window, scale, sinks, softcap, slopes, row_scale, stream);
}
