// The matrix-core attention kernels (attention_mfma.h) for heads of two maps (differential attention): keys of both
// halves side by side, values as wide as both halves together or as wide as one.
#include "attention_mfma.h"

// 1 when it took the call, 0 when there is no kernel for these widths, -1 on error.
int llmrs_attention_bf16_mfma_maps(hipStream_t stream, const bf16* q, bf16* out, const bf16* k_cache, const bf16* v_cache,
                                   const int* block_table, const int* positions, const int* q_starts, const int* seq_lens,
                                   int n_entries, float* scratch, size_t scratch_bytes, int max_seq_len, int n_single,
                                   long single_keys, const AttnArgs& a) {
#define RUN(KD, VD) return launch<KD, VD, 2>(stream, q, out, k_cache, v_cache, block_table, positions, q_starts, seq_lens, n_entries, scratch, scratch_bytes, max_seq_len, n_single, single_keys, a)
    const bool both = a.v_dim == a.head_dim, one = 2 * a.v_dim == a.head_dim;
    switch (a.head_dim) {
        case 32: if (both) RUN(32, 32); break;
        case 64: if (both) RUN(64, 64); if (one) RUN(64, 32); break;
        case 96: if (both) RUN(96, 96); break;
        case 128: if (both) RUN(128, 128); if (one) RUN(128, 64); break;
        case 192: if (both) RUN(192, 192); if (one) RUN(192, 96); break;
        case 256: if (both) RUN(256, 256); if (one) RUN(256, 128); break;
        default: break;
    }
#undef RUN
    return 0;
}
