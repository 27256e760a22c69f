// The matrix-core attention kernels (attention_mfma.h) for heads of one map, what both kinds share, and the rule that
// says by how many keys single tokens are split.
#include "attention_mfma.h"

SideStream* llmrs_attention_side_stream() {
    static SideStream per_device[64];
    static std::mutex mutex;
    int dev = -1;
    if (hipGetDevice(&dev) != hipSuccess || dev < 0 || dev >= 64) return nullptr;
    std::lock_guard<std::mutex> lock(mutex);
    SideStream& s = per_device[dev];
    if (!s.tried) {
        s.tried = true;
        bool ok = hipStreamCreateWithFlags(&s.stream, hipStreamNonBlocking) == hipSuccess &&
                  hipEventCreateWithFlags(&s.fork, hipEventDisableTiming) == hipSuccess &&
                  hipEventCreateWithFlags(&s.join, hipEventDisableTiming) == hipSuccess;
        if (!ok) { (void)hipGetLastError(); s.stream = nullptr; }
    }
    return s.stream != nullptr ? &s : nullptr;
}

// How many waves of the split a compute unit holds at once: eight (see SPLIT16_LDS_BYTES), fewer where the registers
// of the kernel for this head size allow no more (four at head size 256), asked of the runtime once per head size.
// Head sizes without a kernel here: 8.  (The 32-column kernel, for more than 16 heads to a kv head, holds eight at
// head size 128 as well and twelve at 64; its chunks are chosen as if it held eight.)
static int split_waves_to_a_unit(int head_dim) {
    static int known[8] = {0, 0, 0, 0, 0, 0, 0, 0};      // by head_dim / 32 - 1
    static std::mutex mutex;
    if (head_dim % 32 || head_dim < 32 || head_dim > 256) return 8;
    std::lock_guard<std::mutex> lock(mutex);
    int& n = known[head_dim / 32 - 1];
    if (n == 0) {
        int blocks = 0;
        hipError_t e = hipErrorInvalidValue;
        switch (head_dim) {
#define ASK(HD) case HD: e = hipOccupancyMaxActiveBlocksPerMultiprocessor(&blocks, attn_split16_kernel<HD, HD, 1>, 64, SPLIT16_LDS_BYTES); break;
            ASK(32) ASK(64) ASK(96) ASK(128) ASK(192) ASK(256)
#undef ASK
            default: break;
        }
        if (e != hipSuccess) (void)hipGetLastError();
        n = (e == hipSuccess && blocks >= 1) ? std::min(blocks, 32) : 8;
    }
    return n;
}

// Keys per wave of the split, by what the host knows: the number of single-token entries, the bound on their
// length, and (when it says so) how many keys they see together.  Measured on the 8B head shape (8 to 256 requests
// of 520 to 8000 keys, every chunk from 64 to 1024 keys) and on the 1B one: a compute unit holds so many of these
// waves at once (eight) and works through them in turns of that many.  Waves of one
// turn, all of the same length, end together, and the longest chunks that still fill half a turn are the fastest
// (a wave begins with a chain of trips to memory: lengths, page numbers, then keys); one wave more than a turn
// costs a second turn.  So: the smallest chunk that gives a unit no more than three quarters of a turn (the next
// length then still gives it more than a third); and when even chunks of 1024
// keys give more than a turn, 512 if the last turn would be far from full (many short waves share out evenly as they come).
// Against the best chunk of each case (also at sizes and lengths between those it was made from, at 4 and 8 heads
// to a kv head, 2 and 8 kv heads) this rule is within the 3 % that two timings of one case differ by, 6 % at worst;
// the rule before the first of this kind (128 keys, doubled while the waves kept all units busy, by the bound alone)
// lost 7.5 % on average and 19 % at worst.  The chunks of a request are never
// more than a quarter of what the merge takes.
// The number of keys moves with every step while a recorded graph holds the chunk it was recorded with: callers that
// record put this function's result into what they key their recordings by.  The scratch is sized by the smallest
// chunk the entries and the bound allow, taken at an eighth of the bound for every entry; fewer keys than that get
// that chunk too.
// LLMRS_SPLIT_CHUNK in the environment (64 to 1024, a power of two) takes the choice away from the rule, for measuring it.
extern "C" int llmrs_attention_split_chunk(long singles, int n_kv_heads, int head_dim, int max_seq_len, long single_keys) {
    if (const char* e = getenv("LLMRS_SPLIT_CHUNK")) {
        int c = atoi(e);
        if (c >= ATTN_CHUNK / 2 && c <= 8 * ATTN_CHUNK && (c & (c - 1)) == 0) return c;
    }
    double cus = (double)llmrs_compute_units();
    if (singles < 1) singles = 1;
    if (max_seq_len < 1) max_seq_len = 1;
    const double turn = split_waves_to_a_unit(head_dim);
    const int longest = 8 * ATTN_CHUNK;
    auto pick = [&](double keys) {
        // waves to a compute unit with chunks of c keys, every entry taken at the mean length; the last chunk of a
        // request counts as a wave unless it is so short that it is gone before it matters
        auto to_a_unit = [&](int c) {
            double q = keys / singles / c, whole = floor(q), rest = q - whole;
            return singles * n_kv_heads * (whole + (rest > 0.125 ? 1.0 : 0.0)) / cus;
        };
        const double full = turn * 1.001;
        // With the 16-column kernel a unit does best on about half a turn of waves, one to a SIMD: a full turn of
        // chunks half as long takes 2-7 % longer, a quarter of a turn of chunks twice as long 15-25 % (8 to 128
        // requests of 520 to 8000 keys, every chunk forced).  So chunks are doubled while a unit would get more than
        // three quarters of a turn: the next length still leaves it more than a third.
        const double enough = 0.75 * turn;
        int c = ATTN_CHUNK / 2;
        while (c < longest && to_a_unit(c) > enough) c *= 2;
        if (c == longest && to_a_unit(c) > full) {
            double last = fmod(to_a_unit(c), turn) / turn;
            if (last > 0.006 && last < 0.69) c /= 2;
        }
        while (c < longest && (max_seq_len + c - 1) / c > MERGE_MAX_CHUNKS / 4) c *= 2;
        return c;
    };
    double bound_keys = (double)singles * max_seq_len;
    int least = pick(bound_keys / 8.0);
    double keys = single_keys > 0 ? fmin((double)single_keys, bound_keys) : 0.75 * bound_keys;
    return std::max(pick(keys), least);
}

// Heads of two maps (attention_mfma_maps.hip).
int llmrs_attention_bf16_mfma_maps(hipStream_t stream, const bf16* q, bf16* out, const bf16* k_cache, const bf16* v_cache,
                                   const int* block_table, const int* positions, const int* q_starts, const int* seq_lens,
                                   int n_entries, float* scratch, size_t scratch_bytes, int max_seq_len, int n_single,
                                   long single_keys, const AttnArgs& a);

int llmrs_attention_bf16_mfma(hipStream_t stream, const bf16* q, bf16* out, const bf16* k_cache, const bf16* v_cache,
                              const int* block_table, const int* token_entry, const int* positions,
                              const int* q_starts, const int* seq_lens, int n_entries, float* scratch,
                              size_t scratch_bytes, int max_seq_len, int n_single, long single_keys, const AttnArgs& a) {
    (void)token_entry;
    int G = a.n_heads / a.n_kv_heads * a.maps;
    // (a distance penalty is these kernels' too)
    if (a.v_dim != a.head_dim && !(a.maps == 2 && 2 * a.v_dim == a.head_dim)) return 0;
    if (a.maps == 2 && a.v_dim > 256) return 0;
    if (a.keep_first > 1024) return 0;                 // (the tiles of kept first keys: at most 32 a block)
    if (a.page_size != 16 || a.head_dim % 32 || G > 32 || q_starts == nullptr) return 0;
    if (a.q_stride % 8 || a.out_stride % 4 || ((uintptr_t)q & 15) || ((uintptr_t)out & 7)) return 0;
    if (n_entries > 65535 || a.n_kv_heads > 65535) return 0;
    int rc;
    if (a.maps == 2) {
        rc = llmrs_attention_bf16_mfma_maps(stream, q, out, k_cache, v_cache, block_table, positions, q_starts, seq_lens, n_entries,
                                            scratch, scratch_bytes, max_seq_len, n_single, single_keys, a);
        if (rc <= 0) return rc;
    } else switch (a.head_dim) {
#define CASE(HD) case HD: rc = launch<HD, HD, 1>(stream, q, out, k_cache, v_cache, block_table, positions, q_starts, seq_lens, n_entries, scratch, scratch_bytes, max_seq_len, n_single, single_keys, a); break;
        CASE(32) CASE(64) CASE(96) CASE(128) CASE(192) CASE(256)
#undef CASE
        default: return 0;
    }
    hipError_t err = hipGetLastError();
    if (err != hipSuccess) {
        llmrs_fail("attention (mfma): launch failed: %s", hipGetErrorString(err));
        return -1;
    }
    return rc;
}
