// Products of a mixture of experts over the rows that chose each expert, bfloat16, 32-bit accumulation.
//
// The chosen (token, expert) pairs of a step lie expert by expert (routed_ff.hip: counts, row_token, row_weight).  One
// launch runs every expert's product over its own rows: a block finds out from the counts, which stay on the device, which
// expert's tile of rows it is, so that the host never waits for them and a step may be recorded.  The rows of the first
// product are gathered on their way into LDS (each lane's address is a token's row), its epilogue applies the activation
// and the pair's weight to the 32-bit sums and rounds once; the second product leaves 32-bit rows, which
// llmrs_combine_rows adds up token by token.
//
// The tile loop is that of gemm_dma_kernel (gemm_mfma.hip): k-tiles of 64 straight into LDS, rows of 128 bytes whose
// 16-byte chunks are swizzled, STAGES of them in turn, v_mfma_f32_32x32x16_bf16.  An expert's weight may have rows further
// apart than they are long (ldw), so that the experts' down matrices can lie side by side.
//
// Steps of few tokens (the second half of this file) read every chosen expert's matrices once, straight into operands,
// for all of the step's tokens, and leave the experts that no token chose unread.
#include "gemm_tile.h"

enum ExpertAct { EXPERT_RELU2 = 0, EXPERT_CLAMPED = 1, EXPERT_SWIGLU = 2, EXPERT_NONE = 3 };

// Which expert the tile-th tile of `per` rows belongs to: its number, the tile's first row among all rows, and how many
// rows the tile has.  All lanes of a wave call this with the same arguments; false when there are fewer tiles.
__device__ __forceinline__ bool locate_expert_tile(const int* __restrict__ counts, int E, int per, int tile, int& expert, int& row0, int& rows) {
    int lane = threadIdx.x & 63, left = tile, before = 0;
    for (int base = 0; base < E; base += 64) {
        int n = base + lane < E ? counts[base + lane] : 0;
        int tiles = (n + per - 1) / per;
        int it = tiles, in = n;                       // sums over the lanes up to this one
#pragma unroll
        for (int d = 1; d < 64; d <<= 1) {
            int a = __shfl_up(it, d), b = __shfl_up(in, d);
            if (lane >= d) { it += a; in += b; }
        }
        int all = __shfl(it, 63);
        if (left < all) {
            unsigned long long holds = __ballot(left >= it - tiles && left < it);
            int src = __ffsll((long long)holds) - 1;
            int within = left - __shfl(it - tiles, src);
            expert = base + src;
            row0 = before + __shfl(in - n, src) + within * per;
            rows = min(per, __shfl(n, src) - within * per);
            return true;
        }
        left -= all;
        before += __shfl(in, 63);
    }
    return false;
}

template <int ACT>
__device__ __forceinline__ float expert_act(float g, float u, float limit, float alpha2) {
    if constexpr (ACT == EXPERT_SWIGLU) return silu_fast_f32(g) * u;
    g = fminf(g, limit);
    u = fminf(fmaxf(u, -limit), limit);
    return g * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(g * alpha2)) * (u + 1.0f);
}

// A: rows of K values, lda apart; row r of the experts' rows is A's row row_token[r] (null: r).  W: expert e's [N][K] at
// e * w_expert, rows ldw apart.  out: a row for every row; bf16 [.., N / 2] (gated activations) or [.., N] (relu2), times
// row_weight[r]; or 32-bit [.., N] (EXPERT_NONE).
template <int BM, int BN, int WGM, int WGN, int STAGES, int ACT>
__global__ __launch_bounds__(64 * WGM * WGN) void expert_tiles_kernel(const bf16* __restrict__ A, int lda, const int* __restrict__ row_token,
                                                                      const bf16* __restrict__ W, size_t w_expert, int ldw,
                                                                      const int* __restrict__ counts, int E, const float* __restrict__ row_weight,
                                                                      void* __restrict__ out, int ldc, int N, int K, float limit, float alpha2) {
    extern __shared__ __attribute__((aligned(1024))) unsigned char ex_smem[];
    constexpr int WAVES = WGM * WGN;
    constexpr int TM = BM / WGM, TN = BN / WGN, FM = TM / 32, FN = TN / 32;
    constexpr int STAGE_BYTES = (BM + BN) * 128;
    // a tile's groups of 8 rows (1 KB, a load instruction of a wave) are dealt out to the waves in turn; some waves may get one less
    constexpr int A_ALL = BM / 8, W_ALL = BN / 8, A_GROUPS = (A_ALL + WAVES - 1) / WAVES, W_GROUPS = (W_ALL + WAVES - 1) / WAVES;
    constexpr bool A_EVEN = A_ALL % WAVES == 0, W_EVEN = W_ALL % WAVES == 0;
    constexpr int LOADS = A_GROUPS + W_GROUPS;
    static_assert(STAGES == 2 || (A_EVEN && W_EVEN), "with more than two stages a wave counts its own loads: the same number in all waves");
    int expert = 0, row0 = 0, rows = 0;
    if (!locate_expert_tile(counts, E, BM, blockIdx.y, expert, row0, rows)) return;      // (the grid is sized for the most tiles the rows could make)
    expert = __builtin_amdgcn_readfirstlane(expert);
    row0 = __builtin_amdgcn_readfirstlane(row0);
    rows = __builtin_amdgcn_readfirstlane(rows);
    int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    int wm = wave / WGN, wn = wave % WGN;
    int n0 = blockIdx.x * BN;
    int lrow = lane >> 3, lslot = lane & 7;
    const bf16* We = W + (size_t)expert * w_expert;
    const bf16* ga[A_GROUPS];
    const bf16* gw[W_GROUPS];
#pragma unroll
    for (int i = 0; i < A_GROUPS; ++i) {
        int row = (wave + i * WAVES) * 8 + lrow;
        int r = row0 + min(row, rows - 1);
        int src = row_token ? row_token[r] : r;
        ga[i] = A + (size_t)src * lda + ((lslot ^ ((row >> 1) & 7)) * 8);
    }
#pragma unroll
    for (int i = 0; i < W_GROUPS; ++i) {
        int row = (wave + i * WAVES) * 8 + lrow;
        gw[i] = We + (size_t)min(n0 + row, N - 1) * ldw + ((lslot ^ ((row >> 1) & 7)) * 8);
    }
    const int nk = K / 64;
    auto issue = [&](int kt, int stage) {
        unsigned base = __builtin_amdgcn_readfirstlane(stage * STAGE_BYTES + wave * 1024);
#pragma unroll
        for (int i = 0; i < A_GROUPS; ++i)
            if (A_EVEN || wave + i * WAVES < A_ALL)
                __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)(ga[i] + kt * 64),
                                                 (__attribute__((address_space(3))) void*)(ex_smem + base + i * WAVES * 1024), 16, 0, 0);
        unsigned wbase = __builtin_amdgcn_readfirstlane(stage * STAGE_BYTES + BM * 128 + wave * 1024);
#pragma unroll
        for (int i = 0; i < W_GROUPS; ++i)
            if (W_EVEN || wave + i * WAVES < W_ALL)
                __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)(gw[i] + kt * 64),
                                                 (__attribute__((address_space(3))) void*)(ex_smem + wbase + i * WAVES * 1024), 16, 0, 0);
    };
    f32x16 acc[FM][FN];
#pragma unroll
    for (int i = 0; i < FM; ++i)
#pragma unroll
        for (int j = 0; j < FN; ++j)
#pragma unroll
            for (int r = 0; r < 16; ++r) acc[i][j][r] = 0.0f;
#pragma unroll
    for (int p = 0; p < STAGES - 1; ++p)
        if (p < nk) issue(p, p);
    if (nk >= STAGES - 1) wait_vmcnt<(STAGES - 2) * LOADS>(); else wait_vmcnt<0>();
    __syncthreads();
    int frow = lane & 31, h = lane >> 5;
    for (int kt = 0; kt < nk; ++kt) {
        int stage = kt % STAGES;
        if (kt + STAGES - 1 < nk) issue(kt + STAGES - 1, (kt + STAGES - 1) % STAGES);
        const unsigned char* as = ex_smem + stage * STAGE_BYTES;
        const unsigned char* ws = as + BM * 128;
#pragma unroll
        for (int ks = 0; ks < 4; ++ks) {
            bf16x8 a[FM], b[FN];
#pragma unroll
            for (int i = 0; i < FM; ++i) {
                int row = wm * TM + i * 32 + frow;
                a[i] = *(const bf16x8*)(as + row * 128 + (((ks * 2 + h) ^ ((row >> 1) & 7)) * 16));
            }
#pragma unroll
            for (int j = 0; j < FN; ++j) {
                int row = wn * TN + j * 32 + frow;
                b[j] = *(const bf16x8*)(ws + row * 128 + (((ks * 2 + h) ^ ((row >> 1) & 7)) * 16));
            }
#pragma unroll
            for (int i = 0; i < FM; ++i)
#pragma unroll
                for (int j = 0; j < FN; ++j) acc[i][j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a[i], b[j], acc[i][j], 0, 0, 0);
        }
        if (kt + STAGES - 1 < nk) wait_vmcnt<(STAGES - 2) * LOADS>(); else wait_vmcnt<0>();
        block_sync_lds();
    }
    if constexpr (ACT == EXPERT_NONE) {
        float* o = (float*)out;
        static_for<0, FM * FN>([&](auto idx) {
            constexpr int i = decltype(idx)::value / FN, j = decltype(idx)::value % FN;
            int n = n0 + wn * TN + j * 32 + frow;
#pragma unroll
            for (int r = 0; r < 16; ++r) {
                int m = wm * TM + i * 32 + 8 * (r >> 2) + 4 * h + (r & 3);
                if (m < rows && n < N) o[(size_t)(row0 + m) * ldc + n] = acc[i][j][r];
            }
        });
        return;
    } else {
        // The wave's tile through LDS (free after the loop's last barrier), stored row by row, 16 bytes a lane.  A lane holds
        // one column of 16 rows and its neighbour the next: they trade one value of each pair of rows, after which each has
        // both columns (gate and up, or two of relu2's) of one row.
        constexpr bool gated = ACT != EXPERT_RELU2;
        constexpr int cols = gated ? TN / 2 : TN, row_bytes = cols * 2;
        static_assert(TN * 2 * TM * WAVES <= STAGES * STAGE_BYTES, "the waves' tiles must fit in the tile buffers");
        unsigned char* mine = ex_smem + wave * (TN * 2 * TM);
        const bool odd = lane & 1;
        static_for<0, FM>([&](auto ic) {
            constexpr int i = decltype(ic)::value;
            float weight[8];
#pragma unroll
            for (int r = 0; r < 16; r += 2) {
                int row = wm * TM + i * 32 + 8 * (r >> 2) + 4 * h + (r & 3) + (odd ? 1 : 0);
                weight[r / 2] = row_weight[row0 + min(row, rows - 1)];
            }
            static_for<0, FN>([&](auto jc) {
                constexpr int j = decltype(jc)::value;
                int c = j * 32 + frow;
#pragma unroll
                for (int r = 0; r < 16; r += 2) {
                    int row = i * 32 + 8 * (r >> 2) + 4 * h + (r & 3) + (odd ? 1 : 0);
                    float v0 = acc[i][j][r], v1 = acc[i][j][r + 1];
                    float got = swap_neighbours(odd ? v0 : v1);
                    float left = odd ? got : v0, right = odd ? v1 : got;       // columns c & ~1 and c | 1 of `row`
                    if constexpr (gated) *(bf16*)(mine + row * row_bytes + (c / 2) * 2) = (bf16)(expert_act<ACT>(left, right, limit, alpha2) * weight[r / 2]);
                    else {
                        bf16x2 two;
                        left = fmaxf(left, 0.0f);
                        right = fmaxf(right, 0.0f);
                        two[0] = (bf16)(left * left * weight[r / 2]);
                        two[1] = (bf16)(right * right * weight[r / 2]);
                        *(bf16x2*)(mine + row * row_bytes + (c & ~1) * 2) = two;
                    }
                }
            });
        });
        __builtin_amdgcn_s_waitcnt(0xc07f);                       // lgkmcnt(0): the wave's own LDS writes are done
        constexpr int lanes_per_row = cols / 8, rows_per_pass = 64 / lanes_per_row;
        int lr = lane / lanes_per_row, lc = (lane % lanes_per_row) * 8;
        int n_out = (gated ? (n0 + wn * TN) / 2 : n0 + wn * TN) + lc, n_lim = gated ? N / 2 : N;
        for (int row = lr; row < TM; row += rows_per_pass) {
            int m = wm * TM + row;
            if (m < rows && n_out < n_lim)                        // (n_lim is a multiple of 8: a lane's 8 columns are in or out together)
                *(bf16x8*)((bf16*)out + (size_t)(row0 + m) * ldc + n_out) = *(const bf16x8*)(mine + row * row_bytes + lc * 2);
        }
    }
}

template <int BM, int BN, int WGM, int WGN, int STAGES, int ACT>
static int launch_expert_tiles(hipStream_t stream, const bf16* A, int lda, const int* row_token, const bf16* W, size_t w_expert, int ldw, const int* counts,
                               int E, long n_rows, const float* row_weight, void* out, int ldc, int N, int K, float limit, float alpha) {
    static bool configured = false;
    size_t bytes = (size_t)STAGES * (BM + BN) * 128;
    if (!configured) {
        hipError_t e = hipFuncSetAttribute((const void*)expert_tiles_kernel<BM, BN, WGM, WGN, STAGES, ACT>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes);
        if (e != hipSuccess) return llmrs_fail("expert_gemm: cannot reserve %zu bytes of LDS: %s", bytes, hipGetErrorString(e));
        configured = true;
    }
    // every expert with rows may end in a tile that is not full
    long tiles = n_rows / BM + (n_rows < E ? n_rows : E);
    LLMRS_REQUIRE(tiles <= 65535, "expert_gemm: %ld rows are too many for one launch", n_rows);
    dim3 grid(ceil_div(N, BN), (unsigned)tiles);
    expert_tiles_kernel<BM, BN, WGM, WGN, STAGES, ACT><<<grid, 64 * WGM * WGN, bytes, stream>>>(A, lda, row_token, W, w_expert, ldw, counts, E, row_weight, out, ldc,
                                                                                               N, K, limit, -alpha * 1.44269504088896341f);
    LLMRS_LAUNCH_CHECK("expert_gemm");
    return 0;
}

// Whether the grouped products take experts of these sizes: rows of `hidden` values, `ff` hidden units.
extern "C" int llmrs_expert_gemm_takes(int hidden, int ff) { return hidden > 0 && ff > 0 && hidden % 64 == 0 && ff % 64 == 0; }

// out[r, :] = act(x[row_token[r], :] Wup_e^T) * row_weight[r], one rounding; act 0: relu^2 (Wup_e [ff][hidden]), 1: clamped gated
// (limit, alpha), 2: silu gated (Wup_e [2 ff][hidden], gate and up row by row).  up: the experts one under the other.  counts
// [E]: rows of each expert, on the device; n_rows: the most there can be (their sum is no more); row_token, row_weight [n_rows].
extern "C" int llmrs_expert_up(hipStream_t stream, const void* x, int ldx, int n_tokens, const int* row_token, const void* up, const int* counts, int E,
                               long n_rows, const float* row_weight, void* out, int ldc, int ff, int hidden, int act, float limit, float alpha) {
    LLMRS_REQUIRE(x && row_token && up && counts && row_weight && out && E > 0 && E <= 65535 && n_rows >= 0 && n_tokens > 0, "expert_up: bad arguments");
    LLMRS_REQUIRE(llmrs_expert_gemm_takes(hidden, ff), "expert_up: sizes must be multiples of 64, got %d and %d", hidden, ff);
    LLMRS_REQUIRE(act >= 0 && act <= 2 && (act != 1 || limit > 0.0f), "expert_up: unknown activation %d, or a limit that is not positive", act);
    LLMRS_REQUIRE(ldx >= hidden && ldx % 8 == 0 && ldc >= ff && ldc % 8 == 0 && ((uintptr_t)x & 15) == 0 && ((uintptr_t)up & 15) == 0 && ((uintptr_t)out & 15) == 0,
                  "expert_up: rows of whole 16-byte pieces");
    if (n_rows == 0) return 0;
    const int N = (act == 0 ? 1 : 2) * ff;
    // (192 x 256 against 128 x 128 tiles: 8192 rows of 16 experts of 2048 x 2048 203 against 229 us, 3584 x 4096 620 against 672;
    // 16384 rows of 64 experts of 1024 x 2048 231 against 245; the down products below 6 % the other way on average)
#define UP(ACT) launch_expert_tiles<192, 256, 2, 4, 2, ACT>(stream, (const bf16*)x, ldx, row_token, (const bf16*)up, (size_t)N * hidden, hidden, counts, E, n_rows, \
                                                            row_weight, out, ldc, N, hidden, limit, alpha)
    return act == 0 ? UP(EXPERT_RELU2) : act == 1 ? UP(EXPERT_CLAMPED) : UP(EXPERT_SWIGLU);
#undef UP
}

// y[r, :] = a[r, :] Wdown_e^T, 32-bit; down: [hidden][E * ff], the experts' matrices side by side; a [n_rows, ff].
extern "C" int llmrs_expert_down(hipStream_t stream, const void* a, int lda, const void* down, const int* counts, int E, long n_rows, float* y, int ldy,
                                 int hidden, int ff) {
    LLMRS_REQUIRE(a && down && counts && y && E > 0 && E <= 65535 && n_rows >= 0, "expert_down: bad arguments");
    LLMRS_REQUIRE(llmrs_expert_gemm_takes(hidden, ff), "expert_down: sizes must be multiples of 64, got %d and %d", hidden, ff);
    LLMRS_REQUIRE((long)E * ff <= 0x7fffffffL && lda >= ff && lda % 8 == 0 && ldy >= hidden && ((uintptr_t)a & 15) == 0 && ((uintptr_t)down & 15) == 0,
                  "expert_down: rows of whole 16-byte pieces");
    if (n_rows == 0) return 0;
    return launch_expert_tiles<128, 128, 2, 2, 2, EXPERT_NONE>(stream, (const bf16*)a, lda, nullptr, (const bf16*)down, (size_t)ff, E * ff, counts, E, n_rows, nullptr,
                                                                y, ldy, hidden, ff, 0.0f, 0.0f);
}

// ---- steps of few tokens ------------------------------------------------------------------------------------------------
// Up to 64 tokens.  weights [T][ldw] 32-bit: what each token gives each expert, zero for those it did not choose.  Operands as
// in gemm_skinny_kernel (gemm_mfma.hip): v_mfma_f32_16x16x32_bf16 with the weight's rows as A and the tokens' rows as B, the
// block's waves taking the 64-wide k-blocks in turn and adding their sums in wave order through LDS.
#define EXPERT_FEW_TOKENS 64

__device__ __forceinline__ bf16x8 ex_load8(const bf16* p) { return *(const bf16x8*)p; }

// act[t, e * ff + f] = act(x[t] . Wup_e rows) * weights[t, e] for every token t and every expert e that some token chose (a
// token that did not choose it gets zeros); the other experts' columns are not written.  blockIdx.y: the expert.
template <int MT, int NT, int NW, int U, int ACT>
__global__ __launch_bounds__(NW * 64) void expert_few_up_kernel(const bf16* __restrict__ x, int ldx, int T, const bf16* __restrict__ up,
                                                                const float* __restrict__ weights, int ldw, int ff, int K, bf16* __restrict__ out, int ldc,
                                                                float limit, float alpha2) {
    __shared__ float red[NW * MT * NT * 4 * 64];
    constexpr bool gated = ACT != EXPERT_RELU2;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, row = lane & 15, g = lane >> 4, e = blockIdx.y;
    const float mine = lane < T ? weights[(size_t)lane * ldw + e] : 0.0f;
    if (__ballot(mine != 0.0f) == 0) return;                     // (the same in every wave of the block)
    const int N = gated ? 2 * ff : ff, n0 = blockIdx.x * NT * 16;
    const bf16* wp[NT];
    const bf16* xp[MT];
#pragma unroll
    for (int nt = 0; nt < NT; ++nt) wp[nt] = up + ((size_t)e * N + n0 + nt * 16 + row) * K + g * 8;
#pragma unroll
    for (int mt = 0; mt < MT; ++mt) xp[mt] = x + (size_t)min(mt * 16 + row, T - 1) * ldx + g * 8;
    f32x4 acc[MT][NT];
#pragma unroll
    for (int mt = 0; mt < MT; ++mt)
#pragma unroll
        for (int nt = 0; nt < NT; ++nt) acc[mt][nt] = f32x4{0.f, 0.f, 0.f, 0.f};
    const int nkb = K / 64;
    for (int j = wave; j < nkb; j += U * NW) {
        bf16x8 w[U][NT][2], xv[U][MT][2];
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const bool in = j + u * NW < nkb;                    // (the wave's: past the end the first block once more, times nothing)
            const int k = (in ? j + u * NW : j) * 64;
#pragma unroll
            for (int nt = 0; nt < NT; ++nt) { w[u][nt][0] = ex_load8(wp[nt] + k); w[u][nt][1] = ex_load8(wp[nt] + k + 32); }
#pragma unroll
            for (int mt = 0; mt < MT; ++mt) { xv[u][mt][0] = ex_load8(xp[mt] + k); xv[u][mt][1] = ex_load8(xp[mt] + k + 32); }
        }
        __builtin_amdgcn_sched_barrier(0);                       // keep the round's loads together, ahead of its MFMAs
#pragma unroll
        for (int u = 0; u < U; ++u) {
            if (j + u * NW >= nkb) break;
#pragma unroll
            for (int mt = 0; mt < MT; ++mt)
#pragma unroll
                for (int nt = 0; nt < NT; ++nt) {
                    acc[mt][nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w[u][nt][0], xv[u][mt][0], acc[mt][nt], 0, 0, 0);
                    acc[mt][nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w[u][nt][1], xv[u][mt][1], acc[mt][nt], 0, 0, 0);
                }
        }
    }
#pragma unroll
    for (int mt = 0; mt < MT; ++mt)
#pragma unroll
        for (int nt = 0; nt < NT; ++nt)
#pragma unroll
            for (int r = 0; r < 4; ++r) red[(((wave * MT + mt) * NT + nt) * 4 + r) * 64 + lane] = acc[mt][nt][r];
    __syncthreads();
    for (int tile = wave; tile < MT * NT; tile += NW) {
        int mt = tile / NT, nt = tile % NT;
        float v[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            float s = 0.0f;
#pragma unroll
            for (int w = 0; w < NW; ++w) s += red[(((w * MT + mt) * NT + nt) * 4 + r) * 64 + lane];
            v[r] = s;
        }
        int m = mt * 16 + row, n = n0 + nt * 16 + 4 * g;
        float wt = __shfl(mine, min(m, 63), 64);                 // (every lane holds its token's weight)
        if (m >= T) continue;
        bf16* o = out + (size_t)m * ldc + (size_t)e * ff;
        if constexpr (gated) {
            bf16x2 two;
            two[0] = (bf16)(expert_act<ACT>(v[0], v[1], limit, alpha2) * wt);
            two[1] = (bf16)(expert_act<ACT>(v[2], v[3], limit, alpha2) * wt);
            *(bf16x2*)(o + n / 2) = two;
        } else {
            bf16x4 four;
#pragma unroll
            for (int r = 0; r < 4; ++r) { float a = fmaxf(v[r], 0.0f); four[r] = (bf16)(a * a * wt); }
            *(bf16x4*)(o + n) = four;
        }
    }
}

// h[t, :] += sum over the experts that some token chose of act[t, e * ff ..] Wdown_e^T: the product of the activations with the
// matrices side by side, [hidden][E * ff], whose other experts' columns are not read.  A block takes LAST features (8: half a
// tile, whose other rows are never asked for) for all tokens.
template <int MT, int LAST, int NW, int U>
__global__ __launch_bounds__(NW * 64) void expert_few_down_kernel(const bf16* __restrict__ act, int lda, int T, const bf16* __restrict__ down,
                                                                  const float* __restrict__ weights, int ldw, int E, int ff, int D, float* __restrict__ h, int ldh) {
    __shared__ float red[NW * MT * 4 * 64];
    __shared__ int used[1024];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, row = lane & 15, g = lane >> 4;
    const int n0 = blockIdx.x * LAST;
    int n_used = 0;
    for (int base = 0; base < E; base += 64) {                   // (every wave makes the same list)
        bool any = false;
        if (base + lane < E) {
#pragma unroll 8
            for (int t = 0; t < T; ++t) any |= weights[(size_t)t * ldw + base + lane] != 0.0f;
        }
        unsigned long long has = __ballot(any);
        if (any && wave == 0) used[n_used + __popcll(has & ((1ull << lane) - 1ull))] = base + lane;
        n_used += __popcll(has);
    }
    float old[4] = {0.0f, 0.0f, 0.0f, 0.0f};                     // what the sums are added to, asked for beside the weights
    if (wave < MT) {
        int m = wave * 16 + row, n = n0 + 4 * g;
        if (m < T && (LAST == 16 || 4 * g < LAST))
#pragma unroll
            for (int r = 0; r < 4; ++r)
                if (n + r < D) old[r] = h[(size_t)m * ldh + n + r];
    }
    __syncthreads();
    const bool asks = LAST == 16 || row < LAST;
    const bf16* wp = down + (size_t)min(n0 + (asks ? row : 0), D - 1) * ((size_t)E * ff) + g * 8;
    const bf16* xp[MT];
#pragma unroll
    for (int mt = 0; mt < MT; ++mt) xp[mt] = act + (size_t)min(mt * 16 + row, T - 1) * lda + g * 8;
    f32x4 acc[MT];
#pragma unroll
    for (int mt = 0; mt < MT; ++mt) acc[mt] = f32x4{0.f, 0.f, 0.f, 0.f};
    bf16x8 nothing;
#pragma unroll
    for (int i = 0; i < 8; ++i) nothing[i] = (bf16)0.0f;
    const int per = ff / 64, nkb = n_used * per;
    for (int j = wave; j < nkb; j += U * NW) {
        bf16x8 w[U][2], xv[U][MT][2];
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int jj = j + u * NW < nkb ? j + u * NW : j;
            const int at = jj / per;
            const int k = __builtin_amdgcn_readfirstlane(used[at] * ff + (jj - at * per) * 64);
            w[u][0] = asks ? ex_load8(wp + k) : nothing;
            w[u][1] = asks ? ex_load8(wp + k + 32) : nothing;
#pragma unroll
            for (int mt = 0; mt < MT; ++mt) { xv[u][mt][0] = ex_load8(xp[mt] + k); xv[u][mt][1] = ex_load8(xp[mt] + k + 32); }
        }
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int u = 0; u < U; ++u) {
            if (j + u * NW >= nkb) break;
#pragma unroll
            for (int mt = 0; mt < MT; ++mt) {
                acc[mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w[u][0], xv[u][mt][0], acc[mt], 0, 0, 0);
                acc[mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w[u][1], xv[u][mt][1], acc[mt], 0, 0, 0);
            }
        }
    }
#pragma unroll
    for (int mt = 0; mt < MT; ++mt)
#pragma unroll
        for (int r = 0; r < 4; ++r) red[((wave * MT + mt) * 4 + r) * 64 + lane] = acc[mt][r];
    __syncthreads();
    if (wave >= MT) return;
    int m = wave * 16 + row, n = n0 + 4 * g;
    if (m >= T || (LAST < 16 && 4 * g >= LAST)) return;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        float s = 0.0f;
#pragma unroll
        for (int w = 0; w < NW; ++w) s += red[((w * MT + wave) * 4 + r) * 64 + lane];
        if (n + r < D) h[(size_t)m * ldh + n + r] = old[r] + s;
    }
}

// Up to EXPERT_FEW_TOKENS tokens; x [n_tokens, hidden], weights [n_tokens, E] 32-bit, out [n_tokens, E * ff]; up and act as for
// llmrs_expert_up.
extern "C" int llmrs_expert_few_up(hipStream_t stream, const void* x, int ldx, int n_tokens, const void* up, const float* weights, int ldw, int E, void* out,
                                   int ldc, int ff, int hidden, int act, float limit, float alpha) {
    LLMRS_REQUIRE(x && up && weights && out && n_tokens >= 0 && n_tokens <= EXPERT_FEW_TOKENS && E > 0 && E <= 1024 && ldw >= E, "expert_few_up: bad arguments");
    LLMRS_REQUIRE(llmrs_expert_gemm_takes(hidden, ff), "expert_few_up: sizes must be multiples of 64, got %d and %d", hidden, ff);
    LLMRS_REQUIRE(act >= 0 && act <= 2 && (act != 1 || limit > 0.0f), "expert_few_up: unknown activation %d, or a limit that is not positive", act);
    LLMRS_REQUIRE(ldx >= hidden && ldx % 8 == 0 && (long)ldc >= (long)E * ff && ldc % 8 == 0 && ((uintptr_t)x & 15) == 0 && ((uintptr_t)up & 15) == 0 && ((uintptr_t)out & 15) == 0,
                  "expert_few_up: rows of whole 16-byte pieces");
    if (n_tokens == 0) return 0;
    const int N = (act == 0 ? 1 : 2) * ff;
    const float alpha2 = -alpha * 1.44269504088896341f;
#define FEW(MT, NT, NW, U, ACT) expert_few_up_kernel<MT, NT, NW, U, ACT><<<dim3(N / (16 * NT), E), NW * 64, 0, stream>>>((const bf16*)x, ldx, n_tokens, (const bf16*)up, \
                                                                              weights, ldw, ff, hidden, (bf16*)out, ldc, limit, alpha2)
#define BY_ACT(MT, NT, NW, U) do { if (act == 0) FEW(MT, NT, NW, U, EXPERT_RELU2); else if (act == 1) FEW(MT, NT, NW, U, EXPERT_CLAMPED); else FEW(MT, NT, NW, U, EXPERT_SWIGLU); } while (0)
    if (n_tokens <= 4) BY_ACT(1, 1, 4, 8);
    else if (n_tokens <= 16) BY_ACT(1, 4, 4, 2);
    else if (n_tokens <= 32) BY_ACT(2, 4, 4, 2);
    else BY_ACT(4, 4, 4, 1);
#undef BY_ACT
#undef FEW
    LLMRS_LAUNCH_CHECK("expert_few_up");
    return 0;
}

// h [n_tokens, hidden] 32-bit += the experts' outputs; act as llmrs_expert_few_up leaves it, down [hidden][E * ff].
extern "C" int llmrs_expert_few_down(hipStream_t stream, const void* act, int lda, int n_tokens, const void* down, const float* weights, int ldw, int E, int ff,
                                     int hidden, float* h, int ldh) {
    LLMRS_REQUIRE(act && down && weights && h && n_tokens >= 0 && n_tokens <= EXPERT_FEW_TOKENS && E > 0 && E <= 1024 && ldw >= E, "expert_few_down: bad arguments");
    LLMRS_REQUIRE(llmrs_expert_gemm_takes(hidden, ff) && (long)E * ff <= 0x7fffffffL, "expert_few_down: sizes must be multiples of 64, got %d and %d", hidden, ff);
    LLMRS_REQUIRE((long)lda >= (long)E * ff && lda % 8 == 0 && ldh >= hidden && ((uintptr_t)act & 15) == 0 && ((uintptr_t)down & 15) == 0, "expert_few_down: rows of whole 16-byte pieces");
    if (n_tokens == 0) return 0;
#define FEW(MT, LAST, U) expert_few_down_kernel<MT, LAST, 8, U><<<ceil_div(hidden, LAST), 512, 0, stream>>>((const bf16*)act, lda, n_tokens, (const bf16*)down, weights, ldw, \
                                                                                                        E, ff, hidden, h, ldh)
    // (narrow streams: half tiles, so that every compute unit has a block)
    const bool half = ceil_div(hidden, 16) * 2 <= llmrs_compute_units();
    if (n_tokens <= 16) { if (half) FEW(1, 8, 4); else FEW(1, 16, 4); }
    else if (n_tokens <= 32) FEW(2, 16, 4);
    else FEW(4, 16, 2);
#undef FEW
    LLMRS_LAUNCH_CHECK("expert_few_down");
    return 0;
}
