// Products of few rows (up to 16 a tile; decoding) whose result passes something before it is stored: a gated feed-forward's
// activation, experts by tile, or the gate of a layer's per-token table. As in the skinny kernel of gemm_mfma.hip the weights
// are streamed once from memory straight into matrix operands (v_mfma_f32_16x16x32_bf16), a workgroup owning 16 output columns
// (a gated product: the 16 gate and the 16 up rows of 16 units) and its wavefronts splitting k between them in chunks of 128
// elements; they add up through LDS and what follows the product is done on the sums.
//
//   a [rows, K], w [N, K] (gated: 2 N rows, gate and up rows in alternating groups of 16; N a multiple of 16), both bfloat16,
//   K a multiple of 8, 16-byte aligned rows; w row-major or in the blocked layout (see gemm_mfma.hip).
//   groups: w [groups, rows, K] row-major; tile t (blockIdx.y) holds 16 places t * 16 .., exists if t < n_tiles[0] and belongs to
//   group tile_group[t]; a place's row of `a` is row_index[place] / gather_div (gather_div 0: the place itself; a negative
//   row_index: a row of zeros).
#include "common.h"

namespace llme {

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(4))) __bf16 bf16x4;
typedef __attribute__((ext_vector_type(4))) float f32x4;

enum FewMode : int { kFewStore = 0, kFewGated = 1, kFewTokenGate = 2 };

struct FewArgs {
    const bf16* a;
    const bf16* w;
    void* out;                  // kFewStore: [.., N] 32-bit; otherwise bfloat16
    int M, N, K, blocked, act;  // act of kFewGated: 0 SiLU, 1 rectifier, 2 tanh form of GELU
    // groups
    const int* tile_group;
    const int* n_tiles;
    const int* row_index;
    int gather_div;
    long w_stride;
    const float* pair_scale;    // kFewGated with row_index: the sums of a place times pair_scale[row_index[place]] first (or null)
    // kFewTokenGate: out = gelu_tanh(sum) * table[tokens[row] * ld_table + col + n]
    const bf16* table;
    const int* tokens;
    int ld_table, col;
};

__device__ __forceinline__ float few_gelu(float z) { return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z))); }
__device__ __forceinline__ float few_act(float g, int act) {
    return act == 1 ? fmaxf(g, 0.f) : act == 2 ? few_gelu(g) : g / (1.0f + expf(-g));
}
__device__ __forceinline__ bf16x8 few_zero() {
    bf16x8 z;
#pragma unroll
    for (int i = 0; i < 8; ++i) z[i] = static_cast<__bf16>(0.f);
    return z;
}

template <int NW, int MODE, bool GROUPED>
__global__ __launch_bounds__(NW * 64) void gemm_few_kernel(FewArgs p) {
    constexpr int U = 4, CHUNK = 32 * U, PARTS = MODE == kFewGated ? 2 : 1;
    __shared__ f32x4 red[NW * PARTS * 64];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int r = lane & 15, q = lane >> 4;
    const int K = p.K, tile = GROUPED ? blockIdx.y : 0;
    const bf16* w = p.w;
    int xr = r < p.M ? r : -1;
    if (GROUPED) {
        if (tile >= p.n_tiles[0]) return;                   // (the whole workgroup)
        w += static_cast<size_t>(p.tile_group[tile]) * p.w_stride;
        const int pair = p.row_index[tile * 16 + r];
        xr = pair < 0 ? -1 : p.gather_div > 0 ? pair / p.gather_div : tile * 16 + r;
    }
    // this lane's weights at k: row-major, row n0 + r from k + 8 q on; blocked, piece `lane` of block k / 32 of the row group
    const int n0 = blockIdx.x * 16 * PARTS;
    const bool wrow_ok = MODE == kFewGated || n0 + r < p.N;
    const bf16* wrow[PARTS];
#pragma unroll
    for (int g = 0; g < PARTS; ++g)
        wrow[g] = p.blocked ? w + static_cast<size_t>(blockIdx.x * PARTS + g) * 16 * K + lane * 8
                            : w + static_cast<size_t>(wrow_ok ? n0 + g * 16 + r : 0) * K + q * 8;
    const int wstep = p.blocked ? 16 : 1;
    const bf16* xrow = p.a + static_cast<size_t>(xr < 0 ? 0 : xr) * K + q * 8;
    f32x4 acc[PARTS];
#pragma unroll
    for (int g = 0; g < PARTS; ++g) acc[g] = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int k = wave * CHUNK; k < K; k += NW * CHUNK) {
        bf16x8 fw[PARTS][U], fx[U];
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int kk = k + u * 32;
            const bool k_ok = kk + q * 8 < K;
#pragma unroll
            for (int g = 0; g < PARTS; ++g)
                fw[g][u] = wrow_ok && (p.blocked ? kk < K : k_ok)
                               ? __builtin_nontemporal_load(reinterpret_cast<const bf16x8*>(wrow[g] + static_cast<size_t>(kk) * wstep))
                               : few_zero();
            fx[u] = xr >= 0 && k_ok ? *reinterpret_cast<const bf16x8*>(xrow + kk) : few_zero();
        }
#pragma unroll
        for (int u = 0; u < U; ++u)
#pragma unroll
            for (int g = 0; g < PARTS; ++g) acc[g] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fw[g][u], fx[u], acc[g], 0, 0, 0);
    }
#pragma unroll
    for (int g = 0; g < PARTS; ++g) red[(wave * PARTS + g) * 64 + lane] = acc[g];
    __syncthreads();
    if (tid >= 64) return;
    // result in lane l: row r of the tile, columns 4 q + e
    f32x4 s[PARTS];
#pragma unroll
    for (int g = 0; g < PARTS; ++g) {
        s[g] = red[g * 64 + lane];
        for (int wv = 1; wv < NW; ++wv) {
            const f32x4 o = red[(wv * PARTS + g) * 64 + lane];
            s[g][0] += o[0]; s[g][1] += o[1]; s[g][2] += o[2]; s[g][3] += o[3];
        }
    }
    if (!GROUPED && r >= p.M) return;
    const size_t row = static_cast<size_t>(tile) * 16 + r;
    const int nb = blockIdx.x * 16 + q * 4;
    if (MODE == kFewGated) {
        float scale = 1.f;
        if (GROUPED && p.pair_scale != nullptr) {
            const int pair = p.row_index[row];
            scale = pair < 0 ? 0.f : p.pair_scale[pair];
        }
        bf16x4 y;
#pragma unroll
        for (int e = 0; e < 4; ++e) y[e] = static_cast<__bf16>(few_act(s[0][e] * scale, p.act) * (s[PARTS - 1][e] * scale));
        *reinterpret_cast<bf16x4*>(static_cast<bf16*>(p.out) + row * p.N + nb) = y;
    } else if (MODE == kFewTokenGate) {
        const bf16* side = p.table + static_cast<size_t>(p.tokens[row]) * p.ld_table + p.col;
#pragma unroll
        for (int e = 0; e < 4; ++e)
            if (nb + e < p.N) static_cast<bf16*>(p.out)[row * p.N + nb + e] = static_cast<bf16>(few_gelu(s[0][e]) * static_cast<float>(side[nb + e]));
    } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
            if (nb + e < p.N) static_cast<float*>(p.out)[row * p.N + nb + e] = s[0][e];
    }
}

template <int MODE, bool GROUPED>
static int launch_few(const FewArgs& p, int tiles, hipStream_t stream) {
    const int columns = (p.N + 15) / 16;
    const dim3 grid(columns, tiles);
    // enough wavefronts to cover the chip several times, each with at least one chunk of k
    const long groups = static_cast<long>(columns) * tiles;
    const int chunks = (p.K + 127) / 128;
    int nw = 4;
    while (nw < 16 && groups * nw < 4096 && chunks >= nw * 2) nw *= 2;
    if (nw == 16) hipLaunchKernelGGL((gemm_few_kernel<16, MODE, GROUPED>), grid, dim3(1024), 0, stream, p);
    else if (nw == 8) hipLaunchKernelGGL((gemm_few_kernel<8, MODE, GROUPED>), grid, dim3(512), 0, stream, p);
    else hipLaunchKernelGGL((gemm_few_kernel<4, MODE, GROUPED>), grid, dim3(256), 0, stream, p);
    return launch_status();
}

static bool few_sizes_ok(int N, int K, int blocked, bool gated) {
    return N > 0 && K > 0 && K % 8 == 0 && K < (1 << 23) && !(gated && N % 16) && !(blocked && (N % 16 || K % 32));
}

}  // namespace llme

using namespace llme;

// out [M, N] bfloat16 = act(gate) * up for up to 16 rows; w [2 N, K].
extern "C" int llme_gemm_few_gated(const void* a, const void* w, void* out, int M, int N, int K, int blocked, int act, hipStream_t stream) {
    if (M <= 0) return 0;
    if (M > 16 || !few_sizes_ok(N, K, blocked, true)) return kErrUnsupported;
    if (act < 0 || act > 2) return kErrBadArgument;
    FewArgs p{};
    p.a = static_cast<const bf16*>(a); p.w = static_cast<const bf16*>(w); p.out = out;
    p.M = M; p.N = N; p.K = K; p.blocked = blocked; p.act = act;
    return launch_few<kFewGated, false>(p, 1, stream);
}

// out [M, N] bfloat16 = gelu_tanh(a w^T) * table[tokens[m], col + n] for up to 16 rows; table [.., ld_table] bfloat16.
extern "C" int llme_gemm_few_token_gate(const void* a, const void* w, void* out, int M, int N, int K, int blocked, const void* table, int ld_table,
                                        int col, const int* tokens, hipStream_t stream) {
    if (M <= 0) return 0;
    if (M > 16 || !few_sizes_ok(N, K, blocked, false)) return kErrUnsupported;
    if (col < 0 || col + N > ld_table) return kErrBadArgument;
    FewArgs p{};
    p.a = static_cast<const bf16*>(a); p.w = static_cast<const bf16*>(w); p.out = out;
    p.M = M; p.N = N; p.K = K; p.blocked = blocked;
    p.table = static_cast<const bf16*>(table); p.ld_table = ld_table; p.col = col; p.tokens = tokens;
    return launch_few<kFewTokenGate, false>(p, 1, stream);
}

// Experts in tiles of 16 places (see the head of the file). gated: out [max_tiles * 16, N] bfloat16 = act(gate) * up, w
// [groups, 2 N, K]; otherwise out [max_tiles * 16, N] 32-bit, w [groups, N, K].
extern "C" int llme_gemm_few_grouped(const void* a, const void* w, void* out, int gated, int N, int K, int act, int max_tiles,
                                     const int* tile_group, const int* n_tiles, const int* row_index, int gather_div, const float* pair_scale,
                                     hipStream_t stream) {
    if (max_tiles <= 0) return 0;
    if (!few_sizes_ok(N, K, 0, gated != 0) || max_tiles > 65535) return kErrUnsupported;
    if (act < 0 || act > 2 || tile_group == nullptr || n_tiles == nullptr || row_index == nullptr || (pair_scale != nullptr && !gated))
        return kErrBadArgument;
    FewArgs p{};
    p.a = static_cast<const bf16*>(a); p.w = static_cast<const bf16*>(w); p.out = out;
    p.M = 16; p.N = N; p.K = K; p.act = act;
    p.tile_group = tile_group; p.n_tiles = n_tiles; p.row_index = row_index; p.gather_div = gather_div;
    p.w_stride = static_cast<long>(gated ? 2 : 1) * N * K; p.pair_scale = pair_scale;
    return gated ? launch_few<kFewGated, true>(p, max_tiles, stream) : launch_few<kFewStore, true>(p, max_tiles, stream);
}

LLME_LOAD_ENTRY(gemm_few_rows)
