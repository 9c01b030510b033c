// What a token's id brings to the stream besides the plain embedding:
//   embed_norm : h[t] = w * e / sqrt(mean(e^2) + eps), e the token's row of the embedding table;
//   token_gate : out[t, j] = gelu_tanh(z[t, j]) * table[token_t, col + j], a layer's own slice of a per-token table, gated
//                by a product of the stream (the product back to the stream's width and its norm follow as usual).
// Everything in 32-bit; tables and weights in their stored type.
#include "common.h"

namespace llme {

__device__ __forceinline__ float gelu_tanh(float z) {
    return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}

// One workgroup a row, which waits in LDS between the two passes. blocked: the table is in the matrix kernels' layout
// ([V / 16][H / 32] blocks of [4][16][8]; V a multiple of 16, H of 32).
template <typename TT, typename TW>
__global__ __launch_bounds__(256) void embed_norm_kernel(const TT* __restrict__ table, const int* __restrict__ tokens,
                                                         const TW* __restrict__ w, float* __restrict__ out, int H, float eps,
                                                         int blocked) {
    extern __shared__ float row[];
    __shared__ float scratch[4];
    const int t = blockIdx.x, id = tokens[t];
    const TT* src = blocked ? table + static_cast<size_t>(id / 16) * 16 * H + (id % 16) * 8 : table + static_cast<size_t>(id) * H;
    float ss = 0.f;
    for (int i = threadIdx.x; i < H; i += 256) {
        const int j = i / 8;
        const float v = to_float(src[blocked ? static_cast<size_t>(j / 4) * 512 + (j % 4) * 128 + i % 8 : static_cast<size_t>(i)]);
        row[i] = v;
        ss = fmaf(v, v, ss);
    }
    const float inv = 1.0f / sqrtf(block_sum(ss, scratch, 4) / static_cast<float>(H) + eps);
    for (int i = threadIdx.x; i < H; i += 256) out[static_cast<size_t>(t) * H + i] = (to_float(w[i]) * row[i]) * inv;
}

// The same for rows of up to 8,192 entries in whole pieces of eight, which stay in registers (NV pieces a thread); in either layout
// a piece's entries lie together.
template <typename TT, typename TW, int NV>
__global__ __launch_bounds__(256) void embed_norm_vec_kernel(const TT* __restrict__ table, const int* __restrict__ tokens,
                                                             const TW* __restrict__ w, float* __restrict__ out, int H, float eps, int blocked) {
    __shared__ float scratch[4];
    struct alignas(16) TablePiece { TT x[8]; };
    struct alignas(16) WeightPiece { TW x[8]; };
    const int t = blockIdx.x, id = tokens[t];
    const TT* src = blocked ? table + static_cast<size_t>(id / 16) * 16 * H + (id % 16) * 8 : table + static_cast<size_t>(id) * H;
    float v[NV][8], wv[NV][8], ss = 0.f;
#pragma unroll
    for (int k = 0; k < NV; ++k) {
        const int j = threadIdx.x + 256 * k;
#pragma unroll
        for (int e = 0; e < 8; ++e) v[k][e] = wv[k][e] = 0.f;
        if (j * 8 >= H) continue;
        const TablePiece p = *reinterpret_cast<const TablePiece*>(src + (blocked ? static_cast<size_t>(j / 4) * 512 + (j % 4) * 128 : static_cast<size_t>(j) * 8));
        const WeightPiece q = *reinterpret_cast<const WeightPiece*>(w + j * 8);
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            v[k][e] = to_float(p.x[e]);
            wv[k][e] = to_float(q.x[e]);
            ss = fmaf(v[k][e], v[k][e], ss);
        }
    }
    const float inv = 1.0f / sqrtf(block_sum(ss, scratch, 4) / static_cast<float>(H) + eps);
#pragma unroll
    for (int k = 0; k < NV; ++k) {
        const int j = threadIdx.x + 256 * k;
        if (j * 8 >= H) continue;
        float y[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) y[e] = (wv[k][e] * v[k][e]) * inv;
        float4* dst = reinterpret_cast<float4*>(out + static_cast<size_t>(t) * H + j * 8);
        dst[0] = float4{y[0], y[1], y[2], y[3]};
        dst[1] = float4{y[4], y[5], y[6], y[7]};
    }
}

template <typename TT, typename TO>
__global__ __launch_bounds__(256) void token_gate_kernel(const float* __restrict__ z, int ld_z, const TT* __restrict__ table, int ld_table,
                                                         int col, const int* __restrict__ tokens, TO* __restrict__ out, int n, size_t total) {
    const size_t i = static_cast<size_t>(blockIdx.x) * 256 + threadIdx.x;
    if (i >= total) return;
    const size_t t = i / n;
    const int j = static_cast<int>(i % n);
    out[i] = from_float<TO>(gelu_tanh(z[t * ld_z + j]) * to_float(table[static_cast<size_t>(tokens[t]) * ld_table + col + j]));
}

}  // namespace llme

using namespace llme;

extern "C" int llme_embed_norm(const void* table, int table_dtype, const int* tokens, const void* w, int w_dtype, float* out, int T, int H,
                               float eps, int blocked, hipStream_t stream) {
    if (T <= 0) return 0;
    if (H <= 0 || H > 15000) return kErrUnsupported;
    if (blocked && (table_dtype != kBF16 || H % 32 != 0)) return kErrUnsupported;
    const size_t lds = static_cast<size_t>(H) * sizeof(float);
    const bool vec = H % 8 == 0 && H <= 8192 && reinterpret_cast<uintptr_t>(table) % 16 == 0 && reinterpret_cast<uintptr_t>(w) % 16 == 0 &&
                     reinterpret_cast<uintptr_t>(out) % 16 == 0;
    const int nv = !vec ? 0 : H <= 2048 ? 1 : H <= 4096 ? 2 : 4;
#define LLME_EN_V(TT, TW, NV)                                                                                                        \
    hipLaunchKernelGGL((embed_norm_vec_kernel<TT, TW, NV>), dim3(T), dim3(256), 0, stream, static_cast<const TT*>(table), tokens,     \
                       static_cast<const TW*>(w), out, H, eps, blocked)
#define LLME_EN(TT, TW)                                                                                                             \
    do {                                                                                                                            \
        if (nv == 1) LLME_EN_V(TT, TW, 1);                                                                                          \
        else if (nv == 2) LLME_EN_V(TT, TW, 2);                                                                                     \
        else if (nv == 4) LLME_EN_V(TT, TW, 4);                                                                                     \
        else                                                                                                                        \
            hipLaunchKernelGGL((embed_norm_kernel<TT, TW>), dim3(T), dim3(256), lds, stream, static_cast<const TT*>(table), tokens, \
                               static_cast<const TW*>(w), out, H, eps, blocked);                                                    \
    } while (0)
    switch (table_dtype * 2 + w_dtype) {
        case 0: LLME_EN(float, float); break;
        case 1: LLME_EN(float, bf16); break;
        case 2: LLME_EN(bf16, float); break;
        case 3: LLME_EN(bf16, bf16); break;
        default: return kErrBadArgument;
    }
#undef LLME_EN
#undef LLME_EN_V
    return launch_status();
}

extern "C" int llme_token_gate(const float* z, int ld_z, const void* table, int table_dtype, int ld_table, int col, const int* tokens,
                               void* out, int out_dtype, int T, int n, hipStream_t stream) {
    if (T <= 0 || n <= 0) return 0;
    if (ld_z < n || col < 0 || col + n > ld_table) return kErrBadArgument;
    const size_t total = static_cast<size_t>(T) * n;
    const dim3 grid(static_cast<unsigned>((total + 255) / 256));
#define LLME_TG(TT, TO)                                                                                                           \
    hipLaunchKernelGGL((token_gate_kernel<TT, TO>), grid, dim3(256), 0, stream, z, ld_z, static_cast<const TT*>(table), ld_table, col, \
                       tokens, static_cast<TO*>(out), n, total)
    switch (table_dtype * 2 + out_dtype) {
        case 0: LLME_TG(float, float); break;
        case 1: LLME_TG(float, bf16); break;
        case 2: LLME_TG(bf16, float); break;
        case 3: LLME_TG(bf16, bf16); break;
        default: return kErrBadArgument;
    }
#undef LLME_TG
    return launch_status();
}

LLME_LOAD_ENTRY(token_input)
