// Mixture of experts: every token runs `top` of E small gated feed-forward layers.
//
//   moe_route    logits [T, E] (32-bit, rows ld apart) -> per token the `top` experts with the largest scores (softmax over
//                the experts, or a sigmoid of each logit on its own; the lower index wins a tie) and their
//                weights = score * scale, renormalised over the chosen ones or not; pairs are numbered t * top + k
//   moe_plan     the pairs grouped by expert: every expert's pairs take a run of places padded to whole
//                tiles of `tile` rows; place -> pair (-1: padding), pair -> place, tile -> expert, number
//                of tiles. One workgroup; which place of its expert's run a pair takes depends on the
//                order of atomics, which no result depends on (every place is computed on its own).
//   moe_gemm     per tile of places: rows gathered (token = pair / top, or the place itself) times the
//                tile's expert's matrix [N, K]; plain or gated (act(gate) * up, gate and up rows in one matrix);
//                the plain-precision kernel; bfloat16 steps take the grouped instances of the matrix-core tile kernel
//   moe_combine  out[t] (+)= sum_k weight[t, k] * y[place of (t, k)], k in order (no weights: each counts once); where a
//                shared layer's rows are given, first out[t] (+)= sigmoid(gate[t]) * shared[t]
//
//   moe_decide   the router's product, moe_route and moe_plan of a step of few tokens in one launch, in one workgroup
//   moe_combine_norm  moe_combine, then the norm behind the layer, the sum into the residual stream and the copy of the
//                updated rows that the next layer reads (layers whose sublayers are normed behind), in one pass over a row
//
// Everything that depends on the routing is read from device memory: a step's launches are the same
// whatever the tokens choose (grids are sized for the most tiles there can be; workgroups beyond the
// number of tiles leave at once).
#include "common.h"
#include <math.h>

namespace llme {

__device__ __forceinline__ float moe_act(float g, int act) {
    if (act == 0) return g / (1.0f + expf(-g));
    if (act == 1) return fmaxf(g, 0.f);
    return 0.5f * g * (1.0f + tanhf(0.7978845608028654f * (g + 0.044715f * g * g * g)));
}

constexpr int kMoeMaxPerLane = 16;      // experts per lane: up to 1024 experts

// One wavefront: the `top` experts with the largest scores of the logits z [E] and their weights. PER * 64 >= E.
template <int PER>
__device__ __forceinline__ void choose_experts(const float* z, int E, int top, float scale, int renorm, int sigmoid, int* ids, float* wts) {
    const int lane = threadIdx.x & (kWave - 1);
    float v[PER];
    float mx = -INFINITY;
#pragma unroll
    for (int i = 0; i < PER; ++i) {
        const int e = lane + i * kWave;
        v[i] = e < E ? z[e] : -INFINITY;
        mx = fmaxf(mx, v[i]);
    }
    mx = wave_max(mx);
    float sum = 0.f;
    if (!sigmoid) {
#pragma unroll
        for (int i = 0; i < PER; ++i) {
            v[i] = expf(v[i] - mx);                 // 0 beyond E
            sum += v[i];
        }
    }
    // (sigmoid scores: the experts are chosen by their logits, which order them as the scores do and still tell
    // experts apart where the 32-bit sigmoid has run into 1 or 0; a chosen expert's score is made from its logit)
    const float inv = sigmoid ? 1.0f : 1.0f / wave_sum(sum);
    const float none = sigmoid ? -INFINITY : -1.f;
    float chosen_sum = 0.f;
    for (int k = 0; k < top; ++k) {
        float best = none;
        int at = 0x7fffffff;
#pragma unroll
        for (int i = 0; i < PER; ++i) {
            const int e = lane + i * kWave;
            if (e < E && v[i] > best) {         // (within a lane the experts rise: the first maximum stays)
                best = v[i];
                at = e;
            }
        }
#pragma unroll
        for (int off = kWave / 2; off > 0; off >>= 1) {
            const float ob = __shfl_xor(best, off, kWave);
            const int oa = __shfl_xor(at, off, kWave);
            if (ob > best || (ob == best && oa < at)) {
                best = ob;
                at = oa;
            }
        }
        if (at >= E) at = E - 1;                // (logits that are no numbers choose nothing: any expert, so that places exist)
        const float s = sigmoid ? 1.0f / (1.0f + expf(-best)) : best * inv;
        chosen_sum += s;
        if (lane == 0) {
            ids[k] = at;
            wts[k] = s;
        }
#pragma unroll
        for (int i = 0; i < PER; ++i)
            if (lane + i * kWave == at) v[i] = sigmoid ? -INFINITY : -2.f;        // taken
    }
    if (lane == 0) {
        const float f = renorm ? scale / chosen_sum : scale;
        for (int k = 0; k < top; ++k) wts[k] *= f;
    }
}

template <int PER>
__global__ __launch_bounds__(256) void moe_route_kernel(const float* __restrict__ logits, int ld, int T, int E, int top,
                                                        float scale, int renorm, int sigmoid, int* __restrict__ ids,
                                                        float* __restrict__ wts) {
    const int t = blockIdx.x * 4 + threadIdx.x / kWave;
    if (t >= T) return;
    choose_experts<PER>(logits + static_cast<size_t>(t) * ld, E, top, scale, renorm, sigmoid, ids + static_cast<size_t>(t) * top,
                                   wts + static_cast<size_t>(t) * top);
}

// The router of up to 16 tokens, all in one workgroup of 16 wavefronts: the logits on the matrix cores
// (v_mfma_f32_16x16x32_bf16; the wavefronts split k between them in chunks of 128 elements and add up through LDS), the choice,
// a wavefront a token, and the plan. w [rows, K] has E rows, or E + 1 where a gate's row stands behind the experts'; its logit is
// left in logits [T, ld] with the others and takes no part in the choice. TILES * 16 >= rows.
constexpr int kDecideTokens = 16, kDecideRows = 128, kDecideTop = 32;

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(4))) float f32x4;

template <int TILES>
__global__ __launch_bounds__(1024) void moe_decide_kernel(const bf16* __restrict__ x, const bf16* __restrict__ w, int T, int K, int rows, int E,
                                                          int top, float scale, int renorm, int sigmoid, float* __restrict__ logits, int ld,
                                                          float* __restrict__ wts, int tile, int cap, int* __restrict__ place_pair,
                                                          int* __restrict__ pair_place, int* __restrict__ tile_expert,
                                                          int* __restrict__ n_tiles) {
    extern __shared__ __align__(16) unsigned char lds_raw[];
    f32x4* red = reinterpret_cast<f32x4*>(lds_raw);         // [16 wavefronts][TILES][64]
    __shared__ float z[kDecideTokens][TILES * 16];
    __shared__ int ids[kDecideTokens * kDecideTop];
    __shared__ int count[TILES * 16], offset[TILES * 16 + 1], fill[TILES * 16];
    const int tid = threadIdx.x, lane = tid & (kWave - 1), wave = tid / kWave, r = lane & 15, q = lane >> 4;
    bf16x8 none;
#pragma unroll
    for (int i = 0; i < 8; ++i) none[i] = static_cast<__bf16>(0.f);
    f32x4 acc[TILES];
#pragma unroll
    for (int c = 0; c < TILES; ++c) acc[c] = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int k0 = wave * 128; k0 < K; k0 += 16 * 128) {
        bf16x8 fx[4];
#pragma unroll
        for (int u = 0; u < 4; ++u) {
            const int k = k0 + u * 32 + q * 8;
            fx[u] = r < T && k < K ? *reinterpret_cast<const bf16x8*>(x + static_cast<size_t>(r) * K + k) : none;
        }
        constexpr int TOGETHER = 3;                         // tiles whose operands are asked for together (registers)
#pragma unroll
        for (int c0 = 0; c0 < TILES; c0 += TOGETHER) {
            bf16x8 fw[TOGETHER][4];
#pragma unroll
            for (int i = 0; i < TOGETHER; ++i)
#pragma unroll
                for (int u = 0; u < 4; ++u) {
                    const int k = k0 + u * 32 + q * 8, n = (c0 + i) * 16 + r;
                    fw[i][u] = c0 + i < TILES && n < rows && k < K ? *reinterpret_cast<const bf16x8*>(w + static_cast<size_t>(n) * K + k) : none;
                }
#pragma unroll
            for (int i = 0; i < TOGETHER; ++i)
#pragma unroll
                for (int u = 0; u < 4; ++u)
                    if (c0 + i < TILES) acc[c0 + i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fw[i][u], fx[u], acc[c0 + i], 0, 0, 0);
            __builtin_amdgcn_sched_barrier(0);
        }
    }
#pragma unroll
    for (int c = 0; c < TILES; ++c) red[(wave * TILES + c) * 64 + lane] = acc[c];
    for (int e = tid; e < TILES * 16; e += 1024) count[e] = fill[e] = 0;
    for (int i = tid; i < cap; i += 1024) place_pair[i] = -1;
    __syncthreads();
    // item: token r, rows c * 16 + 4 q + e
    for (int item = tid; item < TILES * 64; item += 1024) {
        const int c = item >> 6, l = item & 63, t = l & 15, n = c * 16 + (l >> 4) * 4;
        f32x4 s = red[c * 64 + l];
#pragma unroll
        for (int wv = 1; wv < 16; ++wv) {
            const f32x4 p = red[(wv * TILES + c) * 64 + l];
            s[0] += p[0]; s[1] += p[1]; s[2] += p[2]; s[3] += p[3];
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            z[t][n + e] = s[e];
            if (t < T && n + e < rows) logits[static_cast<size_t>(t) * ld + n + e] = s[e];
        }
    }
    __syncthreads();
    if (wave < T) {
        choose_experts<(TILES * 16 + kWave - 1) / kWave>(z[wave], E, top, scale, renorm, sigmoid, ids + wave * top,
                                                         wts + static_cast<size_t>(wave) * top);
    }
    __syncthreads();
    const int pairs = T * top;
    for (int i = tid; i < pairs; i += 1024) atomicAdd(&count[ids[i]], 1);
    __syncthreads();
    if (wave == 0) {
        // padded offsets: every lane adds up its run of experts, the lanes' sums are added up across the wavefront
        constexpr int PER = (TILES * 16 + kWave - 1) / kWave;
        int mine[PER], sum = 0;
#pragma unroll
        for (int i = 0; i < PER; ++i) {
            const int e = lane * PER + i;
            mine[i] = e < E ? (count[e] + tile - 1) / tile * tile : 0;
            sum += mine[i];
        }
        int upto = sum;
#pragma unroll
        for (int off = 1; off < kWave; off <<= 1) {
            const int o = __shfl_up(upto, off, kWave);
            if (lane >= off) upto += o;
        }
        int at = upto - sum;
#pragma unroll
        for (int i = 0; i < PER; ++i) {
            const int e = lane * PER + i;
            if (e < E) offset[e] = at;
            at += mine[i];
        }
        if (lane == kWave - 1) {
            offset[E] = upto;
            n_tiles[0] = upto / tile;
        }
    }
    __syncthreads();
    for (int e = tid; e < E; e += 1024)
        for (int i = offset[e] / tile; i < offset[e + 1] / tile; ++i) tile_expert[i] = e;
    for (int i = tid; i < pairs; i += 1024) {
        const int e = ids[i];
        const int at = offset[e] + atomicAdd(&fill[e], 1);
        place_pair[at] = i;
        pair_place[i] = at;
    }
}

// counts -> padded offsets -> places. E <= 1024.
__global__ __launch_bounds__(1024) void moe_plan_kernel(const int* __restrict__ ids, int pairs, int E, int tile,
                                                        int cap, int* __restrict__ place_pair, int* __restrict__ pair_place,
                                                        int* __restrict__ tile_expert, int* __restrict__ n_tiles) {
    __shared__ int count[1024];
    __shared__ int offset[1025];
    __shared__ int fill[1024];
    for (int e = threadIdx.x; e < E; e += 1024) {
        count[e] = 0;
        fill[e] = 0;
    }
    __syncthreads();
    for (int i = threadIdx.x; i < pairs; i += 1024) atomicAdd(&count[ids[i]], 1);
    __syncthreads();
    if (threadIdx.x == 0) {
        int at = 0;
        for (int e = 0; e < E; ++e) {
            offset[e] = at;
            at += (count[e] + tile - 1) / tile * tile;
        }
        offset[E] = at;
        n_tiles[0] = at / tile;
    }
    __syncthreads();
    const int used = offset[E];
    for (int i = threadIdx.x; i < cap; i += 1024) place_pair[i] = -1;
    for (int e = threadIdx.x; e < E; e += 1024)
        for (int i = offset[e] / tile; i < offset[e + 1] / tile; ++i) tile_expert[i] = e;
    __syncthreads();
    for (int i = threadIdx.x; i < pairs; i += 1024) {
        const int e = ids[i];
        const int at = offset[e] + atomicAdd(&fill[e], 1);
        place_pair[at] = i;
        pair_place[i] = at;
    }
    (void)used;
}

// Pieces of 16 places x 64 columns (a tile of `tile` places is tile / 16 pieces), k in slabs of 32 through LDS, 32-bit
// sums. GATED: out = act(a . gate) * (a . up), the expert's matrix holding gate and up rows in alternating groups of
// `group` rows (2 N rows in all). gather_div > 0: row of `a` = pair / gather_div (the token); 0: the place itself.
// Rows of padding give zeros.
template <typename TA, typename TW, typename TO, bool GATED>
__global__ __launch_bounds__(256) void moe_gemm_kernel(const TA* __restrict__ a, const TW* __restrict__ w, TO* __restrict__ out,
                                                       const int* __restrict__ place_pair, const int* __restrict__ tile_expert,
                                                       const int* __restrict__ n_tiles, int tile, int gather_div, int N, int K,
                                                       int group, int act) {
    __shared__ float As[16][33];
    __shared__ float Ws[64][33];
    __shared__ float Us[GATED ? 64 : 1][33];
    __shared__ int rows[16];
    const int piece = blockIdx.y;
    const int big = piece * 16 / tile;
    if (big >= n_tiles[0]) return;
    const int n0 = blockIdx.x * 64;
    const int e = tile_expert[big];
    if (threadIdx.x < 16) {
        const int pair = place_pair[piece * 16 + threadIdx.x];
        rows[threadIdx.x] = pair < 0 ? -1 : (gather_div > 0 ? pair / gather_div : piece * 16 + threadIdx.x);
    }
    __syncthreads();
    const int tr = threadIdx.x / 16, tc = threadIdx.x % 16;
    const TW* we = w + static_cast<size_t>(e) * (GATED ? 2 : 1) * N * K;
    float acc[4] = {0.f, 0.f, 0.f, 0.f}, acu[4] = {0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; k0 < K; k0 += 32) {
        for (int i = threadIdx.x; i < 16 * 32; i += 256) {
            const int rr = i / 32, kk = i % 32;
            const int row = rows[rr], k = k0 + kk;
            As[rr][kk] = (row >= 0 && k < K) ? to_float(a[static_cast<size_t>(row) * K + k]) : 0.f;
        }
        for (int i = threadIdx.x; i < 64 * 32; i += 256) {
            const int nn = i / 32, kk = i % 32;
            const int n = n0 + nn, k = k0 + kk;
            const bool in = n < N && k < K;
            const size_t row = GATED ? static_cast<size_t>(n / group) * 2 * group + n % group : n;      // the gate's row; up: group further
            Ws[nn][kk] = in ? to_float(we[row * K + k]) : 0.f;
            if (GATED) Us[nn][kk] = in ? to_float(we[(row + group) * K + k]) : 0.f;
        }
        __syncthreads();
#pragma unroll 8
        for (int kk = 0; kk < 32; ++kk) {
            const float av = As[tr][kk];
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                acc[j] = fmaf(av, Ws[tc + 16 * j][kk], acc[j]);
                if (GATED) acu[j] = fmaf(av, Us[tc + 16 * j][kk], acu[j]);
            }
        }
        __syncthreads();
    }
    TO* orow = out + (static_cast<size_t>(piece) * 16 + tr) * N;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int n = n0 + tc + 16 * j;
        if (n < N) orow[n] = from_float<TO>(GATED ? moe_act(acc[j], act) * acu[j] : acc[j]);
    }
}

__global__ void moe_combine_kernel(const float* __restrict__ y, const int* __restrict__ pair_place,
                                   const float* __restrict__ wts, float* __restrict__ out, int top, int H, int accumulate,
                                   const float* __restrict__ shared, const float* __restrict__ gate, int ld_gate,
                                   size_t total) {
    const size_t idx = static_cast<size_t>(blockIdx.x) * 256 + threadIdx.x;
    if (idx >= total) return;
    const size_t t = idx / H;
    const int c = static_cast<int>(idx % H);
    float s = accumulate ? out[idx] : 0.f;
    if (shared != nullptr) s += shared[idx] / (1.0f + expf(-gate[t * ld_gate]));
    for (int k = 0; k < top; ++k)
        s = fmaf(wts != nullptr ? wts[t * top + k] : 1.0f, y[static_cast<size_t>(pair_place[t * top + k]) * H + c], s);
    out[idx] = s;
}

// moe_combine and what stands behind the layer: y = sum_k weight y[place] + gate shared, h += scale (w_post y / rms(y)), x_out =
// the updated rows (or null). One workgroup a row of up to 8,192 values that are a multiple of 4 (NV groups of four a thread).
// clear_shared: the shared rows are zeros afterwards (their last product adds its parts).
template <typename TW, typename TO, int NV>
__global__ __launch_bounds__(256) void moe_combine_norm_kernel(const float* __restrict__ y, const int* __restrict__ pair_place,
                                                               const float* __restrict__ wts, int top, float* __restrict__ shared,
                                                               const float* __restrict__ gate, int ld_gate, int clear_shared,
                                                               const TW* __restrict__ w_post, float* __restrict__ h, TO* __restrict__ x_out,
                                                               int H, float eps, float scale) {
    __shared__ float scratch[4];
    const size_t t = blockIdx.x;
    float* hr = h + t * H;
    float v[NV][4], hv[NV][4], wv[NV][4];
    const float g = shared == nullptr ? 0.f : gate == nullptr ? 1.f : 1.0f / (1.0f + expf(-gate[t * ld_gate]));
#pragma unroll
    for (int k = 0; k < NV; ++k) {
        const int i = (threadIdx.x + 256 * k) * 4;
#pragma unroll
        for (int e = 0; e < 4; ++e) v[k][e] = hv[k][e] = wv[k][e] = 0.f;
        if (i >= H) continue;
        const float4 a = *reinterpret_cast<const float4*>(hr + i);
        hv[k][0] = a.x; hv[k][1] = a.y; hv[k][2] = a.z; hv[k][3] = a.w;
        struct alignas(sizeof(TW) * 4) Piece { TW x[4]; };
        const Piece p = *reinterpret_cast<const Piece*>(w_post + i);
#pragma unroll
        for (int e = 0; e < 4; ++e) wv[k][e] = to_float(p.x[e]);
        if (shared != nullptr) {
            float4* sp = reinterpret_cast<float4*>(shared + t * H + i);
            const float4 s = *sp;
            if (clear_shared) *sp = float4{0.f, 0.f, 0.f, 0.f};
            v[k][0] = g * s.x; v[k][1] = g * s.y; v[k][2] = g * s.z; v[k][3] = g * s.w;
        }
    }
    for (int c = 0; c < top; ++c) {
        const float wt = wts != nullptr ? wts[t * top + c] : 1.0f;
        const float* yr = y + static_cast<size_t>(pair_place[t * top + c]) * H;
#pragma unroll
        for (int k = 0; k < NV; ++k) {
            const int i = (threadIdx.x + 256 * k) * 4;
            if (i >= H) continue;
            const float4 a = *reinterpret_cast<const float4*>(yr + i);
            v[k][0] = fmaf(wt, a.x, v[k][0]);
            v[k][1] = fmaf(wt, a.y, v[k][1]);
            v[k][2] = fmaf(wt, a.z, v[k][2]);
            v[k][3] = fmaf(wt, a.w, v[k][3]);
        }
    }
    float ss = 0.f;
#pragma unroll
    for (int k = 0; k < NV; ++k)
#pragma unroll
        for (int e = 0; e < 4; ++e) ss = fmaf(v[k][e], v[k][e], ss);
    const float inv = 1.0f / sqrtf(block_sum(ss, scratch, 4) / static_cast<float>(H) + eps);
#pragma unroll
    for (int k = 0; k < NV; ++k) {
        const int i = (threadIdx.x + 256 * k) * 4;
        if (i >= H) continue;
        struct alignas(sizeof(TO) * 4) Out { TO x[4]; } o;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            hv[k][e] = fmaf(scale, (wv[k][e] * v[k][e]) * inv, hv[k][e]);
            o.x[e] = from_float<TO>(hv[k][e]);
        }
        *reinterpret_cast<float4*>(hr + i) = float4{hv[k][0], hv[k][1], hv[k][2], hv[k][3]};
        if (x_out != nullptr) *reinterpret_cast<Out*>(x_out + t * H + i) = o;
    }
}

}  // namespace llme

using namespace llme;

// x [T, K], w [rows, K] (rows E or E + 1) bfloat16, K a multiple of 8, 16-byte aligned.
extern "C" int llme_moe_decide(const void* x, const void* w, int T, int K, int rows, int E, int top, float scale, int renorm, int sigmoid,
                               float* logits, int ld, float* wts, int tile, int cap, int* place_pair, int* pair_place, int* tile_expert,
                               int* n_tiles, hipStream_t stream) {
    if (T <= 0) return 0;
    if (E <= 0 || top <= 0 || top > E || (rows != E && rows != E + 1) || ld < rows || tile <= 0) return kErrBadArgument;
    if (rows > kDecideRows || T > kDecideTokens || top > kDecideTop || K <= 0 || K % 8 != 0) return kErrUnsupported;
    const int pairs = T * top;
    if (cap % tile || cap < (pairs + E * (tile - 1)) / tile * tile) return kErrBadArgument;
#define LLME_DECIDE(TILES)                                                                                                              \
    do {                                                                                                                                \
        constexpr int LDS = 16 * TILES * 64 * 16;                                                                                       \
        static bool attr_set = false;                                                                                                   \
        if (!attr_set) {                                                                                                                \
            const hipError_t err = hipFuncSetAttribute(reinterpret_cast<const void*>(&moe_decide_kernel<TILES>),                        \
                                                       hipFuncAttributeMaxDynamicSharedMemorySize, LDS);                                \
            if (err != hipSuccess) return static_cast<int>(err);                                                                        \
            attr_set = true;                                                                                                            \
        }                                                                                                                               \
        hipLaunchKernelGGL((moe_decide_kernel<TILES>), dim3(1), dim3(1024), LDS, stream, static_cast<const bf16*>(x),                   \
                           static_cast<const bf16*>(w), T, K, rows, E, top, scale, renorm, sigmoid, logits, ld, wts, tile, cap, place_pair, \
                           pair_place, tile_expert, n_tiles);                                                                           \
    } while (0)
    if (rows <= 16) LLME_DECIDE(1);
    else if (rows <= 32) LLME_DECIDE(2);
    else if (rows <= 80) LLME_DECIDE(5);
    else LLME_DECIDE(8);
#undef LLME_DECIDE
    return launch_status();
}

extern "C" int llme_moe_combine_norm(const float* y, const int* pair_place, const float* wts, int top, float* shared, const float* gate,
                                     int ld_gate, int clear_shared, const void* w_post, int w_dtype, float* h, void* x_out, int xo_dtype, int T,
                                     int H, float eps, float scale, hipStream_t stream) {
    if (T <= 0) return 0;
    if (top <= 0 || (gate != nullptr && ld_gate <= 0)) return kErrBadArgument;
    if (H <= 0 || H % 4 != 0 || H > 8192) return kErrUnsupported;
    const int nv = H <= 2048 ? 2 : H <= 4096 ? 4 : 8;
#define LLME_CN(TW, TO, NV)                                                                                                                      hipLaunchKernelGGL((moe_combine_norm_kernel<TW, TO, NV>), dim3(T), dim3(256), 0, stream, y, pair_place, wts, top, shared, gate, ld_gate,                        clear_shared, static_cast<const TW*>(w_post), h, static_cast<TO*>(x_out), H, eps, scale)
#define LLME_CN_T(TW, TO)                  \
    do {                                   \
        if (nv == 2) LLME_CN(TW, TO, 2);   \
        else if (nv == 4) LLME_CN(TW, TO, 4); \
        else LLME_CN(TW, TO, 8);           \
    } while (0)
    const bool xb = x_out != nullptr && xo_dtype == kBF16;
    if (x_out != nullptr && xo_dtype != kBF16 && xo_dtype != kF32) return kErrBadArgument;
    if (w_dtype == kF32 && !xb) LLME_CN_T(float, float);
    else if (w_dtype == kF32) LLME_CN_T(float, bf16);
    else if (w_dtype == kBF16 && !xb) LLME_CN_T(bf16, float);
    else if (w_dtype == kBF16) LLME_CN_T(bf16, bf16);
    else return kErrBadArgument;
#undef LLME_CN_T
#undef LLME_CN
    return launch_status();
}

extern "C" int llme_moe_route(const float* logits, int ld, int T, int E, int top, float scale, int renorm, int sigmoid, int* ids,
                              float* wts, hipStream_t stream) {
    if (T <= 0) return 0;
    if (E <= 0 || top <= 0 || top > E || ld < E) return kErrBadArgument;
    if (E > kMoeMaxPerLane * kWave) return kErrUnsupported;
#define LLME_ROUTE(PER) \
    hipLaunchKernelGGL((moe_route_kernel<PER>), dim3((T + 3) / 4), dim3(256), 0, stream, logits, ld, T, E, top, scale, renorm, sigmoid, ids, wts)
    if (E <= kWave) LLME_ROUTE(1);
    else if (E <= 4 * kWave) LLME_ROUTE(4);
    else LLME_ROUTE(kMoeMaxPerLane);
#undef LLME_ROUTE
    return launch_status();
}

extern "C" int llme_moe_plan(const int* ids, int pairs, int E, int tile, int cap, int* place_pair, int* pair_place,
                             int* tile_expert, int* n_tiles, hipStream_t stream) {
    if (pairs <= 0) return 0;
    if (E <= 0 || tile <= 0) return kErrBadArgument;
    if (E > 1024) return kErrUnsupported;
    // room for every expert's run rounded up to whole tiles
    if (cap % tile || cap < (pairs + E * (tile - 1)) / tile * tile) return kErrBadArgument;
    hipLaunchKernelGGL(moe_plan_kernel, dim3(1), dim3(1024), 0, stream, ids, pairs, E, tile, cap, place_pair, pair_place,
                       tile_expert, n_tiles);
    return launch_status();
}

// gated: w [experts, 2 N, K] with gate and up rows in alternating groups of `group`; else w [experts, N, K].
extern "C" int llme_moe_gemm(const void* a, int a_dtype, const void* w, int gated, int w_dtype, void* out,
                             int out_dtype, const int* place_pair, const int* tile_expert, const int* n_tiles, int tile,
                             int max_tiles, int gather_div, int N, int K, int group, int act, hipStream_t stream) {
    if (max_tiles <= 0 || N <= 0) return 0;
    if (tile <= 0 || tile % 16 || (gated && (group <= 0 || N % group))) return kErrBadArgument;
    if (K <= 0 || static_cast<long>(max_tiles) * (tile / 16) > 65535) return kErrUnsupported;
    const dim3 grid((N + 63) / 64, max_tiles * (tile / 16));
#define LLME_MG(TA, TW, TO)                                                                                      \
    do {                                                                                                         \
        if (gated)                                                                                               \
            hipLaunchKernelGGL((moe_gemm_kernel<TA, TW, TO, true>), grid, dim3(256), 0, stream,                  \
                               static_cast<const TA*>(a), static_cast<const TW*>(w), static_cast<TO*>(out),      \
                               place_pair, tile_expert, n_tiles, tile, gather_div, N, K, group, act);            \
        else                                                                                                     \
            hipLaunchKernelGGL((moe_gemm_kernel<TA, TW, TO, false>), grid, dim3(256), 0, stream,                 \
                               static_cast<const TA*>(a), static_cast<const TW*>(w), static_cast<TO*>(out),      \
                               place_pair, tile_expert, n_tiles, tile, gather_div, N, K, group, act);            \
    } while (0)
    if (a_dtype == kF32 && w_dtype == kF32 && out_dtype == kF32) LLME_MG(float, float, float);
    else if (a_dtype == kBF16 && w_dtype == kBF16 && out_dtype == kBF16) LLME_MG(bf16, bf16, bf16);
    else if (a_dtype == kBF16 && w_dtype == kBF16 && out_dtype == kF32) LLME_MG(bf16, bf16, float);
    else if (a_dtype == kBF16 && w_dtype == kF32 && out_dtype == kBF16) LLME_MG(bf16, float, bf16);
    else if (a_dtype == kBF16 && w_dtype == kF32 && out_dtype == kF32) LLME_MG(bf16, float, float);
    else return kErrBadArgument;
#undef LLME_MG
    return launch_status();
}

extern "C" int llme_moe_combine(const float* y, const int* pair_place, const float* wts, float* out, int T, int top,
                                int H, int accumulate, const float* shared, const float* gate, int ld_gate, hipStream_t stream) {
    if (T <= 0) return 0;
    if (shared != nullptr && (gate == nullptr || ld_gate <= 0)) return kErrBadArgument;
    const size_t total = static_cast<size_t>(T) * H;
    hipLaunchKernelGGL(moe_combine_kernel, dim3(static_cast<unsigned>((total + 255) / 256)), dim3(256), 0, stream, y,
                       pair_place, wts, out, top, H, accumulate, shared, gate, ld_gate, total);
    return launch_status();
}

LLME_LOAD_ENTRY(moe)
