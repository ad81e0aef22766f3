// Routed experts, token by token on the experts that were chosen and nothing else, with no wait for the host.
//
// A step's work is its pairs (token, chosen expert), sorted by expert: `counts` [E] pairs an expert, which begin at
// `offsets` [E]; `row_of` [P] the token of every pair, ascending within an expert; `slot_of` [T, top] where a token's
// pairs lie (-1: none) beside their weights `weights` [T, top], experts ascending.  Then every expert's two products run
// on its own pairs' rows (experts_gemv here for few pairs an expert; gemm_wreg's pairs mode for many), and a token's
// result is the weighted sum of its pairs' rows, in the order of the experts (in the pass that adds a sub-layer's
// normed output, or pair_sum here).  Everything is planned on the device: a step can be recorded whatever was chosen.
// Router logits, the choice, the weights and all sums are float32.
#include "gemm_common.h"

__device__ __forceinline__ f32x4 mfma16(f16x8 a, f16x8 b, f32x4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_f16(a, b, c, 0, 0, 0);
}
__device__ __forceinline__ f32x4 mfma16(bf16x8 a, bf16x8 b, f32x4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}

struct Pairs {
    int* counts;        // [E]
    int* offsets;       // [E]
    int* row_of;        // [P]
    int* slot_of;       // [T, top]
};

// The pairs of expert e (workgroup e), from `chosen` [n = T * top]: what lies before expert e is counted too, so every
// workgroup knows its own offset and none waits for another.  A wave takes a run of the pairs, 64 at a time; twice: how
// many there are, then where each goes.  Pairs that name no expert (-1) lie nowhere.
#define SORT_WAVES 16

__global__ __launch_bounds__(64 * SORT_WAVES) void sort_pairs_kernel(const int* __restrict__ chosen, int n, int top, Pairs p) {
    __shared__ int eq[SORT_WAVES], lt[SORT_WAVES];
    const int e = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int per = (n + 64 * SORT_WAVES - 1) / (64 * SORT_WAVES) * 64, lo = wave * per, hi = min(n, lo + per);
    int mine = 0, before = 0;
#pragma unroll 4
    for (int i0 = lo; i0 < hi; i0 += 64) {
        const int v = i0 + lane < hi ? chosen[i0 + lane] : -1;
        mine += __builtin_popcountll(__builtin_amdgcn_ballot_w64(v == e));
        before += __builtin_popcountll(__builtin_amdgcn_ballot_w64(v >= 0 && v < e));
    }
    if (lane == 0) { eq[wave] = mine; lt[wave] = before; }
    __syncthreads();
    int at = 0, total = 0, offset = 0;
#pragma unroll
    for (int w = 0; w < SORT_WAVES; ++w) {
        if (w < wave) at += eq[w];
        total += eq[w];
        offset += lt[w];
    }
    at += offset;
#pragma unroll 4
    for (int i0 = lo; i0 < hi; i0 += 64) {
        const int i = i0 + lane, v = i < hi ? chosen[i] : -2;
        const uint64_t mask = __builtin_amdgcn_ballot_w64(v == e);
        if (v == e) {
            const int s = at + __builtin_popcountll(mask & ((1ull << lane) - 1));
            p.row_of[s] = i / top;
            p.slot_of[i] = s;
        }
        if (e == 0 && v == -1) p.slot_of[i] = -1;
        at += __builtin_popcountll(mask);
    }
    if (threadIdx.x == 0) { p.counts[e] = total; p.offsets[e] = offset; }
}

extern "C" int li_sort_pairs(const int* chosen, int n, int top, int n_experts, int* counts, int* offsets, int* row_of,
                             int* slot_of, hipStream_t stream) {
    if (n <= 0) return LI_OK;
    if (top < 1 || n % top || n_experts < 1 || !chosen || !counts || !offsets || !row_of || !slot_of) return LI_BAD_ARG;
    sort_pairs_kernel<<<n_experts, 64 * SORT_WAVES, 0, stream>>>(chosen, n, top, Pairs{counts, offsets, row_of, slot_of});
    LI_CHECK_LAUNCH();
    return LI_OK;
}

// ---------------------------------------------------------------------------
// The router, 16 tokens a workgroup of 16 waves: logits z = W h + b against the tiled 16-bit matrix W [n, K] on the matrix
// cores, the waves sharing W's tiles of 16 rows and, where there are fewer tiles than waves, K.  W is the sum of `parts`
// 16-bit matrices one behind the other (each of n rows rounded up to 16: the rounding of W and the roundings of what is
// left, one matrix where the file's own numbers are 16-bit), so products are those of a float32 W, summed in float32.  Then a wave a token: the `top` largest logits (the first of
// equals), their weights the softmax over them alone times `scale`.  chosen and weights [T, top], experts ascending.
// With one workgroup (up to 16 tokens) it also sorts the pairs.
// ---------------------------------------------------------------------------
#define ROUTER_WAVES 16
#define ROUTER_MAX 512

// NC: outputs in groups of 64 that a wave holds, ceil(n / 64) rounded up to 1 or 8.
template <class T, int NC>
__global__ __launch_bounds__(64 * ROUTER_WAVES) void router_kernel(const T* __restrict__ X, const T* __restrict__ Wt,
                                                                   const float* __restrict__ bias, int parts, int n_tokens, int K,
                                                                   int n, int top, float scale, int* __restrict__ chosen,
                                                                   float* __restrict__ weights, Pairs p) {
    typedef typename Vec<T>::v8 v8;
    constexpr int U = 8;
    extern __shared__ float lds[];
    __shared__ float part[ROUTER_WAVES][64][4];
    float* z = lds;                                        // [16][n]
    int* picked = (int*)(lds + 16 * n);                    // [16][top]: the chosen experts, for the sort
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r = lane & 15, g = lane >> 4;
    const int t0 = blockIdx.x * 16, steps = K >> 5, tiles = (n + 15) >> 4;
    // kw waves share K for a tile; at_once tiles are worked on at a time
    const int kw = tiles >= ROUTER_WAVES ? 1 : ROUTER_WAVES / tiles, at_once = ROUTER_WAVES / kw;
    const int share = wave % kw, per = (steps + kw - 1) / kw, s_begin = share * per, s_end = min(steps, s_begin + per);
    const bool have = t0 + r < n_tokens;
    const T* xrow = X + (int64_t)(have ? t0 + r : t0) * K + 8 * g;
    for (int first = 0; first < tiles; first += at_once) {
        const int tile = first + wave / kw;
        const bool on = wave / kw < at_once && tile < tiles;
        f32x4 acc = {0.f, 0.f, 0.f, 0.f};
        if (on) {
            for (int pt = 0; pt < parts; ++pt) {
            const T* wt = Wt + ((int64_t)(pt * tiles + tile) * steps * 64 + lane) * 8;
            for (int s0 = s_begin; s0 < s_end; s0 += U) {
                v8 a[U], b[U];
#pragma unroll
                for (int u = 0; u < U; ++u) {
                    const v8 zero = {};
                    const bool in = s0 + u < s_end;
                    a[u] = in ? *(const v8*)(wt + (int64_t)(s0 + u) * 512) : zero;
                    b[u] = in && have ? *(const v8*)(xrow + (s0 + u) * 32) : zero;
                }
#pragma unroll
                for (int u = 0; u < U; ++u) acc = mfma16(a[u], b[u], acc);
            }
            }
        }
#pragma unroll
        for (int q = 0; q < 4; ++q) part[wave][lane][q] = acc[q];
        __syncthreads();
        if (on && share == 0) {
#pragma unroll
            for (int q = 0; q < 4; ++q) {
                float v = part[wave][lane][q];
                for (int k = 1; k < kw; ++k) v += part[wave + k][lane][q];
                const int j = tile * 16 + 4 * g + q;
                if (j < n) z[r * n + j] = v + (bias ? bias[j] : 0.f);
            }
        }
        __syncthreads();
    }
    const int t = t0 + wave;
    if (t < n_tokens) {                                    // (a wave's token, the same for all its lanes)
        float* zt = z + wave * n;
        float mx = 0.f, sum = 0.f;
        float zs[NC];
#pragma unroll
        for (int c = 0; c < NC; ++c) zs[c] = c * 64 + lane < n ? zt[c * 64 + lane] : -INFINITY;
        uint32_t taken = 0;                                // bit c: this lane's output c * 64 + lane is chosen
        for (int k = 0; k < top; ++k) {
            float best = -INFINITY; int bi = 0x7fffffff;
#pragma unroll
            for (int c = 0; c < NC; ++c) {
                const int i = c * 64 + lane;
                if (i < n && !(taken >> c & 1) && (zs[c] > best || bi == 0x7fffffff)) { best = zs[c]; bi = i; }
            }
#pragma unroll
            for (int o = 32; o > 0; o >>= 1) {
                const float ob = __shfl_xor(best, o, WAVE); const int oi = __shfl_xor(bi, o, WAVE);
                if (oi != 0x7fffffff && (bi == 0x7fffffff || ob > best || (ob == best && oi < bi))) { best = ob; bi = oi; }
            }
            bi = __builtin_amdgcn_readfirstlane(bi);       // (one choice for the wave, also where logits are no numbers)
            best = __shfl(best, 0, WAVE);
            if (k == 0) mx = best;
            sum += expf(best - mx);
            if ((bi & 63) == lane) taken |= 1u << (bi >> 6);
        }
        int rank = 0;
#pragma unroll
        for (int c = 0; c < NC; ++c) {
            const bool mine = taken >> c & 1;
            const uint64_t mask = __builtin_amdgcn_ballot_w64(mine);
            if (mine) {
                const int64_t at = (int64_t)t * top + rank + __builtin_popcountll(mask & ((1ull << lane) - 1));
                chosen[at] = c * 64 + lane;
                picked[at - (int64_t)t0 * top] = c * 64 + lane;
                weights[at] = expf(zs[c] - mx) / sum * scale;
            }
            rank += __builtin_popcountll(mask);
        }
    }
    if (gridDim.x == 1 && p.counts) {
        __syncthreads();
        const int pairs = n_tokens * top;
        // a wave an expert: up to 16 * top pairs, 64 at a time
        for (int e = wave; e < n; e += ROUTER_WAVES) {
            int before = 0, total = 0;
            for (int i0 = 0; i0 < pairs; i0 += 64) {
                const int v = i0 + lane < pairs ? picked[i0 + lane] : 0x7fffffff;
                before += __builtin_popcountll(__builtin_amdgcn_ballot_w64(v < e));
                total += __builtin_popcountll(__builtin_amdgcn_ballot_w64(v == e));
            }
            int at = before;
            for (int i0 = 0; i0 < pairs && total; i0 += 64) {
                const bool mine = i0 + lane < pairs && picked[i0 + lane] == e;
                const uint64_t mask = __builtin_amdgcn_ballot_w64(mine);
                if (mine) {
                    const int s = at + __builtin_popcountll(mask & ((1ull << lane) - 1));
                    p.row_of[s] = (i0 + lane) / top;
                    p.slot_of[i0 + lane] = s;
                }
                at += __builtin_popcountll(mask);
            }
            if (lane == 0) { p.counts[e] = total; p.offsets[e] = before; }
        }
    }
}

// counts (and the other three) not null with up to 16 tokens: the pairs are sorted too.
extern "C" int li_router(const void* X, const void* Wt, int dt, const float* bias, int parts, int n_tokens, int K, int n, int top, float scale,
                         int* chosen, float* weights, int* counts, int* offsets, int* row_of, int* slot_of, hipStream_t stream) {
    if (n_tokens <= 0) return LI_OK;
    if (!X || !Wt || !chosen || !weights || n < 1 || top < 1 || top > n || parts < 1 || parts > 3) return LI_BAD_ARG;
    if (n > ROUTER_MAX || K < 32 || K % 32 || ((uintptr_t)X & 15) || ((uintptr_t)Wt & 15)) return LI_UNSUPPORTED;
    if (counts && (n_tokens > 16 || !offsets || !row_of || !slot_of)) return LI_BAD_ARG;
    const Pairs p{counts, offsets, row_of, slot_of};
    const size_t lds = (size_t)16 * (n + top) * sizeof(float);
    if (lds > 40 * 1024) return LI_UNSUPPORTED;
    const int blocks = (n_tokens + 15) / 16;
#define GO(T, NC) router_kernel<T, NC><<<blocks, 64 * ROUTER_WAVES, lds, stream>>>((const T*)X, (const T*)Wt, bias, parts, n_tokens, K, n, top, scale, chosen, weights, p)
    if (dt == DT_F16) { if (n <= 64) GO(f16, 1); else GO(f16, 8); }
    else if (dt == DT_BF16) { if (n <= 64) GO(bf16, 1); else GO(bf16, 8); }
#undef GO
    else return LI_BAD_ARG;
    LI_CHECK_LAUNCH();
    return LI_OK;
}

// ---------------------------------------------------------------------------
// An expert's product on its own pairs' rows, few of them: C[pair] = epilogue(W_e X[row_of[pair]]) for the pairs of
// the blockIdx.y-th expert that has any (row_of null: X[pair]).  gemv_tiled's structure: a workgroup takes 16 rows of W_e
// for the whole of K, its KW waves share K; 16 MT pairs at a time (W is read again, from the caches, for the next ones).
// ---------------------------------------------------------------------------
template <class T, int MT, int KW>
__global__ __launch_bounds__(64 * KW) void experts_gemv_kernel(const T* __restrict__ X, const T* __restrict__ Wt, int K,
                                                               int64_t w_stride, Epilogue e, int n_experts,
                                                               const int* __restrict__ counts, const int* __restrict__ offsets,
                                                               const int* __restrict__ row_of) {
    typedef typename Vec<T>::v8 v8;
    constexpr int U = MT == 1 ? 8 : 4;
    __shared__ float part[KW][MT][64][4];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r = lane & 15, g = lane >> 4;
    int expert = -1, nth = blockIdx.y;
    for (int e0 = 0; e0 < n_experts; e0 += 64) {
        uint64_t any = __builtin_amdgcn_ballot_w64(e0 + lane < n_experts && counts[min(e0 + lane, n_experts - 1)] > 0);
        const int here = __builtin_popcountll(any);
        if (nth < here) {
            for (int i = 0; i < nth; ++i) any &= any - 1;
            expert = e0 + __builtin_ctzll(any);
            break;
        }
        nth -= here;
    }
    if (expert < 0) return;
    const int count = counts[expert], row0 = offsets[expert];
    Wt += expert * w_stride;
    const int tile = blockIdx.x, steps = K >> 5;
    const int per = (steps + KW - 1) / KW, s_begin = wave * per, s_end = min(steps, s_begin + per);
    const T* wt = Wt + ((int64_t)tile * steps * 64 + lane) * 8;
    e.M = row0 + count;
    for (int r0 = 0; r0 < count; r0 += 16 * MT) {
        bool have[MT];
        const T* xrow[MT];
        f32x4 acc[MT];
#pragma unroll
        for (int j = 0; j < MT; ++j) {
            have[j] = r0 + 16 * j + r < count;
            const int pair = row0 + (have[j] ? r0 + 16 * j + r : 0);
            xrow[j] = X + (int64_t)(row_of ? row_of[pair] : pair) * K + 8 * g;
            acc[j] = f32x4{0.f, 0.f, 0.f, 0.f};
        }
        for (int s0 = s_begin; s0 < s_end; s0 += U) {
            v8 a[U], b[U][MT];
#pragma unroll
            for (int u = 0; u < U; ++u) {
                const bool in = s0 + u < s_end;
                const v8 z = {};
                a[u] = in ? *(const v8*)(wt + (int64_t)(s0 + u) * 512) : z;
#pragma unroll
                for (int j = 0; j < MT; ++j) b[u][j] = in && have[j] ? *(const v8*)(xrow[j] + (s0 + u) * 32) : z;
            }
#pragma unroll
            for (int u = 0; u < U; ++u)
#pragma unroll
                for (int j = 0; j < MT; ++j) acc[j] = mfma16(a[u], b[u][j], acc[j]);
        }
        if (r0) __syncthreads();                           // wave 0 has read the sums of the pairs before
#pragma unroll
        for (int j = 0; j < MT; ++j)
#pragma unroll
            for (int q = 0; q < 4; ++q) part[wave][j][lane][q] = acc[j][q];
        __syncthreads();
        if (wave == 0) {
#pragma unroll
            for (int j = 0; j < MT; ++j) {
                float v[4];
#pragma unroll
                for (int q = 0; q < 4; ++q) {
                    v[q] = part[0][j][lane][q];
                    for (int w = 1; w < KW; ++w) v[q] += part[w][j][lane][q];
                }
                if (have[j]) epilogue4_base(e, row0 + r0 + 16 * j + r, tile * 16 + 4 * g, v);
            }
        }
    }
}

// mode: EPI_STORE or EPI_SWIGLU.  Wt: the experts' tiled matrices [N, K] one behind the other, w_stride elements apart.
extern "C" int li_experts_gemv(const void* X, const void* Wt, int dt, void* C, int out_dt, int mode, int n_pairs, int N, int K,
                               int64_t w_stride, int n_experts, const int* counts, const int* offsets, const int* row_of,
                               hipStream_t stream) {
    int rc = check_common(X, Wt, C, n_pairs, N, K, mode, out_dt);
    if (rc) return rc;
    if ((dt != DT_F16 && dt != DT_BF16) || (mode != EPI_STORE && mode != EPI_SWIGLU) || !counts || !offsets || n_experts < 1) return LI_BAD_ARG;
    if (K % 32 || ((uintptr_t)X & 15) || ((uintptr_t)Wt & 15) || w_stride % 8) return LI_UNSUPPORTED;
    if (n_pairs == 0) return LI_OK;
    Epilogue e;
    rc = make_epilogue(e, C, mode, out_dt, n_pairs, N, nullptr);
    if (rc) return rc;
    dim3 grid((N + 15) / 16, min(n_experts, n_pairs));
#define GO(T, MT, KW)                                                                                                             \
    experts_gemv_kernel<T, MT, KW><<<grid, 64 * KW, 0, stream>>>((const T*)X, (const T*)Wt, K, w_stride, e, n_experts, counts, offsets, row_of)
#define BY_K(T, MT) do { if (K >= 2048) GO(T, MT, 8); else GO(T, MT, 4); } while (0)
#define BY_M(T) do { if (n_pairs <= 8 * n_experts) BY_K(T, 1); else BY_K(T, 2); } while (0)
    if (dt == DT_F16) BY_M(f16); else BY_M(bf16);
#undef BY_M
#undef BY_K
#undef GO
    LI_CHECK_LAUNCH();
    return LI_OK;
}

// ---------------------------------------------------------------------------
// out[t] (+)= sum over j < top of weights[t][j] * rows[slot_of[t][j]], in the order of j.
// ---------------------------------------------------------------------------
__global__ void pair_sum_kernel(const float* __restrict__ rows, const int* __restrict__ slot_of, const float* __restrict__ weights,
                                int top, int width, float* __restrict__ out, int add) {
    const int64_t t = blockIdx.x;
    for (int i = blockIdx.y * blockDim.x + threadIdx.x; i < width; i += gridDim.y * blockDim.x) {
        float v = add ? out[t * width + i] : 0.f;
        for (int j = 0; j < top; ++j) {
            const int s = slot_of[t * top + j];
            if (s >= 0) v += weights[t * top + j] * rows[(int64_t)s * width + i];
        }
        out[t * width + i] = v;
    }
}

extern "C" int li_pair_sum(const float* rows, const int* slot_of, const float* weights, int n_tokens, int top, int width, float* out,
                           int add, hipStream_t stream) {
    if (n_tokens <= 0 || width <= 0) return LI_OK;
    if (!rows || !slot_of || !weights || !out || top < 1) return LI_BAD_ARG;
    dim3 grid(n_tokens, n_tokens >= 1024 ? 1 : (width + 1023) / 1024);
    pair_sum_kernel<<<grid, 256, 0, stream>>>(rows, slot_of, weights, top, width, out, add);
    LI_CHECK_LAUNCH();
    return LI_OK;
}
