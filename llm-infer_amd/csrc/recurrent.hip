// Recurrent mixers with a float32 state per sequence: the gated delta rule, the selective scan with a decay for every
// channel and state, and the time mixing with a decay for every key channel and a bonus for the current token.  Each
// has a kernel that walks a sequence's tokens in order (decode steps, float32 models), and a form for the prompts of a
// 16-bit model that works on many tokens at a time.  Every size is a run-time value.  Unit norms, decays and their
// logarithms, step sizes, gates of the recurrences and the states are float32 whatever the type of the matrices.
#include "common.h"

__device__ __forceinline__ float rc_sigmoid(float z) { return 1.f / (1.f + expf(-z)); }
__device__ __forceinline__ float rc_silu(float z) { return z / (1.f + expf(-z)); }
__device__ __forceinline__ float rc_softplus(float z) { return z > 20.f ? z : log1pf(expf(z)); }

#define DISPATCH_T(dt, CALL)                                     \
    do {                                                         \
        if ((dt) == DT_F32) { typedef float T; CALL; }           \
        else if ((dt) == DT_F16) { typedef f16 T; CALL; }        \
        else if ((dt) == DT_BF16) { typedef bf16 T; CALL; }      \
        else return LI_BAD_ARG;                                  \
    } while (0)

// The tokens of a step: row i of the step stands at pos[i] of the sequence in slot tok_slot[i]; sequence s brings
// seq_qlen[s] rows from seq_qstart[s] on (both null: one row a sequence, row s).
struct Steps {
    const int* pos;
    const int* tok_slot;
    const int* seq_slot;
    const int* seq_qstart;
    const int* seq_qlen;
};

// Segments of a step's sequences that run side by side: segment g is seg_n[g] tokens from the seg_t0[g]-th token of
// sequence seg_seq[g] on; sequence s has seq_nseg[s] of them from seq_seg0[s] on.
struct Segments {
    const int* seg_seq;
    const int* seg_t0;
    const int* seg_n;
    const int* seq_seg0;
    const int* seq_nseg;
};

// One column of float32 rows through a causal convolution over time (weights [channels, taps], the last tap the
// token's own), then silu: inputs before the first token that a sequence brings to the step come from `hist` [slots,
// taps - 1, channels] (oldest first), before position 0 they are zero.  `inside`: how many tokens before this one its
// sequence has in this step (at most taps - 1 of them matter).
struct Conv {
    const float* w;
    const float* b;          // [channels] or null
    const float* hist;
    int taps, channels;
};
__device__ __forceinline__ int tokens_inside(const int* tok_slot, int t, int slot, int taps) {
    int inside = 0;
    while (inside < taps - 1 && t - inside - 1 >= 0 && tok_slot[t - inside - 1] == slot) ++inside;
    return inside;
}
__device__ __forceinline__ float conv_silu_at(const float* row, int64_t stride, int c, const Conv& cv, int inside, int p, int slot) {
    float acc = cv.b ? cv.b[c] : 0.f;
    const float* h = cv.hist + (int64_t)slot * (cv.taps - 1) * cv.channels;
    for (int back = 0; back < cv.taps; ++back) {
        float u = 0.f;
        if (back <= inside) u = row[c - back * stride];
        else if (p - back >= 0) u = h[(int64_t)(cv.taps - 1 - (back - inside)) * cv.channels + c];
        acc += cv.w[(int64_t)c * cv.taps + (cv.taps - 1 - back)] * u;
    }
    return rc_silu(acc);
}

// ---------------------------------------------------------------------------
// The gated delta rule.  Per sequence and head h with key head e = h / (H / G), S [d, dv] float32:
//   S <- g S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q
// q, k, v: columns of the rows `proj` (from col0 on: q [G, d], k [G, d], v [H, dv]) behind a convolution and silu; q
// and k then unit vectors, x / sqrt(sum x^2 + 1e-6), q times d^(-1/2); beta = sigmoid(proj[b_col + h]),
// g = exp(-exp(A_log[h]) softplus(proj[a_col + h] + dt_bias[h])).
// delta_prep_kernel: a wave a (token, key head), (token, 64 values) or (token) for the gates.  `qkv` [T, 2 G d + H dv]
// float32 receives q and k as unit vectors and v; `gates` [T, H, 2] log g and beta; `kq` [T, G] k . q.
// ---------------------------------------------------------------------------
#define DELTA_UNIT_EPS 1e-6f
#define DELTA_MAXV 4             // keys up to 64 * DELTA_MAXV wide

__global__ __launch_bounds__(256) void delta_prep_kernel(const float* __restrict__ proj, int stride, int col0, int b_col,
                                                         int a_col, Conv cv, Steps st, const float* __restrict__ A_log,
                                                         const float* __restrict__ dt_bias, float* __restrict__ qkv,
                                                         float* __restrict__ gates, float* __restrict__ kq, int H, int G,
                                                         int d, int dv) {
    const int t = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int p = st.pos[t], slot = st.tok_slot[t], inside = tokens_inside(st.tok_slot, t, slot, cv.taps);
    const float* row = proj + (int64_t)t * stride + col0;
    float* out = qkv + (int64_t)t * cv.channels;
    const int nv = (H * dv + 63) / 64, units = G + nv + 1;
    const float qs = 1.f / sqrtf((float)d);
    for (int u = blockIdx.y * 4 + wave; u < units; u += gridDim.y * 4) {
        if (u < G) {
            float q[DELTA_MAXV], k[DELTA_MAXV], sq = 0.f, sk = 0.f, dot = 0.f;
#pragma unroll
            for (int v = 0; v < DELTA_MAXV; ++v) {
                const int i = v * 64 + lane;
                q[v] = k[v] = 0.f;
                if (i < d) {
                    q[v] = conv_silu_at(row, stride, u * d + i, cv, inside, p, slot);
                    k[v] = conv_silu_at(row, stride, (G + u) * d + i, cv, inside, p, slot);
                }
                sq += q[v] * q[v];
                sk += k[v] * k[v];
            }
            const float rq = qs / sqrtf(wave_sum(sq) + DELTA_UNIT_EPS), rk = 1.f / sqrtf(wave_sum(sk) + DELTA_UNIT_EPS);
#pragma unroll
            for (int v = 0; v < DELTA_MAXV; ++v) {
                const int i = v * 64 + lane;
                q[v] *= rq;
                k[v] *= rk;
                dot += q[v] * k[v];
                if (i < d) { out[u * d + i] = q[v]; out[(G + u) * d + i] = k[v]; }
            }
            dot = wave_sum(dot);
            if (lane == 0) kq[(int64_t)t * G + u] = dot;
        } else if (u < G + nv) {
            const int c = 2 * G * d + (u - G) * 64 + lane;
            if (c < cv.channels) out[c] = conv_silu_at(row, stride, c, cv, inside, p, slot);
        } else {
            const float* r = proj + (int64_t)t * stride;
            for (int h = lane; h < H; h += 64) {
                gates[((int64_t)t * H + h) * 2] = -expf(A_log[h]) * rc_softplus(r[a_col + h] + dt_bias[h]);
                gates[((int64_t)t * H + h) * 2 + 1] = rc_sigmoid(r[b_col + h]);
            }
        }
    }
}

// Token by token: a workgroup of 4 waves per (sequence, head, 64 columns of S); a lane keeps one column's NR rows of
// its wave's share in registers.  Both read-outs come from the state before the token, a = S^T k and c = S^T q:
// u = beta (v - g a),  o = g c + u (k . q),  S <- g S + k u^T; the waves' shares of a and c meet in LDS.
#define SCAN_WAVES 4

template <int NR>
__global__ __launch_bounds__(64 * SCAN_WAVES) void delta_scan_kernel(const float* __restrict__ qkv, const float* __restrict__ gates,
                                                                     const float* __restrict__ kq, float* __restrict__ state,
                                                                     Steps st, float* __restrict__ y, int H, int G, int d, int dv) {
    constexpr int DP = NR * SCAN_WAVES;                  // rows of S, padded
    __shared__ __attribute__((aligned(16))) float sk[3][DP], sq[3][DP];
    __shared__ float part[2][SCAN_WAVES][2][64];
    const int seq = blockIdx.x, h = blockIdx.y, e = h / (H / G), tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int col = blockIdx.z * 64 + lane, C = 2 * G * d + H * dv, r0 = wave * NR;
    const int q0 = st.seq_qstart ? st.seq_qstart[seq] : seq, n = st.seq_qlen ? st.seq_qlen[seq] : 1;
    if (n <= 0) return;
    const bool live = col < dv;
    float* S = state + (((int64_t)st.seq_slot[seq] * H + h) * d) * dv + col;
    float s[NR];
#pragma unroll
    for (int r = 0; r < NR; ++r) s[r] = (live && r0 + r < d) ? S[(int64_t)(r0 + r) * dv] : 0.f;
    auto stage = [&](int t) {
        const float* row = qkv + (int64_t)(q0 + t) * C;
        for (int i = tid; i < DP; i += 64 * SCAN_WAVES) {
            sq[t % 3][i] = i < d ? row[e * d + i] : 0.f;
            sk[t % 3][i] = i < d ? row[(G + e) * d + i] : 0.f;
        }
    };
    stage(0);
    __syncthreads();
    for (int t = 0; t < n; ++t) {
        const int64_t tok = q0 + t;
        const float v = live ? qkv[tok * C + 2 * G * d + h * dv + col] : 0.f;
        const float g = expf(gates[(tok * H + h) * 2]), beta = gates[(tok * H + h) * 2 + 1], dot = kq[tok * G + e];
        const float *k = sk[t % 3] + r0, *q = sq[t % 3] + r0;
        float a = 0.f, c = 0.f;
#pragma unroll
        for (int r = 0; r < NR; ++r) { a += s[r] * k[r]; c += s[r] * q[r]; }
        part[t & 1][wave][0][lane] = a;
        part[t & 1][wave][1][lane] = c;
        if (t + 1 < n) stage(t + 1);
        __syncthreads();
        a = c = 0.f;
#pragma unroll
        for (int w = 0; w < SCAN_WAVES; ++w) { a += part[t & 1][w][0][lane]; c += part[t & 1][w][1][lane]; }
        const float u = beta * (v - g * a);
        if (wave == 0 && live) y[tok * H * dv + h * dv + col] = g * c + u * dot;
#pragma unroll
        for (int r = 0; r < NR; ++r) s[r] = g * s[r] + k[r] * u;
    }
    if (live) {
#pragma unroll
        for (int r = 0; r < NR; ++r) if (r0 + r < d) S[(int64_t)(r0 + r) * dv] = s[r];
    }
}

extern "C" int li_delta_prep(const float* proj, int stride, int col0, int b_col, int a_col, const float* conv_w, int taps,
                             const float* hist, const int* pos, const int* tok_slot, const float* A_log, const float* dt_bias,
                             float* qkv, float* gates, float* kq, int n, int H, int G, int d, int dv, hipStream_t stream) {
    if (n <= 0) return LI_OK;
    if (H <= 0 || G <= 0 || H % G || d <= 0 || dv <= 0 || taps < 1 || taps > 16 || !hist) return LI_BAD_ARG;
    if (d > 64 * DELTA_MAXV) return LI_UNSUPPORTED;
    const int channels = 2 * G * d + H * dv;
    if (col0 < 0 || col0 + channels > stride || b_col < 0 || b_col + H > stride || a_col < 0 || a_col + H > stride) return LI_BAD_ARG;
    Conv cv{conv_w, nullptr, hist, taps, channels};
    Steps st{pos, tok_slot, nullptr, nullptr, nullptr};
    const int units = G + (H * dv + 63) / 64 + 1;
    delta_prep_kernel<<<dim3(n, (units + 3) / 4), 256, 0, stream>>>(proj, stride, col0, b_col, a_col, cv, st, A_log, dt_bias, qkv,
                                                                    gates, kq, H, G, d, dv);
    LI_CHECK_LAUNCH();
    return LI_OK;
}

extern "C" int li_delta_scan(const float* qkv, const float* gates, const float* kq, float* state, const int* seq_slot,
                             const int* seq_qstart, const int* seq_qlen, float* y, int n_seqs, int H, int G, int d, int dv,
                             hipStream_t stream) {
    if (n_seqs <= 0) return LI_OK;
    if (H <= 0 || G <= 0 || H % G || d <= 0 || dv <= 0) return LI_BAD_ARG;
    if (d > 64 * DELTA_MAXV) return LI_UNSUPPORTED;
    Steps st{nullptr, nullptr, seq_slot, seq_qstart, seq_qlen};
    dim3 grid(n_seqs, H, (dv + 63) / 64), block(64 * SCAN_WAVES);
#define GO(NR) delta_scan_kernel<NR><<<grid, block, 0, stream>>>(qkv, gates, kq, state, st, y, H, G, d, dv)
    if (d <= 16) GO(4); else if (d <= 32) GO(8); else if (d <= 64) GO(16); else if (d <= 128) GO(32); else GO(64);
#undef GO
    LI_CHECK_LAUNCH();
    return LI_OK;
}

// ---------------------------------------------------------------------------
// The selective scan with a decay for every channel and state.  Per sequence, channel c and state i:
//   dt_c = softplus(raw_c + bias_c);   S[c, i] <- exp(dt_c A[c, i]) S[c, i] + dt_c x_c B_i;
//   y_c = sum_i S[c, i] C_i + D_c x_c;   out_c = y_c silu(z_c)
// x [T, channels] and out in type T; raw [T, channels], B and C (columns b_col and c_col of the rows `bc`, the same for
// all channels) and z (columns of the rows `zr`) float32; A2 = A log2(e) [N, channels] (so that exp is one 2^x);
// the state is [slots, N, channels] float32.
// `parts` neighbouring lanes (a power of two) share a channel, NS of its states each in registers.  A workgroup's waves
// share B and C of SEL_TILE tokens in LDS; x, raw and z of the next tile are fetched while a tile is at work.
// PASS 0: a sequence's tokens in order.  A prompt may be walked in segments side by side instead: PASS 1 runs every
// segment from zero and leaves what it adds to the state and the sum of its step sizes (a segment's decay is
// exp(A sum dt)); sel_combine_kernel walks a sequence's segments in order and leaves the state before every segment
// where its contribution was; PASS 3 runs every segment again from there and writes out.
// ---------------------------------------------------------------------------
#define SEL_TILE 8
#define SEL_THREADS 128

template <class T, int NS, int PASS>
__global__ __launch_bounds__(SEL_THREADS) void sel_scan_kernel(
    const T* __restrict__ x, const float* __restrict__ raw, const float* __restrict__ dt_bias, const float* __restrict__ bc,
    int bc_stride, int b_col, int c_col, const float* __restrict__ zr, int z_stride, int z_col, const float* __restrict__ A2,
    const float* __restrict__ D, float* __restrict__ state, Steps st, Segments sg, float* __restrict__ seg_state,
    float* __restrict__ seg_dt, T* __restrict__ out, int channels, int N, int parts) {
    extern __shared__ __attribute__((aligned(16))) float sel_lds[];      // B [2][SEL_TILE][NP], then C
    const int NP = NS * parts;
    float *sb = sel_lds, *sc = sel_lds + 2 * SEL_TILE * NP;
    const int tid = threadIdx.x, part = tid & (parts - 1), i0 = part * NS;
    const int c = blockIdx.y * (SEL_THREADS / parts) + tid / parts;
    const bool live = c < channels;
    const int cc = live ? c : channels - 1;
    int q0, n;
    float* S;
    if (PASS == 0) {
        const int seq = blockIdx.x;
        q0 = st.seq_qstart ? st.seq_qstart[seq] : seq;
        n = st.seq_qlen ? st.seq_qlen[seq] : 1;
        S = state + (int64_t)st.seq_slot[seq] * N * channels + cc;
    } else {
        const int seg = blockIdx.x;
        q0 = st.seq_qstart[sg.seg_seq[seg]] + sg.seg_t0[seg];
        n = sg.seg_n[seg];
        S = seg_state + (int64_t)seg * N * channels + cc;
    }
    if (n <= 0) return;
    float s[NS], a[NS];
#pragma unroll
    for (int i = 0; i < NS; ++i) {
        s[i] = (PASS != 1 && i0 + i < N) ? S[(int64_t)(i0 + i) * channels] : 0.f;
        a[i] = i0 + i < N ? A2[(int64_t)(i0 + i) * channels + cc] : 0.f;
    }
    const float bias = dt_bias[cc], dc = D[cc];
    float sum_dt = 0.f;
    float xn[SEL_TILE], rn[SEL_TILE], zn[SEL_TILE];
    auto fetch = [&](int t0) {
#pragma unroll
        for (int k = 0; k < SEL_TILE; ++k) {
            const int64_t t = q0 + min(t0 + k, n - 1);
            xn[k] = to_f32(x[t * channels + cc]);
            rn[k] = raw[t * channels + cc];
            if (PASS != 1) zn[k] = zr[t * z_stride + z_col + cc];
        }
    };
    auto stage = [&](int t0, int buf) {
        for (int e = tid; e < SEL_TILE * NP; e += SEL_THREADS) {
            const int k = e / NP, i = e - k * NP;
            const float* row = bc + (int64_t)(q0 + min(t0 + k, n - 1)) * bc_stride;
            sb[buf * SEL_TILE * NP + e] = i < N ? row[b_col + i] : 0.f;
            if (PASS != 1) sc[buf * SEL_TILE * NP + e] = i < N ? row[c_col + i] : 0.f;
        }
    };
    fetch(0);
    stage(0, 0);
    int buf = 0;
    for (int t0 = 0; t0 < n; t0 += SEL_TILE, buf ^= 1) {
        __syncthreads();
        float xt[SEL_TILE], rt[SEL_TILE], zt[SEL_TILE];
#pragma unroll
        for (int k = 0; k < SEL_TILE; ++k) { xt[k] = xn[k]; rt[k] = rn[k]; zt[k] = PASS != 1 ? zn[k] : 0.f; }
        if (t0 + SEL_TILE < n) { fetch(t0 + SEL_TILE); stage(t0 + SEL_TILE, buf ^ 1); }
#pragma unroll
        for (int k = 0; k < SEL_TILE; ++k) {
            if (t0 + k < n) {
                const float dt = rc_softplus(rt[k] + bias), dx = dt * xt[k];
                const float *B = sb + (buf * SEL_TILE + k) * NP + i0, *C = sc + (buf * SEL_TILE + k) * NP + i0;
                float acc = 0.f;
#pragma unroll
                for (int i = 0; i < NS; ++i) {
                    s[i] = __builtin_amdgcn_exp2f(dt * a[i]) * s[i] + dx * B[i];
                    if (PASS != 1) acc += s[i] * C[i];
                }
                sum_dt += dt;
                if (PASS != 1) for (int o = 1; o < parts; o <<= 1) acc += __shfl_xor(acc, o, WAVE);
                if (PASS != 1 && live && part == 0)
                    out[(int64_t)(q0 + t0 + k) * channels + c] = from_f32<T>((acc + dc * xt[k]) * rc_silu(zt[k]));
            }
        }
    }
    if (PASS != 3 && live) {
#pragma unroll
        for (int i = 0; i < NS; ++i) if (i0 + i < N) S[(int64_t)(i0 + i) * channels] = s[i];
        if (PASS == 1 && part == 0) seg_dt[(int64_t)blockIdx.x * channels + c] = sum_dt;
    }
}

// One thread per (state, channel): walks a sequence's segments in order.
__global__ void sel_combine_kernel(float* __restrict__ state, const int* __restrict__ seq_slot, Segments sg,
                                   float* __restrict__ seg_state, const float* __restrict__ seg_dt,
                                   const float* __restrict__ A2, int channels, int N) {
    const int seq = blockIdx.x, i = blockIdx.z, c = blockIdx.y * blockDim.x + threadIdx.x;
    if (c >= channels) return;
    const int g0 = sg.seq_seg0[seq], ng = sg.seq_nseg[seq];
    float* S = state + ((int64_t)seq_slot[seq] * N + i) * channels + c;
    const float a = A2[(int64_t)i * channels + c];
    float s = *S;
    for (int g = g0; g < g0 + ng; ++g) {
        float* L = seg_state + ((int64_t)g * N + i) * channels + c;
        const float own = *L;
        *L = s;
        s = __builtin_amdgcn_exp2f(a * seg_dt[(int64_t)g * channels + c]) * s + own;
    }
    *S = s;
}

extern "C" int li_sel_scan(const void* x, int dt, const float* raw, const float* dt_bias, const float* bc, int bc_stride, int b_col,
                           int c_col, const float* zr, int z_stride, int z_col, const float* A2, const float* D, float* state,
                           const int* seq_slot, const int* seq_qstart, const int* seq_qlen, void* out, int n_seqs, int channels,
                           int N, const int* seg_seq, const int* seg_t0, const int* seg_n, const int* seq_seg0,
                           const int* seq_nseg, int n_segs, float* seg_state, float* seg_dt, hipStream_t stream) {
    if (n_seqs <= 0) return LI_OK;
    if (channels <= 0 || N <= 0 || b_col < 0 || c_col < 0 || b_col + N > bc_stride || c_col + N > bc_stride || z_col < 0 ||
        z_col + channels > z_stride)
        return LI_BAD_ARG;
    if (N > 256) return LI_UNSUPPORTED;
    Steps st{nullptr, nullptr, seq_slot, seq_qstart, seq_qlen};
    Segments sg{seg_seq, seg_t0, seg_n, seq_seg0, seq_nseg};
    // states a lane (8, 16 or 32), lanes a channel
    const int ns = N <= 8 ? 8 : (N <= 16 ? 16 : 32);
    int parts = 1;
    while (parts * ns < N) parts *= 2;
    const int cb = (channels + SEL_THREADS / parts - 1) / (SEL_THREADS / parts);
    const size_t lds = (size_t)4 * SEL_TILE * ns * parts * sizeof(float);
#define GO1(NS, PASS, ITEMS) sel_scan_kernel<T, NS, PASS><<<dim3(ITEMS, cb), SEL_THREADS, lds, stream>>>((const T*)x, raw, dt_bias, bc, \
        bc_stride, b_col, c_col, zr, z_stride, z_col, A2, D, state, st, sg, seg_state, seg_dt, (T*)out, channels, N, parts)
#define GO(PASS, ITEMS)                                                                                                      \
    do {                                                                                                                     \
        if (ns == 8) GO1(8, PASS, ITEMS); else if (ns == 16) GO1(16, PASS, ITEMS); else GO1(32, PASS, ITEMS);                 \
    } while (0)
    if (n_segs <= 0) {
        DISPATCH_T(dt, GO(0, n_seqs));
    } else {
        if (!seq_qstart || !seq_qlen || !seg_seq || !seg_t0 || !seg_n || !seq_seg0 || !seq_nseg || !seg_state || !seg_dt) return LI_BAD_ARG;
        DISPATCH_T(dt, GO(1, n_segs));
        sel_combine_kernel<<<dim3(n_seqs, (channels + 255) / 256, N), 256, 0, stream>>>(state, seq_slot, sg, seg_state, seg_dt, A2,
                                                                                       channels, N);
        DISPATCH_T(dt, GO(3, n_segs));
    }
#undef GO
#undef GO1
    LI_CHECK_LAUNCH();
    return LI_OK;
}

// ---------------------------------------------------------------------------
// Time mixing with a decay for every key channel and a bonus for the current token.  Per sequence and head, S [d, d]
// float32 (rows: key channels), w = exp(-exp(raw)) per key channel:
//   o = (S + diag(u) k v^T)^T r;   S <- diag(w) S + k v^T
// r, k, v [T, H d] in type T, raw [T, H d] float32 (its bias included), u [H, d].
// A workgroup of 4 waves per (sequence or segment, head, 64 columns); a lane keeps its column's NR rows of its wave's share
// in registers, the waves' shares of o meet in LDS.  PASS 0, 1 and 3 as above (a segment's decay: exp of the sum of
// its logarithms, one a key channel).
// ---------------------------------------------------------------------------
template <class T, int NR, int PASS>
__global__ __launch_bounds__(64 * SCAN_WAVES) void wkv_scan_kernel(const T* __restrict__ r_, const T* __restrict__ k_,
                                                                   const T* __restrict__ v_, const float* __restrict__ raw,
                                                                   const float* __restrict__ bonus, float* __restrict__ state,
                                                                   Steps st, Segments sg, float* __restrict__ seg_state,
                                                                   float* __restrict__ seg_lw, float* __restrict__ y, int H, int d) {
    constexpr int DP = NR * SCAN_WAVES;
    __shared__ __attribute__((aligned(16))) float sr[3][DP], sk[3][DP], sw[3][DP];
    __shared__ float part[2][SCAN_WAVES][64], ruk[3][SCAN_WAVES];
    const int h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, col = blockIdx.z * 64 + lane, r0 = wave * NR;
    int q0, n;
    float* S;
    if (PASS == 0) {
        const int seq = blockIdx.x;
        q0 = st.seq_qstart ? st.seq_qstart[seq] : seq;
        n = st.seq_qlen ? st.seq_qlen[seq] : 1;
        S = state + (((int64_t)st.seq_slot[seq] * H + h) * d) * d + col;
    } else {
        const int seg = blockIdx.x;
        q0 = st.seq_qstart[sg.seg_seq[seg]] + sg.seg_t0[seg];
        n = sg.seg_n[seg];
        S = seg_state + (((int64_t)seg * H + h) * d) * d + col;
    }
    if (n <= 0) return;
    const bool live = col < d;
    float s[NR];
#pragma unroll
    for (int r = 0; r < NR; ++r) s[r] = (PASS != 1 && live && r0 + r < d) ? S[(int64_t)(r0 + r) * d] : 0.f;
    float lw_sum = 0.f;
    static_assert(DP <= 64 * SCAN_WAVES, "a thread a key channel");
    const float ub = tid < d ? bonus[h * d + tid] : 0.f;
    auto stage = [&](int t) {
        const int64_t at = (int64_t)(q0 + t) * H * d + h * d;
        float rr = 0.f, kk = 0.f, lw = 0.f;
        if (tid < d) {
            kk = to_f32(k_[at + tid]);
            lw = -expf(raw[at + tid]);
            if (PASS != 1) rr = to_f32(r_[at + tid]);
        }
        if (tid < DP) { sr[t % 3][tid] = rr; sk[t % 3][tid] = kk; sw[t % 3][tid] = expf(lw); }
        lw_sum += lw;
        if (PASS != 1) {
            const float b = wave_sum(rr * ub * kk);
            if (lane == 0) ruk[t % 3][wave] = b;
        }
    };
    stage(0);
    __syncthreads();
    for (int t = 0; t < n; ++t) {
        const int64_t tok = q0 + t;
        const float v = live ? to_f32(v_[tok * H * d + h * d + col]) : 0.f;
        const float *k = sk[t % 3] + r0, *rr = sr[t % 3] + r0, *w = sw[t % 3] + r0;
        float a = 0.f;
#pragma unroll
        for (int r = 0; r < NR; ++r) {
            if (PASS != 1) a += s[r] * rr[r];
            s[r] = w[r] * s[r] + k[r] * v;
        }
        if (PASS != 1) part[t & 1][wave][lane] = a;
        if (t + 1 < n) stage(t + 1);
        __syncthreads();
        if (PASS != 1 && wave == 0 && live) {
            float o = 0.f, b = 0.f;
#pragma unroll
            for (int i = 0; i < SCAN_WAVES; ++i) { o += part[t & 1][i][lane]; b += ruk[t % 3][i]; }
            y[tok * H * d + h * d + col] = o + b * v;
        }
    }
    if (PASS != 3 && live) {
#pragma unroll
        for (int r = 0; r < NR; ++r) if (r0 + r < d) S[(int64_t)(r0 + r) * d] = s[r];
    }
    if (PASS == 1 && blockIdx.z == 0 && tid < d) seg_lw[((int64_t)blockIdx.x * H + h) * d + tid] = lw_sum;
}

// One thread per element of a head's state: walks a sequence's segments in order, a decay a key channel.
__global__ void wkv_combine_kernel(float* __restrict__ state, const int* __restrict__ seq_slot, Segments sg,
                                   float* __restrict__ seg_state, const float* __restrict__ seg_lw, int H, int d) {
    const int seq = blockIdx.x, h = blockIdx.y, e = blockIdx.z * blockDim.x + threadIdx.x, per = d * d;
    if (e >= per) return;
    const int g0 = sg.seq_seg0[seq], ng = sg.seq_nseg[seq], row = e / d;
    float* S = state + ((int64_t)seq_slot[seq] * H + h) * per + e;
    float s = *S;
    for (int g = g0; g < g0 + ng; ++g) {
        float* L = seg_state + ((int64_t)g * H + h) * per + e;
        const float own = *L;
        *L = s;
        s = expf(seg_lw[((int64_t)g * H + h) * d + row]) * s + own;
    }
    *S = s;
}

extern "C" int li_wkv_scan(const void* r, const void* k, const void* v, int dt, const float* raw, const float* bonus, float* state,
                           const int* seq_slot, const int* seq_qstart, const int* seq_qlen, float* y, int n_seqs, int H, int d,
                           const int* seg_seq, const int* seg_t0, const int* seg_n, const int* seq_seg0, const int* seq_nseg,
                           int n_segs, float* seg_state, float* seg_lw, hipStream_t stream) {
    if (n_seqs <= 0) return LI_OK;
    if (H <= 0 || d <= 0) return LI_BAD_ARG;
    if (d > 256) return LI_UNSUPPORTED;
    Steps st{nullptr, nullptr, seq_slot, seq_qstart, seq_qlen};
    Segments sg{seg_seq, seg_t0, seg_n, seq_seg0, seq_nseg};
#define GO1(NR, PASS, ITEMS) wkv_scan_kernel<T, NR, PASS><<<dim3(ITEMS, H, (d + 63) / 64), 64 * SCAN_WAVES, 0, stream>>>((const T*)r, \
        (const T*)k, (const T*)v, raw, bonus, state, st, sg, seg_state, seg_lw, y, H, d)
#define GO(PASS, ITEMS)                                                                                               \
    do {                                                                                                              \
        if (d <= 16) GO1(4, PASS, ITEMS); else if (d <= 32) GO1(8, PASS, ITEMS); else if (d <= 64) GO1(16, PASS, ITEMS); \
        else if (d <= 128) GO1(32, PASS, ITEMS); else GO1(64, PASS, ITEMS);                                            \
    } while (0)
    if (n_segs <= 0) {
        DISPATCH_T(dt, GO(0, n_seqs));
    } else {
        if (!seq_qstart || !seq_qlen || !seg_seq || !seg_t0 || !seg_n || !seq_seg0 || !seq_nseg || !seg_state || !seg_lw) return LI_BAD_ARG;
        DISPATCH_T(dt, GO(1, n_segs));
        wkv_combine_kernel<<<dim3(n_seqs, H, (d * d + 255) / 256), 256, 0, stream>>>(state, seq_slot, sg, seg_state, seg_lw, H, d);
        DISPATCH_T(dt, GO(3, n_segs));
    }
#undef GO
#undef GO1
    LI_CHECK_LAUNCH();
    return LI_OK;
}
