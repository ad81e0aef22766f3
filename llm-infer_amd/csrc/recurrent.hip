// Recurrent mixers with a float32 state per sequence: the gated delta rule, the selective scan with a decay for every
// channel and state, and the time mixing with a decay for every key channel and a bonus for the current token.  Each
// has a kernel that walks a sequence's tokens in order (decode steps, float32 models); for the prompts of a 16-bit model
// the selective scan runs in segments side by side, the other two in recurrent_chunks.hip.  Every size is a run-time value.  Unit norms, decays and their
// logarithms, step sizes, gates of the recurrences and the states are float32 whatever the type of the matrices.
#include "common.h"
#include "conv.h"

__device__ __forceinline__ float rc_sigmoid(float z) { return 1.f / (1.f + expf(-z)); }
__device__ __forceinline__ float rc_silu(float z) { return z / (1.f + expf(-z)); }
// log(1 + e^z) = max(z, 0) + log(1 + u), u = e^-|z|; with w = 1 + u as rounded, log(1 + u) = log(w) u / (w - 1) to the last
// bits (the rounding of w cancels), and u itself where w is 1.
__device__ __forceinline__ float rc_softplus(float z) {
    const float u = __builtin_amdgcn_exp2f(-fabsf(z) * 1.4426950408889634f), w = 1.f + u, d = w - 1.f;
    const float l = d == 0.f ? u : __builtin_amdgcn_logf(w) * 0.6931471805599453f * u * __builtin_amdgcn_rcpf(d);
    return fmaxf(z, 0.f) + l;
}

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

// ---------------------------------------------------------------------------
// The gated delta rule.  Per sequence and head h with key head e = h / (H / G), S [d, dv] float32:
//   S <- g S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q
// q, k, v: columns of the rows `proj` (from col0 on: q [G, d], k [G, d], v [H, dv]) behind a convolution and silu; q
// and k then unit vectors, x / sqrt(sum x^2 + 1e-6), q times d^(-1/2); beta = sigmoid(proj[b_col + h]),
// g = exp(-exp(A_log[h]) softplus(proj[a_col + h] + dt_bias[h])).
// delta_prep_kernel: a wave a key head, 64 values or the gates, for `tile` consecutive tokens of the step; the gates go to
// `gates` [T, H, 2], log g (no less than LOG_DECAY_MIN, whose exponential is 0 next to anything) and beta.  For the kernel
// that walks token by token: q and k as unit vectors and v to `rows` [T, 2 G d + H dv] float32, k . q to `aux` [T, G].  For
// the chunked kernels (HALF): q, k and v behind silu to `rows` in bfloat16, d^(-1/2) / |q| and 1 / |k| of what was written to
// `aux` [T, G, 2].
// ---------------------------------------------------------------------------
#define DELTA_UNIT_EPS 1e-6f
#define DELTA_MAXV 4             // keys up to 64 * DELTA_MAXV wide
#define LOG_DECAY_MIN -88.f

struct DeltaPrep {
    const float* proj;
    int stride, col0, b_col, a_col;
    const float* w;              // [channels, taps]
    float* hist;                 // [slots, taps - 1, channels]
    const int* pos;
    const int* tok_slot;
    const float* A_log;
    const float* dt_bias;
    void* rows;
    float* gates;
    float* aux;
    int n, taps, H, G, d, dv, tile;
    int single;                  // every sequence brings one token: the history is brought up to date here
};

// Up to NV channels a lane, c0 + 64 v + lane, from token to token.
template <int TAPS, int NV>
struct ConvLanes {
    static constexpr int K = TAPS ? TAPS : 1;
    ConvWindow<K> win[NV];
    float w[NV][K];
    __device__ __forceinline__ void weights(const DeltaPrep& p, int c0, int lane, int count) {
        if (TAPS) {
#pragma unroll
            for (int v = 0; v < NV; ++v)
                if (v * 64 + lane < count) {
#pragma unroll
                    for (int j = 0; j < K; ++j) w[v][j] = p.w[(int64_t)(c0 + v * 64 + lane) * K + j];
                }
        }
    }
    // silu of the convolution at token t, 0 beyond `count`
    __device__ __forceinline__ void at(const DeltaPrep& p, int channels, int c0, int lane, int count, int t, int slot, bool fresh, int inside,
                                       float (&out)[NV]) {
        float* h = p.hist + (int64_t)slot * (p.taps - 1) * channels;
#pragma unroll
        for (int v = 0; v < NV; ++v) {
            out[v] = 0.f;
            if (v * 64 + lane < count) {
                const int c = c0 + v * 64 + lane;
                const float* x = p.proj + (int64_t)t * p.stride + p.col0 + c;
                float acc;
                if (TAPS) {
                    if (fresh) win[v].start(x, p.stride, inside, p.pos[t], h, channels, c);
                    else win[v].next(*x);
                    acc = win[v].sum(w[v], 0.f);
                    if (p.single) win[v].keep(h, channels, c);
                } else {
                    acc = conv_at(x, p.stride, inside, p.pos[t], h, channels, c, p.w, p.taps, 0.f);
                    if (p.single) conv_keep(*x, h, channels, c, p.taps);
                }
                out[v] = rc_silu(acc);
            }
        }
    }
};

template <int TAPS, bool HALF, int NV>
__global__ __launch_bounds__(256) void delta_prep_kernel(DeltaPrep p) {
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), H = p.H, G = p.G, d = p.d;
    const int t0 = blockIdx.x * p.tile, t1 = min(p.n, t0 + p.tile), channels = 2 * G * d + H * p.dv;
    const int nv = (H * p.dv + 63) / 64, units = G + nv + 1, u = blockIdx.y * 4 + wave;
    if (u >= units) return;
    const float qs = 1.f / sqrtf((float)d);
    int last = -1;
    if (u < G) {
        ConvLanes<TAPS, NV> cq, ck;
        cq.weights(p, u * d, lane, d);
        ck.weights(p, (G + u) * d, lane, d);
        for (int t = t0; t < t1; ++t) {
            const int slot = p.tok_slot[t];
            const bool fresh = slot != last;
            const int inside = !p.single && (fresh || !TAPS) ? conv_inside(p.tok_slot, t, slot, p.taps) : 0;
            last = slot;
            float q[NV], k[NV], sq = 0.f, sk = 0.f;
            cq.at(p, channels, u * d, lane, d, t, slot, fresh, inside, q);
            ck.at(p, channels, (G + u) * d, lane, d, t, slot, fresh, inside, k);
#pragma unroll
            for (int v = 0; v < NV; ++v) {
                if (HALF) { q[v] = (float)(bf16)q[v]; k[v] = (float)(bf16)k[v]; }
                sq += q[v] * q[v];
                sk += k[v] * k[v];
            }
            const float rq = qs / sqrtf(wave_sum(sq) + DELTA_UNIT_EPS), rk = 1.f / sqrtf(wave_sum(sk) + DELTA_UNIT_EPS);
            if (HALF) {
                bf16* out = (bf16*)p.rows + (int64_t)t * channels;
#pragma unroll
                for (int v = 0; v < NV; ++v) {
                    const int i = v * 64 + lane;
                    if (i < d) { out[u * d + i] = (bf16)q[v]; out[(G + u) * d + i] = (bf16)k[v]; }
                }
                if (lane == 0) { p.aux[((int64_t)t * G + u) * 2] = rq; p.aux[((int64_t)t * G + u) * 2 + 1] = rk; }
            } else {
                float* out = (float*)p.rows + (int64_t)t * channels;
                float dot = 0.f;
#pragma unroll
                for (int v = 0; v < NV; ++v) {
                    const int i = v * 64 + lane;
                    q[v] *= rq;
                    k[v] *= rk;
                    dot += q[v] * k[v];
                    if (i < d) { out[u * d + i] = q[v]; out[(G + u) * d + i] = k[v]; }
                }
                dot = wave_sum(dot);
                if (lane == 0) p.aux[(int64_t)t * G + u] = dot;
            }
        }
    } else if (u < G + nv) {
        const int c0 = 2 * G * d + (u - G) * 64, count = min(64, channels - c0);
        ConvLanes<TAPS, 1> cv;
        cv.weights(p, c0, lane, count);
        for (int t = t0; t < t1; ++t) {
            const int slot = p.tok_slot[t];
            const bool fresh = slot != last;
            const int inside = !p.single && (fresh || !TAPS) ? conv_inside(p.tok_slot, t, slot, p.taps) : 0;
            last = slot;
            float v[1];
            cv.at(p, channels, c0, lane, count, t, slot, fresh, inside, v);
            if (lane < count) {
                const int64_t at = (int64_t)t * channels + c0 + lane;
                if (HALF) ((bf16*)p.rows)[at] = (bf16)v[0];
                else ((float*)p.rows)[at] = v[0];
            }
        }
    } else {
        for (int t = t0; t < t1; ++t) {
            const float* r = p.proj + (int64_t)t * p.stride;
            for (int h = lane; h < H; h += 64) {
                float* g = p.gates + ((int64_t)t * H + h) * 2;
                g[0] = fmaxf(-expf(p.A_log[h]) * rc_softplus(r[p.a_col + h] + p.dt_bias[h]), LOG_DECAY_MIN);
                g[1] = rc_sigmoid(r[p.b_col + h]);
            }
        }
    }
}

// What stands behind a recurrence: every head's o divided by its root mean square over dv, times a weight (`w_shared`: dv
// numbers for all heads, else H dv) and the silu of a gate (float32 rows), in type `dt`.  w null: o as it is, float32.
struct HeadOut {
    const float* w;
    int w_shared;
    const float* gate;
    int64_t gate_stride;
    float eps;
    void* out;
    int dt;
};
// element `i` of head h of token t (the heads' elements side by side, n = H dv of them), ss the head's sum of squares
__device__ __forceinline__ void store_head(const HeadOut& ho, int64_t t, int n, int h, int dv, int i, float o, float ss) {
    const int64_t at = t * n + h * dv + i;
    if (!ho.w) { ((float*)ho.out)[at] = o; return; }
    const float z = ho.gate[t * ho.gate_stride + h * dv + i];
    const float v = o / sqrtf(ss / (float)dv + ho.eps) * ho.w[ho.w_shared ? i : h * dv + i] * rc_silu(z);
    if (ho.dt == DT_F32) ((float*)ho.out)[at] = v;
    else if (ho.dt == DT_F16) ((f16*)ho.out)[at] = (f16)v;
    else ((bf16*)ho.out)[at] = (bf16)v;
}

// Token by token: a workgroup per (sequence, head), and per 64 columns of S where nothing stands behind the recurrence; 4 waves
// to 64 columns, a lane keeps one column's NR rows of its wave's share in registers.  Both read-outs come from the state
// before the token, a = S^T k and c = S^T q: u = beta (v - g a),  o = g c + u (k . q),  S <- g S + k u^T; the waves'
// shares of a and c meet in LDS.
#define SCAN_WAVES 4
#define SCAN_COLS 2              // at most this many blocks of 64 columns a workgroup

template <int NR, int CB>
__global__ __launch_bounds__(64 * SCAN_WAVES * CB) void delta_scan_kernel(const float* __restrict__ qkv, const float* __restrict__ gates,
                                                                          const float* __restrict__ kq, float* __restrict__ state,
                                                                          Steps st, HeadOut ho, int H, int G, int d, int dv) {
    constexpr int DP = NR * SCAN_WAVES;                  // rows of S, padded
    __shared__ __attribute__((aligned(16))) float sk[3][DP], sq[3][DP];
    __shared__ float part[2][CB][SCAN_WAVES][2][64], sq_sum[2][CB];
    const int seq = blockIdx.x, h = blockIdx.y, e = h / (H / G), tid = threadIdx.x, lane = tid & 63;
    const int wave = (tid >> 6) % SCAN_WAVES, cb = (tid >> 6) / SCAN_WAVES;
    const int col = (blockIdx.z * CB + cb) * 64 + lane, C = 2 * G * d + H * dv, r0 = wave * NR;
    const int q0 = st.seq_qstart ? st.seq_qstart[seq] : seq, n = st.seq_qlen ? st.seq_qlen[seq] : 1;
    if (n <= 0) return;
    const bool live = col < dv;
    float* S = state + (((int64_t)st.seq_slot[seq] * H + h) * d) * dv + col;
    float s[NR];
#pragma unroll
    for (int r = 0; r < NR; ++r) s[r] = (live && r0 + r < d) ? S[(int64_t)(r0 + r) * dv] : 0.f;
    auto stage = [&](int t) {
        const float* row = qkv + (int64_t)(q0 + t) * C;
        for (int i = tid; i < DP; i += 64 * SCAN_WAVES * CB) {
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
        part[t & 1][cb][wave][0][lane] = a;
        part[t & 1][cb][wave][1][lane] = c;
        if (t + 1 < n) stage(t + 1);
        __syncthreads();
        a = c = 0.f;
#pragma unroll
        for (int w = 0; w < SCAN_WAVES; ++w) { a += part[t & 1][cb][w][0][lane]; c += part[t & 1][cb][w][1][lane]; }
        const float u = beta * (v - g * a), o = g * c + u * dot;
        float ss = 0.f;
        if (ho.w) {
            if (wave == 0) ss = wave_sum(live ? o * o : 0.f);
            if (CB > 1) {
                if (wave == 0 && lane == 0) sq_sum[t & 1][cb] = ss;
                __syncthreads();
                ss = 0.f;
#pragma unroll
                for (int b = 0; b < CB; ++b) ss += sq_sum[t & 1][b];
            }
        }
        if (wave == 0 && live) store_head(ho, tok, H * dv, h, dv, col, o, ss);
#pragma unroll
        for (int r = 0; r < NR; ++r) s[r] = g * s[r] + k[r] * u;
    }
    if (live) {
#pragma unroll
        for (int r = 0; r < NR; ++r) if (r0 + r < d) S[(int64_t)(r0 + r) * dv] = s[r];
    }
}

// half 0: rows float32, aux [T, G]; half 1: rows bfloat16, aux [T, G, 2] (see delta_prep_kernel).  single: every
// sequence brings one token, and the history is brought up to date on the way (else the caller does that afterwards).
extern "C" int li_delta_prep(const float* proj, int stride, int col0, int b_col, int a_col, const float* conv_w, int taps,
                             float* hist, const int* pos, const int* tok_slot, const float* A_log, const float* dt_bias,
                             void* rows, float* gates, float* aux, int half, int single, int n, int H, int G, int d, int dv, hipStream_t stream) {
    if (n <= 0) return LI_OK;
    if (H <= 0 || G <= 0 || H % G || d <= 0 || dv <= 0 || taps < 1 || taps > CONV_MAX_TAPS || !hist) return LI_BAD_ARG;
    if (d > 64 * DELTA_MAXV) return LI_UNSUPPORTED;
    const int channels = 2 * G * d + H * dv;
    if (col0 < 0 || col0 + channels > stride || b_col < 0 || b_col + H > stride || a_col < 0 || a_col + H > stride) return LI_BAD_ARG;
    const DeltaPrep p{proj, stride, col0, b_col, a_col, conv_w, hist, pos, tok_slot, A_log, dt_bias, rows, gates, aux, n, taps, H, G, d, dv,
                      !single && n >= 256 && taps == 4 ? 8 : 1, single};
    const int units = G + (H * dv + 63) / 64 + 1;
    dim3 grid((n + p.tile - 1) / p.tile, (units + 3) / 4);
#define GO1(TAPS, HALF) do { if (d <= 64) delta_prep_kernel<TAPS, HALF, 1><<<grid, 256, 0, stream>>>(p); \
        else if (d <= 128) delta_prep_kernel<TAPS, HALF, 2><<<grid, 256, 0, stream>>>(p); else delta_prep_kernel<TAPS, HALF, 4><<<grid, 256, 0, stream>>>(p); } while (0)
#define GO(TAPS) do { if (half) GO1(TAPS, true); else GO1(TAPS, false); } while (0)
    if (taps == 4) GO(4); else GO(0);
#undef GO
#undef GO1
    LI_CHECK_LAUNCH();
    return LI_OK;
}

// norm_w null: out float32 [T, H dv] is o as it is.
extern "C" int li_delta_scan(const float* qkv, const float* gates, const float* kq, float* state, const int* seq_slot,
                             const int* seq_qstart, const int* seq_qlen, const float* norm_w, int w_shared, const float* gate,
                             int64_t gate_stride, float eps, void* out, int out_dt, int n_seqs, int H, int G, int d, int dv,
                             hipStream_t stream) {
    if (n_seqs <= 0) return LI_OK;
    if (H <= 0 || G <= 0 || H % G || d <= 0 || dv <= 0 || (norm_w && !gate) || (!norm_w && out_dt != DT_F32)) return LI_BAD_ARG;
    if (d > 64 * DELTA_MAXV || (norm_w && dv > 64 * SCAN_COLS)) return LI_UNSUPPORTED;
    Steps st{nullptr, nullptr, seq_slot, seq_qstart, seq_qlen};
    const HeadOut ho{norm_w, w_shared, gate, gate_stride, eps, out, out_dt};
    const int blocks = (dv + 63) / 64, cb = norm_w ? blocks : 1;
#define GO1(NR, CB) delta_scan_kernel<NR, CB><<<dim3(n_seqs, H, (blocks + CB - 1) / CB), 64 * SCAN_WAVES * CB, 0, stream>>>(qkv, gates, kq, \
                                                                                                    state, st, ho, H, G, d, dv)
#define GO(NR) do { if (cb == 1) GO1(NR, 1); else GO1(NR, 2); } while (0)
    if (d <= 16) GO(4); else if (d <= 32) GO(8); else if (d <= 64) GO(16); else if (d <= 128) GO(32); else GO(64);
#undef GO
#undef GO1
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
// r, k, v float32, head h's d elements at columns h d of rows `stride` apart; raw [T, H d] float32 (its bias included), u [H, d].
// A workgroup per (sequence, head), and per 64 columns of S where nothing stands behind the recurrence (HeadOut); 4 waves to
// 64 columns, a lane keeps its column's NR rows of its wave's share in registers, the waves' shares of o meet in LDS.
// ---------------------------------------------------------------------------
template <int NR, int CB>
__global__ __launch_bounds__(64 * SCAN_WAVES * CB) void wkv_scan_kernel(const float* __restrict__ r_, const float* __restrict__ k_,
                                                                        const float* __restrict__ v_, int stride,
                                                                        const float* __restrict__ raw, const float* __restrict__ bonus,
                                                                        float* __restrict__ state, Steps st, HeadOut ho, int H, int d) {
    constexpr int DP = NR * SCAN_WAVES;
    __shared__ __attribute__((aligned(16))) float sr[3][DP], sk[3][DP], sw[3][DP];
    __shared__ float part[2][CB][SCAN_WAVES][64], ruk[3][SCAN_WAVES * CB], sq_sum[2][CB];
    const int seq = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63;
    const int wave = (tid >> 6) % SCAN_WAVES, cb = (tid >> 6) / SCAN_WAVES, r0 = wave * NR;
    const int col = (blockIdx.z * CB + cb) * 64 + lane;
    const int q0 = st.seq_qstart ? st.seq_qstart[seq] : seq, n = st.seq_qlen ? st.seq_qlen[seq] : 1;
    if (n <= 0) return;
    const bool live = col < d;
    float* S = state + (((int64_t)st.seq_slot[seq] * H + h) * d) * d + col;
    float s[NR];
#pragma unroll
    for (int r = 0; r < NR; ++r) s[r] = (live && r0 + r < d) ? S[(int64_t)(r0 + r) * d] : 0.f;
    static_assert(DP <= 64 * SCAN_WAVES, "a thread a key channel");
    const float ub = tid < d ? bonus[h * d + tid] : 0.f;
    auto stage = [&](int t) {
        const int64_t at = (int64_t)(q0 + t) * stride + h * d;
        float rr = 0.f, kk = 0.f, w = 0.f;
        if (tid < d) {
            rr = r_[at + tid];
            kk = k_[at + tid];
            w = expf(-expf(raw[(int64_t)(q0 + t) * H * d + h * d + tid]));
        }
        if (tid < DP) { sr[t % 3][tid] = rr; sk[t % 3][tid] = kk; sw[t % 3][tid] = w; }
        const float b = wave_sum(rr * ub * kk);
        if (lane == 0) ruk[t % 3][tid >> 6] = b;
    };
    stage(0);
    __syncthreads();
    for (int t = 0; t < n; ++t) {
        const int64_t tok = q0 + t;
        const float v = live ? v_[tok * stride + h * d + col] : 0.f;
        const float *k = sk[t % 3] + r0, *rr = sr[t % 3] + r0, *w = sw[t % 3] + r0;
        float a = 0.f;
#pragma unroll
        for (int r = 0; r < NR; ++r) {
            a += s[r] * rr[r];
            s[r] = w[r] * s[r] + k[r] * v;
        }
        part[t & 1][cb][wave][lane] = a;
        if (t + 1 < n) stage(t + 1);
        __syncthreads();
        float o = 0.f, ss = 0.f;
        if (wave == 0) {
            float b = 0.f;
#pragma unroll
            for (int i = 0; i < SCAN_WAVES; ++i) o += part[t & 1][cb][i][lane];
#pragma unroll
            for (int i = 0; i < SCAN_WAVES * CB; ++i) b += ruk[t % 3][i];
            o += b * v;
            if (ho.w) ss = wave_sum(live ? o * o : 0.f);
        }
        if (CB > 1 && ho.w) {
            if (wave == 0 && lane == 0) sq_sum[t & 1][cb] = ss;
            __syncthreads();
            ss = 0.f;
#pragma unroll
            for (int i = 0; i < CB; ++i) ss += sq_sum[t & 1][i];
        }
        if (wave == 0 && live) store_head(ho, tok, H * d, h, d, col, o, ss);
    }
    if (live) {
#pragma unroll
        for (int r = 0; r < NR; ++r) if (r0 + r < d) S[(int64_t)(r0 + r) * d] = s[r];
    }
}

// norm_w null: out float32 [T, H d] is o as it is.
extern "C" int li_wkv_scan(const float* r, const float* k, const float* v, int stride, const float* raw, const float* bonus,
                           float* state, const int* seq_slot, const int* seq_qstart, const int* seq_qlen, const float* norm_w,
                           int w_shared, const float* gate, int64_t gate_stride, float eps, void* out, int out_dt, int n_seqs, int H,
                           int d, hipStream_t stream) {
    if (n_seqs <= 0) return LI_OK;
    if (H <= 0 || d <= 0 || stride < H * d || (norm_w && !gate) || (!norm_w && out_dt != DT_F32)) return LI_BAD_ARG;
    if (d > 256 || (norm_w && d > 64 * SCAN_COLS)) return LI_UNSUPPORTED;
    Steps st{nullptr, nullptr, seq_slot, seq_qstart, seq_qlen};
    const HeadOut ho{norm_w, w_shared, gate, gate_stride, eps, out, out_dt};
    const int blocks = (d + 63) / 64, cb = norm_w ? blocks : 1;
#define GO(NR, CB) wkv_scan_kernel<NR, CB><<<dim3(n_seqs, H, (blocks + CB - 1) / CB), 64 * SCAN_WAVES * CB, 0, stream>>>( \
        r, k, v, stride, raw, bonus, state, st, ho, H, d)
    if (d <= 16) GO(4, 1); else if (d <= 32) GO(8, 1); else if (d <= 64) GO(16, 1);
    else if (d <= 128 && cb == 2) GO(32, 2); else if (d <= 128) GO(32, 1); else GO(64, 1);
#undef GO
    LI_CHECK_LAUNCH();
    return LI_OK;
}
