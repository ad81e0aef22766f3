// The recurrences of recurrent.hip for the prompts of a 16-bit model, 32 tokens (a chunk) at a time on the matrix cores:
// the gated delta rule and the time mixing with a decay for every key channel.  Two kernels each.  The first, all
// chunks of the step at once, makes what depends on a chunk's own tokens only and leaves it in the order in which the
// second feeds it to the matrix cores; the second, a workgroup per (sequence, head, 16 columns of the state), walks the
// chunks in order with the state in registers, 32 of its rows a wave.
//
// The state, decays, gates and unit norms are float32.  A float32 operand of a product enters the matrix cores as the
// sum of NP bfloat16 numbers, its rounding and the roundings of what is left (three hold all 24 bits of it); the delta
// rule's q, k and v and the other's v come in bfloat16, which is exact.  Every product accumulates in float32.
//
// Accumulators of the 16x16x32 instruction: lane l holds column l % 16 and rows 4 (l / 16) + r, r < 4.  Operand A: row
// l % 16, inner indices 8 (l / 16) + e, e < 8; operand B the same with columns.  Where an operand comes out of two
// accumulators of 16 rows, its inner index e of lane l is the row rows(l, e) = 4 (l / 16) + e % 4 + 16 (e / 4) of the 32,
// and the other operand is laid out to match.
#include "common.h"

#define CH 32                   // tokens of a chunk
#define NP 3                    // bfloat16 numbers that a float32 operand becomes
#define LOG_DECAY_MIN -88.f     // (its exponential is 0 next to anything)

__device__ __forceinline__ f32x4 mfma16(bf16x8 a, bf16x8 b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0); }
__device__ __forceinline__ int rows32(int lane, int e) { return 4 * (lane >> 4) + (e & 3) + 16 * (e >> 2); }

// v[0..7] as NP bfloat16 vectors whose sum it is
__device__ __forceinline__ void split(const float (&v)[8], bf16x8 (&p)[NP]) {
    float left[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) left[e] = v[e];
#pragma unroll
    for (int i = 0; i < NP; ++i)
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const bf16 h = (bf16)left[e];
            p[i][e] = h;
            left[e] -= (float)h;
        }
}
// c += a b for split operands (the terms that reach the result's last bits), or one split and one exact
__device__ __forceinline__ f32x4 mul_ss(const bf16x8 (&a)[NP], const bf16x8 (&b)[NP], f32x4 c) {
#pragma unroll
    for (int i = NP - 1; i >= 0; --i)
#pragma unroll
        for (int j = NP - 1 - i; j >= 0; --j) c = mfma16(a[i], b[j], c);
    return c;
}
__device__ __forceinline__ f32x4 mul_es(bf16x8 a, const bf16x8 (&b)[NP], f32x4 c) {
#pragma unroll
    for (int j = NP - 1; j >= 0; --j) c = mfma16(a, b[j], c);
    return c;
}
__device__ __forceinline__ f32x4 mul_se(const bf16x8 (&a)[NP], bf16x8 b, f32x4 c) {
#pragma unroll
    for (int i = NP - 1; i >= 0; --i) c = mfma16(a[i], b, c);
    return c;
}
__device__ __forceinline__ void join(const f32x4& lo, const f32x4& hi, float (&v)[8]) {
#pragma unroll
    for (int r = 0; r < 4; ++r) { v[r] = lo[r]; v[4 + r] = hi[r]; }
}

// sixteen bytes at a base that is the same for the whole wave, and a lane's offset
template <class V, class T>
__device__ __forceinline__ V load_at(const T* base, unsigned off) { return *(const V*)(base + off); }

struct Chunks {
    const int* chunk_seq;       // [chunks] the sequence of a chunk
    const int* chunk_t0;        // [chunks] its first token among the sequence's tokens of this step
    const int* seq_chunk0;      // [sequences] its first chunk
    const int* seq_slot;
    const int* seq_qstart;
    const int* seq_qlen;
};

// a 32 x 32 matrix m (rows `ld` floats apart, in LDS) as operand A, two tiles of 16 rows, split: out [NP][2][64][8]
__device__ __forceinline__ void pack32(const float* m, int ld, bf16* out, int first, int step) {
    for (int u = first; u < 2 * 64; u += step) {
        const int tile = u >> 6, lane = u & 63;
        float v[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] = m[(16 * tile + (lane & 15)) * ld + rows32(lane, e)];
        bf16x8 p[NP];
        split(v, p);
#pragma unroll
        for (int i = 0; i < NP; ++i) *(bf16x8*)(out + ((int64_t)(i * 2 + tile) * 64 + lane) * 8) = p[i];
    }
}

// A chunk's values as operands, a block of 16 columns each: column 16 b + l % 16, tokens rows32(l, e); out [blocks][64][8].
// `v` points at the head's first element of the chunk's first token, rows C apart; a token or column that is not there: 0.
__device__ __forceinline__ void pack_values(const bf16* v, int64_t C, int n, int dv, bf16* out, int first, int step) {
    for (int u = first; u < (dv + 15) / 16 * 64; u += step) {
        const int lane = u & 63, col = 16 * (u >> 6) + (lane & 15);
        bf16x8 p;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const int t = rows32(lane, e);
            p[e] = t < n && col < dv ? v[t * C + col] : (bf16)0.f;
        }
        *(bf16x8*)(out + (int64_t)u * 8) = p;
    }
}

// ---------------------------------------------------------------------------
// The gated delta rule.  In a chunk with the state S before it, b_i the sum of log g up to token i and U the written
// values,
//   (I + L) U = diag(beta) (V - diag(e^b) K S),   L_ij = beta_i e^(b_i - b_j) k_i . k_j  for j < i
//   O = diag(e^b) Q S + A U,   A_ij = e^(b_i - b_j) q_i . k_j  for j <= i
//   S <- e^(b_n) S + K^T diag(e^(b_n - b)) U
// delta_chunk_kernel, a wave per (chunk, head): W = (I + L)^-1 diag(beta) by forward substitution, a column a lane; W and A
// to `mats` [chunk, head, W | A | V] (V: pack_values); the coefficients of the rows to `coef` [chunk, head, 4, 32] (e^b_i / |k_i|, e^b_i
// d^(-1/2) / |q_i|, e^(b_n - b_i) / |k_i|, and e^(b_n)); and, once a key head, the chunk's keys and queries as operands to
// `packs` [chunk, key head, K | Q | K^T], each [blocks of 32 key dimensions][2][64][8].
// rows: bfloat16 [T, 2 G d + H dv], q | k | v behind convolution and silu; norms [T, G, 2]: d^(-1/2) / |q|, 1 / |k|;
// gates [T, H, 2]: log g, beta.
// ---------------------------------------------------------------------------
#define LDM 36                  // floats from row to row of a 32 x 32 matrix in LDS
#define MAT_ELEMS (NP * 2 * 64 * 8)
// elements of `count` 32 x 32 operands and the values behind them
__host__ __device__ __forceinline__ int mat_elems(int count, int dv) { return count * MAT_ELEMS + (dv + 15) / 16 * 64 * 8; }

__global__ __launch_bounds__(64) void delta_chunk_kernel(const bf16* __restrict__ rows, const float* __restrict__ norms,
                                                         const float* __restrict__ gates, Chunks cs, bf16* __restrict__ mats,
                                                         float* __restrict__ coef, bf16* __restrict__ packs, int H, int G, int d,
                                                         int dv) {
    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
    const int DB = (d + 31) / 32, DP = 32 * DB, LK = DP + 8;
    bf16* sQ = (bf16*)smem;                        // [CH][LK]
    bf16* sK = sQ + CH * LK;
    float* sL = (float*)(sK + CH * LK);            // [CH][LDM]
    float* sA = sL + CH * LDM;
    float* sb = sA + CH * LDM;                     // [CH] b, then beta, 1 / |k|, d^(-1/2) / |q|
    float *sbeta = sb + CH, *srk = sbeta + CH, *srq = srk + CH;
    const int lane = threadIdx.x, col = lane & 31, half = lane >> 5;
    const int chunk = blockIdx.x, h = blockIdx.y, e = h / (H / G), seq = cs.chunk_seq[chunk], c0 = cs.chunk_t0[chunk];
    const int n = min(CH, cs.seq_qlen[seq] - c0), C = 2 * G * d + H * dv;
    if (n <= 0) return;
    const int64_t t0 = cs.seq_qstart[seq] + c0;
    if ((d & 7) == 0 && (C & 7) == 0) {
        const int per = DP / 8;
        for (int u = lane; u < CH * per; u += 64) {
            const int t = u / per, i = 8 * (u - t * per);
            bf16x8 q = {}, k = {};
            if (t < n && i < d) {
                const bf16* row = rows + (t0 + t) * C + e * d + i;
                q = *(const bf16x8*)row;
                k = *(const bf16x8*)(row + G * d);
            }
            *(bf16x8*)(sQ + t * LK + i) = q;
            *(bf16x8*)(sK + t * LK + i) = k;
        }
    } else {
        for (int u = lane; u < CH * DP; u += 64) {
            const int t = u / DP, i = u - t * DP;
            const bool ok = t < n && i < d;
            const bf16* row = rows + (t0 + (ok ? t : 0)) * C + e * d + (ok ? i : 0);
            sQ[t * LK + i] = ok ? row[0] : (bf16)0.f;
            sK[t * LK + i] = ok ? row[G * d] : (bf16)0.f;
        }
    }
    // token `col` of the chunk, in both halves of the wave: its gates, and the sum of the logarithms up to it
    const bool ok = col < n;
    float b = ok ? gates[((t0 + col) * H + h) * 2] : 0.f;
    const float beta = ok ? gates[((t0 + col) * H + h) * 2 + 1] : 0.f;
    const float rq = ok ? norms[((t0 + col) * G + e) * 2] : 0.f, rk = ok ? norms[((t0 + col) * G + e) * 2 + 1] : 0.f;
#pragma unroll
    for (int o = 1; o < CH; o <<= 1) {
        const float up = __shfl_up(b, o, 32);
        if (col >= o) b += up;
    }
    const float bn = __shfl(b, CH - 1, 32);        // (tokens that are not there leave the sum as it is)
    if (half == 0) {
        sb[col] = b; sbeta[col] = beta; srk[col] = rk; srq[col] = rq;
        float* c = coef + ((int64_t)chunk * H + h) * 4 * CH;
        c[col] = expf(b) * rk;
        c[CH + col] = expf(b) * rq;
        c[2 * CH + col] = expf(bn - b) * rk;
        c[3 * CH + col] = expf(bn);
    }
    __syncthreads();
    f32x16 kk, qk;
#pragma unroll
    for (int r = 0; r < 16; ++r) kk[r] = qk[r] = 0.f;
    for (int s = 0; s < 2 * DB; ++s) {
        const bf16x8 kf = *(const bf16x8*)(sK + col * LK + 16 * s + 8 * half), qf = *(const bf16x8*)(sQ + col * LK + 16 * s + 8 * half);
        kk = mfma32(kf, kf, kk);
        qk = mfma32(qf, kf, qk);
    }
#pragma unroll
    for (int r = 0; r < 16; ++r) {
        const int i = 8 * (r >> 2) + 4 * half + (r & 3);          // row; this lane's column is col
        const float w = i >= col ? expf(sb[i] - b) * rk : 0.f;
        sL[i * LDM + col] = i > col ? sbeta[i] * srk[i] * w * kk[r] : 0.f;
        sA[i * LDM + col] = srq[i] * w * qk[r];
    }
    __syncthreads();
    // column col of (I + L)^-1, by forward substitution
    float w[CH];
    int row_at = 0;
#pragma unroll
    for (int i = 0; i < CH; ++i) {
        float s[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int j4 = 0; j4 < (i + 3) / 4; ++j4) {
            const f32x4 l = *(const f32x4*)(sL + row_at + i * LDM + 4 * j4);
#pragma unroll
            for (int u = 0; u < 4; ++u) if (4 * j4 + u < i) s[u] += l[u] * w[4 * j4 + u];
        }
        w[i] = (i == col ? 1.f : 0.f) - ((s[0] + s[1]) + (s[2] + s[3]));
        // (the compiler would fetch all of L at once: the next row's address is known once the row before this one is done)
        asm volatile("" : "+v"(row_at) : "v"(w[i > 0 ? i - 1 : 0]));
    }
    __syncthreads();                               // every lane has read L: W takes its place
    if (half == 0) {
#pragma unroll
        for (int i = 0; i < CH; ++i) sL[i * LDM + col] = w[i] * beta;
    }
    __syncthreads();
    bf16* m = mats + ((int64_t)chunk * H + h) * mat_elems(2, dv);
    pack32(sL, LDM, m, lane, 64);
    pack32(sA, LDM, m + MAT_ELEMS, lane, 64);
    pack_values(rows + t0 * C + 2 * G * d + h * dv, C, n, dv, m + 2 * MAT_ELEMS, lane, 64);
    if (h % (H / G) == 0) {
        const int64_t per = (int64_t)DB * 2 * 64 * 8;
        bf16* pk = packs + ((int64_t)chunk * G + e) * 3 * per;
        for (int u = 0; u < 2 * DB; ++u) {
            const int blk = u >> 1, tile = u & 1;
            bf16x8 kf, qf, tf;
#pragma unroll
            for (int x = 0; x < 8; ++x) {
                const int row = rows32(lane, x);
                kf[x] = sK[(16 * tile + (lane & 15)) * LK + 32 * blk + row];
                qf[x] = sQ[(16 * tile + (lane & 15)) * LK + 32 * blk + row];
                tf[x] = sK[row * LK + 32 * blk + 16 * tile + (lane & 15)];
            }
            bf16* at = pk + ((int64_t)u * 64 + lane) * 8;
            *(bf16x8*)at = kf;
            *(bf16x8*)(at + per) = qf;
            *(bf16x8*)(at + 2 * per) = tf;
        }
    }
}

// The walk.  Workgroup: (sequence, head, 16 columns), DB waves of 32 rows of S each.  A wave's shares of K S and Q S meet in LDS
// (one barrier a chunk, two buffers); every wave then has the whole of K S and computes U by itself.
// NO: the tiles of 16 rows of the output that a wave adds up and writes, one of the two (waves 0 and 1), or both where there
// is one wave.
template <int NO>
struct DeltaFrags {
    bf16x8 k[2], q[2], kt[2], w[NP][2], a[NP][NO];
    bf16x8 v;
    f32x4 ck[2], cq[NO], ce[2];
    float gn;
};

template <int NO>
__global__ __launch_bounds__(NO == 2 ? 64 : 512) void delta_walk_kernel(const bf16* __restrict__ mats, const float* __restrict__ coef, const bf16* __restrict__ packs,
                                                         float* __restrict__ state, Chunks cs, float* __restrict__ y, int H, int G,
                                                         int d, int dv) {
    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
    f32x4* part = (f32x4*)smem;                    // [2][waves][4][64]
    const int seq = blockIdx.x, h = blockIdx.y, e = h / (H / G), lane = threadIdx.x & 63;
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), nw = blockDim.x >> 6;
    const int col = 16 * blockIdx.z + (lane & 15), C = 2 * G * d + H * dv, DB = nw, rq = 4 * (lane >> 4);
    const int n = cs.seq_qlen[seq], n_chunks = (n + CH - 1) / CH;
    if (n <= 0) return;
    const int64_t q0 = cs.seq_qstart[seq], first = cs.seq_chunk0[seq], per = (int64_t)DB * 2 * 64 * 8;
    const bool live = col < dv;
    const int cc = live ? col : dv - 1;
    float* S = state + (((int64_t)cs.seq_slot[seq] * H + h) * d) * dv + cc;
    f32x4 s[2];
#pragma unroll
    for (int m = 0; m < 2; ++m)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int row = 32 * wave + 16 * m + rq + r;
            s[m][r] = row < d ? S[(int64_t)row * dv] : 0.f;
        }
    const int o_tile = NO == 2 ? 0 : min(wave, 1);       // the first tile of the output
    const bool writes = wave < 2;
    const unsigned at = lane * 8;
    unsigned none = 0;                             // in a vector register: a scalar load of gn would hold up every wait for LDS
    asm volatile("" : "+v"(none));
    auto fetch = [&](int c, DeltaFrags<NO>& f) {
        const bf16* pk = packs + ((first + c) * G + e) * 3 * per + (int64_t)(2 * wave) * 512;
        const bf16* mt = mats + ((first + c) * H + h) * mat_elems(2, dv);
        const float* cf = coef + ((first + c) * H + h) * 4 * CH;
#pragma unroll
        for (int m = 0; m < 2; ++m) {
            f.k[m] = load_at<bf16x8>(pk + m * 512, at);
            f.q[m] = load_at<bf16x8>(pk + per + m * 512, at);
            f.kt[m] = load_at<bf16x8>(pk + 2 * per + m * 512, at);
            f.ck[m] = load_at<f32x4>(cf + 16 * m, rq);
            f.ce[m] = load_at<f32x4>(cf + 2 * CH + 16 * m, rq);
#pragma unroll
            for (int i = 0; i < NP; ++i) f.w[i][m] = load_at<bf16x8>(mt + (i * 2 + m) * 512, at);
        }
#pragma unroll
        for (int m = 0; m < NO; ++m) {
            f.cq[m] = load_at<f32x4>(cf + CH + 16 * (o_tile + m), rq);
#pragma unroll
            for (int i = 0; i < NP; ++i) f.a[i][m] = load_at<bf16x8>(mt + MAT_ELEMS + (i * 2 + o_tile + m) * 512, at);
        }
        f.v = load_at<bf16x8>(mt + 2 * MAT_ELEMS + blockIdx.z * 512, at);
        f.gn = load_at<float>(cf + 3 * CH, none);
    };
    f32x4 out[NO];                                 // the last chunk's output: written a chunk later, so that no load waits behind it
    auto put = [&](int c) {
        if (!writes || !live || c < 0) return;
#pragma unroll
        for (int m = 0; m < NO; ++m)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int t = c * CH + 16 * (o_tile + m) + rq + r;
                if (t < n) y[(q0 + t) * H * dv + h * dv + col] = out[m][r];
            }
    };
    auto body = [&](int c, const DeltaFrags<NO>& f) {
        const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
        float v8[8];
        bf16x8 sp[NP];
        join(s[0], s[1], v8);
        split(v8, sp);
        f32x4 pk[2], pq[2];
#pragma unroll
        for (int m = 0; m < 2; ++m) { pk[m] = mul_es(f.k[m], sp, zero); pq[m] = mul_es(f.q[m], sp, zero); }
        put(c - 1);
        if (nw > 1) {
            f32x4* buf = part + (c & 1) * nw * 256;
#pragma unroll
            for (int m = 0; m < 2; ++m) {
                buf[(wave * 4 + m) * 64 + lane] = pk[m];
                buf[(wave * 4 + 2 + m) * 64 + lane] = pq[m];
            }
            __syncthreads();
#pragma unroll
            for (int m = 0; m < 2; ++m) { pk[m] = zero; pq[m] = zero; }
            for (int w = 0; w < nw; ++w) {
                pk[0] += buf[(w * 4) * 64 + lane];
                pk[1] += buf[(w * 4 + 1) * 64 + lane];
                pq[0] += buf[(w * 4 + 2 + o_tile) * 64 + lane];          // (more than one wave: one tile each)
            }
        }
        // R = V - diag(e^b / |k|) K S,  U = W R
        float r8[8];
#pragma unroll
        for (int m = 0; m < 2; ++m)
#pragma unroll
            for (int r = 0; r < 4; ++r) r8[4 * m + r] = (float)f.v[4 * m + r] - f.ck[m][r] * pk[m][r];
        bf16x8 rp[NP], up[NP];
        split(r8, rp);
        f32x4 u[2];
#pragma unroll
        for (int m = 0; m < 2; ++m) {
            const bf16x8 w[NP] = {f.w[0][m], f.w[1][m], f.w[2][m]};
            u[m] = mul_ss(w, rp, zero);
        }
        // S <- e^(b_n) S + K^T diag(e^(b_n - b) / |k|) U
#pragma unroll
        for (int m = 0; m < 2; ++m)
#pragma unroll
            for (int r = 0; r < 4; ++r) v8[4 * m + r] = f.ce[m][r] * u[m][r];
        split(v8, up);
#pragma unroll
        for (int m = 0; m < 2; ++m) {
#pragma unroll
            for (int r = 0; r < 4; ++r) s[m][r] *= f.gn;
            s[m] = mul_es(f.kt[m], up, s[m]);
        }
        // O = diag(e^b d^(-1/2) / |q|) Q S + A U
        if (writes) {
            join(u[0], u[1], v8);
            split(v8, up);
#pragma unroll
            for (int m = 0; m < NO; ++m) {
                f32x4 o;
#pragma unroll
                for (int r = 0; r < 4; ++r) o[r] = f.cq[m][r] * pq[m][r];
                const bf16x8 a[NP] = {f.a[0][m], f.a[1][m], f.a[2][m]};
                out[m] = mul_ss(a, up, o);
            }
        }
    };
#pragma unroll
    for (int m = 0; m < 2; ++m) asm volatile("" : "+v"(s[m]));         // the state has come: no wait for it in the loop
    DeltaFrags<NO> fa, fb;                         // the chunk at work and the next one, in turn
    fetch(0, fa);
    // (every turn fetches, the last ones the last chunk again: a branch around the loads would make the wait before their use
    // one for all loads of both ways, the next chunk's among them)
    for (int c = 0; c < n_chunks; c += 2) {
        fetch(min(c + 1, n_chunks - 1), fb);
        __builtin_amdgcn_sched_barrier(0);         // the loads first
        body(c, fa);
        if (c + 1 >= n_chunks) break;
        fetch(min(c + 2, n_chunks - 1), fa);
        __builtin_amdgcn_sched_barrier(0);
        body(c + 1, fb);
    }
    put(n_chunks - 1);
    if (live) {
#pragma unroll
        for (int m = 0; m < 2; ++m)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int row = 32 * wave + 16 * m + rq + r;
                if (row < d) S[(int64_t)row * dv] = s[m][r];
            }
    }
}

// Elements of scratch memory that a (chunk, head) and a (chunk, key head) take, in that order: mats and packs.
extern "C" int li_delta_chunk_elems(int d, int dv, int which) { return which == 0 ? mat_elems(2, dv) : 3 * ((d + 31) / 32) * 2 * 64 * 8; }

// mats bfloat16 [chunks, H, li_delta_chunk_elems(d, dv, 0)], packs bfloat16 [chunks, G, li_delta_chunk_elems(d, dv, 1)], coef float32
// [chunks, H, 4, 32]: scratch memory.
extern "C" int li_delta_chunks(const void* rows, const float* norms, const float* gates, float* state, const int* seq_slot,
                               const int* seq_qstart, const int* seq_qlen, const int* chunk_seq, const int* chunk_t0,
                               const int* seq_chunk0, int n_chunks, void* mats, float* coef, void* packs, float* y, int n_seqs,
                               int H, int G, int d, int dv, hipStream_t stream) {
    if (n_seqs <= 0 || n_chunks <= 0) return LI_OK;
    if (H <= 0 || G <= 0 || H % G || d <= 0 || dv <= 0 || !seq_qstart || !seq_qlen || !chunk_seq || !chunk_t0 || !seq_chunk0) return LI_BAD_ARG;
    if (d > 256) return LI_UNSUPPORTED;
    const Chunks cs{chunk_seq, chunk_t0, seq_chunk0, seq_slot, seq_qstart, seq_qlen};
    const int DB = (d + 31) / 32;
    const size_t lds1 = (size_t)2 * CH * (32 * DB + 8) * 2 + (size_t)(2 * CH * LDM + 4 * CH) * 4;
    if (lds1 > 60000) return LI_UNSUPPORTED;
    delta_chunk_kernel<<<dim3(n_chunks, H), 64, lds1, stream>>>((const bf16*)rows, norms, gates, cs, (bf16*)mats, coef, (bf16*)packs,
                                                                H, G, d, dv);
    LI_CHECK_LAUNCH();
    const size_t lds2 = DB > 1 ? (size_t)2 * DB * 256 * 16 : 0;
    if (lds2 > 48 * 1024 && hipFuncSetAttribute((const void*)delta_walk_kernel<1>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds2) != hipSuccess)
        return LI_HIP_ERROR;
    dim3 grid(n_seqs, H, (dv + 15) / 16), block(64 * DB);
#define GO(NO) delta_walk_kernel<NO><<<grid, block, lds2, stream>>>((const bf16*)mats, coef, (const bf16*)packs, state, \
                                                                    cs, y, H, G, d, dv)
    if (DB == 1) GO(2); else GO(1);
#undef GO
    LI_CHECK_LAUNCH();
    return LI_OK;
}

// ---------------------------------------------------------------------------
// Time mixing with a decay for every key channel.  In a chunk with the state S before it, b_t[c] the sum of log w_s[c]
// over the chunk's tokens s <= t,
//   o_t = (r_t e^(b_(t-1)))^T S + sum over s <= t of A_ts v_s,  A_ts = sum over c of r_t k_s e^(b_(t-1) - b_s)  (s < t),
//   A_tt = sum over c of r_t u k_t;     S <- diag(e^(b_n)) S + sum over s of (k_s e^(b_n - b_s)) v_s^T
// Every exponent is at most 0 (a logarithm is taken as no less than LOG_DECAY_MIN).  wkv_chunk_kernel, four waves per (chunk, head): A's two blocks of 16 tokens on the diagonal pair by
// pair, the block below them as a product of r e^(b_(t-1) - b_15) and k e^(b_15 - b_s) on the float32 matrix cores;
// `mats` [chunk, head, A | V]; `packs` [chunk, head, R | K^T] (r e^(b_(t-1)) and k e^(b_n - b_s) as operands, split, each [blocks
// of 32 channels][NP][2][64][8]); `coef` [chunk, head, 32 blocks]: e^(b_n).
// r, k float32, v bfloat16 [T, H d]; raw float32 [T, H d], log w = -exp(raw).
// ---------------------------------------------------------------------------
__global__ __launch_bounds__(256) void wkv_chunk_kernel(const float* __restrict__ r_, const float* __restrict__ k_,
                                                        const bf16* __restrict__ v_,
                                                        const float* __restrict__ raw, const float* __restrict__ bonus, Chunks cs,
                                                        bf16* __restrict__ mats, float* __restrict__ coef, bf16* __restrict__ packs,
                                                        int H, int d) {
    extern __shared__ __attribute__((aligned(16))) float wl[];
    const int DB = (d + 31) / 32, DP = 32 * DB, LD = DP + 4;
    float* sr = wl;                                // [CH][LD]
    float* sk = sr + CH * LD;
    float* sb = sk + CH * LD;                      // [CH + 1][LD]: row t + 1 is b_t, row 0 zeros
    float* sA = sb + (CH + 1) * LD;                // [CH][LDM]
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int chunk = blockIdx.x, h = blockIdx.y, seq = cs.chunk_seq[chunk], c0 = cs.chunk_t0[chunk];
    const int n = min(CH, cs.seq_qlen[seq] - c0), C = H * d;
    if (n <= 0) return;
    const int64_t at = (int64_t)(cs.seq_qstart[seq] + c0) * C + h * d;
    for (int u = tid; u < CH * DP; u += 256) {
        const int t = u / DP, c = u - t * DP;
        const bool ok = t < n && c < d;
        const int64_t i = at + (int64_t)(ok ? t : 0) * C + (ok ? c : 0);
        sr[t * LD + c] = ok ? r_[i] : 0.f;
        sk[t * LD + c] = ok ? k_[i] : 0.f;
        sb[(t + 1) * LD + c] = ok ? fmaxf(-expf(raw[i]), LOG_DECAY_MIN) : 0.f;
    }
    for (int c = tid; c < DP; c += 256) sb[c] = 0.f;
    for (int u = tid; u < CH * LDM; u += 256) sA[u] = 0.f;
    __syncthreads();
    for (int c = tid; c < DP; c += 256) {          // the sums over time, a channel a thread
        float s = 0.f;
#pragma unroll
        for (int t = 0; t < CH; ++t) { s += sb[(t + 1) * LD + c]; sb[(t + 1) * LD + c] = s; }
        coef[((int64_t)chunk * H + h) * DP + c] = expf(s);
    }
    __syncthreads();
    // the blocks on the diagonal: 16 pairs (t, s) at a time, four lanes a pair, each every fourth four channels.  Rows j and
    // 15 - j of a block have 15 pairs together, so eight rounds a block do; the diagonal itself is one round more.
    const int pr = lane & 15, cg = lane >> 4;
    for (int job = wave; job < 18; job += 4) {
        const int base = job & 1 ? 16 : 0, j = job >> 1;
        int t, s;
        if (j == 8) t = s = pr;
        else if (pr < 15 - j) { t = 15 - j; s = pr; }
        else { t = j; s = pr - (15 - j); }
        const bool valid = j == 8 || s < t;
        float acc = 0.f;
        const float *rt = sr + (base + t) * LD, *ks = sk + (base + s) * LD, *bt = sb + (base + t) * LD, *bs = sb + (base + s + 1) * LD;
        if (valid) {
            for (int c = 4 * cg; c < DP; c += 16) {
                const f32x4 rv = *(const f32x4*)(rt + c), kv = *(const f32x4*)(ks + c);
                if (j == 8) {
#pragma unroll
                    for (int i = 0; i < 4; ++i) acc += c + i < d ? rv[i] * kv[i] * bonus[h * d + c + i] : 0.f;
                } else {
                    const f32x4 b1 = *(const f32x4*)(bt + c), b2 = *(const f32x4*)(bs + c);
#pragma unroll
                    for (int i = 0; i < 4; ++i) acc += rv[i] * kv[i] * __expf(b1[i] - b2[i]);
                }
            }
        }
        acc += __shfl_xor(acc, 16, WAVE);
        acc += __shfl_xor(acc, 32, WAVE);
        if (cg == 0 && valid) sA[(base + t) * LDM + base + s] = acc;
    }
    if (wave == 3) {                               // tokens 16..31 against 0..15
        f32x4 acc = {0.f, 0.f, 0.f, 0.f};
        const float *rt = sr + (16 + pr) * LD, *bt = sb + (16 + pr) * LD, *ks = sk + pr * LD, *bs = sb + (pr + 1) * LD, *ref = sb + 16 * LD;
        for (int c = cg; c < DP; c += 4)
            acc = __builtin_amdgcn_mfma_f32_16x16x4f32(rt[c] * __expf(bt[c] - ref[c]), ks[c] * __expf(ref[c] - bs[c]), acc, 0, 0, 0);
#pragma unroll
        for (int r = 0; r < 4; ++r) sA[(16 + 4 * cg + r) * LDM + pr] = acc[r];
    }
    // the operands
    const int64_t per = (int64_t)DB * NP * 2 * 64 * 8;
    bf16* pk = packs + ((int64_t)chunk * H + h) * 2 * per;
    for (int u = wave; u < 4 * DB; u += 4) {
        const int kind = u & 1, tile = (u >> 1) & 1, blk = u >> 2;
        float v[8];
#pragma unroll
        for (int x = 0; x < 8; ++x) {
            const int in = rows32(lane, x);
            if (kind == 0) {
                const int t = 16 * tile + pr, c = 32 * blk + in;
                v[x] = sr[t * LD + c] * __expf(sb[t * LD + c]);
            } else {
                const int t = in, c = 32 * blk + 16 * tile + pr;
                v[x] = sk[t * LD + c] * __expf(sb[CH * LD + c] - sb[(t + 1) * LD + c]);
            }
        }
        bf16x8 p[NP];
        split(v, p);
#pragma unroll
        for (int i = 0; i < NP; ++i) *(bf16x8*)(pk + kind * per + (((int64_t)blk * NP + i) * 2 + tile) * 512 + lane * 8) = p[i];
    }
    __syncthreads();
    bf16* m = mats + ((int64_t)chunk * H + h) * mat_elems(1, d);
    pack32(sA, LDM, m, tid, 256);
    pack_values(v_ + at, C, n, d, m + MAT_ELEMS, tid, 256);
}

template <int NO>
struct WkvFrags {
    bf16x8 r[NP][2], kt[NP][2], a[NP][NO], v;
    f32x4 dec[2];
};

template <int NO>
__global__ __launch_bounds__(NO == 2 ? 64 : 512) void wkv_walk_kernel(const bf16* __restrict__ mats, const float* __restrict__ coef, const bf16* __restrict__ packs,
                                                       float* __restrict__ state, Chunks cs, float* __restrict__ y, int H, int d) {
    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
    f32x4* part = (f32x4*)smem;                    // [2][waves][2][64]
    const int seq = blockIdx.x, h = blockIdx.y, lane = threadIdx.x & 63;
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), nw = blockDim.x >> 6, DB = nw;
    const int col = 16 * blockIdx.z + (lane & 15), C = H * d, rq = 4 * (lane >> 4);
    const int n = cs.seq_qlen[seq], n_chunks = (n + CH - 1) / CH;
    if (n <= 0) return;
    const int64_t q0 = cs.seq_qstart[seq], first = cs.seq_chunk0[seq], per = (int64_t)DB * NP * 2 * 64 * 8;
    const bool live = col < d;
    const int cc = live ? col : d - 1;
    float* S = state + (((int64_t)cs.seq_slot[seq] * H + h) * d) * d + cc;
    f32x4 s[2];
#pragma unroll
    for (int m = 0; m < 2; ++m)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int row = 32 * wave + 16 * m + rq + r;
            s[m][r] = row < d ? S[(int64_t)row * d] : 0.f;
        }
    const int o_tile = NO == 2 ? 0 : min(wave, 1);       // the first tile of the output
    const bool writes = wave < 2;
    const unsigned at = lane * 8;
    auto fetch = [&](int c, WkvFrags<NO>& f) {
        const bf16* pk = packs + ((first + c) * H + h) * 2 * per + (int64_t)wave * NP * 2 * 512;
        const bf16* mt = mats + ((first + c) * H + h) * mat_elems(1, d);
        const float* cf = coef + ((first + c) * H + h) * 32 * DB + 32 * wave;
#pragma unroll
        for (int m = 0; m < 2; ++m) {
            f.dec[m] = load_at<f32x4>(cf + 16 * m, rq);
#pragma unroll
            for (int i = 0; i < NP; ++i) {
                f.r[i][m] = load_at<bf16x8>(pk + (i * 2 + m) * 512, at);
                f.kt[i][m] = load_at<bf16x8>(pk + per + (i * 2 + m) * 512, at);
            }
        }
#pragma unroll
        for (int m = 0; m < NO; ++m)
#pragma unroll
            for (int i = 0; i < NP; ++i) f.a[i][m] = load_at<bf16x8>(mt + (i * 2 + o_tile + m) * 512, at);
        f.v = load_at<bf16x8>(mt + MAT_ELEMS + blockIdx.z * 512, at);
    };
    f32x4 out[NO];                                 // the last chunk's output: written a chunk later, so that no load waits behind it
    auto put = [&](int c) {
        if (!writes || !live || c < 0) return;
#pragma unroll
        for (int m = 0; m < NO; ++m)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int t = c * CH + 16 * (o_tile + m) + rq + r;
                if (t < n) y[(q0 + t) * C + h * d + col] = out[m][r];
            }
    };
    auto body = [&](int c, const WkvFrags<NO>& f) {
        const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
        float v8[8];
        bf16x8 sp[NP];
        join(s[0], s[1], v8);
        split(v8, sp);
        f32x4 o[2];
#pragma unroll
        for (int m = 0; m < 2; ++m) {
            const bf16x8 r[NP] = {f.r[0][m], f.r[1][m], f.r[2][m]}, kt[NP] = {f.kt[0][m], f.kt[1][m], f.kt[2][m]};
            o[m] = mul_ss(r, sp, zero);
#pragma unroll
            for (int i = 0; i < 4; ++i) s[m][i] *= f.dec[m][i];
            s[m] = mul_se(kt, f.v, s[m]);
        }
        put(c - 1);
        if (nw > 1) {
            f32x4* buf = part + (c & 1) * nw * 128;
#pragma unroll
            for (int m = 0; m < 2; ++m) buf[(wave * 2 + m) * 64 + lane] = o[m];
            __syncthreads();
            o[0] = zero;                           // (more than one wave: one tile each)
            if (writes) for (int w = 0; w < nw; ++w) o[0] += buf[(w * 2 + o_tile) * 64 + lane];
        }
#pragma unroll
        for (int m = 0; m < NO; ++m) {
            if (!writes) continue;
            const bf16x8 a[NP] = {f.a[0][m], f.a[1][m], f.a[2][m]};
            out[m] = mul_se(a, f.v, o[m]);
        }
    };
#pragma unroll
    for (int m = 0; m < 2; ++m) asm volatile("" : "+v"(s[m]));         // the state has come: no wait for it in the loop
    WkvFrags<NO> fa, fb;                           // the chunk at work and the next one, in turn
    fetch(0, fa);
    // (every turn fetches, the last ones the last chunk again: a branch around the loads would make the wait before their use
    // one for all loads of both ways, the next chunk's among them)
    for (int c = 0; c < n_chunks; c += 2) {
        fetch(min(c + 1, n_chunks - 1), fb);
        __builtin_amdgcn_sched_barrier(0);         // the loads first
        body(c, fa);
        if (c + 1 >= n_chunks) break;
        fetch(min(c + 2, n_chunks - 1), fa);
        __builtin_amdgcn_sched_barrier(0);
        body(c + 1, fb);
    }
    put(n_chunks - 1);
    if (live) {
#pragma unroll
        for (int m = 0; m < 2; ++m)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int row = 32 * wave + 16 * m + rq + r;
                if (row < d) S[(int64_t)row * d] = s[m][r];
            }
    }
}

// Elements of scratch memory of a (chunk, head): mats (0), packs (1), coef (2, float32).
extern "C" int li_wkv_chunk_elems(int d, int which) {
    const int DB = (d + 31) / 32;
    return which == 0 ? mat_elems(1, d) : (which == 1 ? 2 * DB * NP * 2 * 64 * 8 : 32 * DB);
}

extern "C" int li_wkv_chunks(const float* r, const float* k, const void* v, const float* raw, const float* bonus, float* state,
                             const int* seq_slot, const int* seq_qstart, const int* seq_qlen, const int* chunk_seq,
                             const int* chunk_t0, const int* seq_chunk0, int n_chunks, void* mats, float* coef, void* packs, float* y,
                             int n_seqs, int H, int d, hipStream_t stream) {
    if (n_seqs <= 0 || n_chunks <= 0) return LI_OK;
    if (H <= 0 || d <= 0 || !seq_qstart || !seq_qlen || !chunk_seq || !chunk_t0 || !seq_chunk0) return LI_BAD_ARG;
    if (d > 256) return LI_UNSUPPORTED;
    const Chunks cs{chunk_seq, chunk_t0, seq_chunk0, seq_slot, seq_qstart, seq_qlen};
    const int DB = (d + 31) / 32;
    const size_t lds1 = (size_t)((3 * CH + 1) * (32 * DB + 4) + CH * LDM) * sizeof(float);
    if (lds1 > 48 * 1024 && hipFuncSetAttribute((const void*)wkv_chunk_kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds1) != hipSuccess)
        return LI_HIP_ERROR;
    wkv_chunk_kernel<<<dim3(n_chunks, H), 256, lds1, stream>>>(r, k, (const bf16*)v, raw, bonus, cs, (bf16*)mats, coef,
                                                               (bf16*)packs, H, d);
    LI_CHECK_LAUNCH();
    const size_t lds2 = DB > 1 ? (size_t)2 * DB * 128 * 16 : 0;
    dim3 grid(n_seqs, H, (d + 15) / 16), block(64 * DB);
#define GO(NO) wkv_walk_kernel<NO><<<grid, block, lds2, stream>>>((const bf16*)mats, coef, (const bf16*)packs, state, cs, y, H, d)
    if (DB == 1) GO(2); else GO(1);
#undef GO
    LI_CHECK_LAUNCH();
    return LI_OK;
}
