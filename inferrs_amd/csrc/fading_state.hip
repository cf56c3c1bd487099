// A matrix a head whose ROWS fade, each by a factor of its own a token, and take in what the factor leaves open:
//     k_t = (1 - l) * sigmoid(-(z_t + b)),   f_t = 1 - k_t = l + (1 - l) * sigmoid(z_t + b)      (a gate a channel, l its floor)
//     S_t = diag(f_t) S_(t-1) + k_t v_t^T,   o_t = S_t^T silu(u_t)                                S: [dim x vdim]
// and behind it an RMS norm a head with one weight of vdim entries (the HGRN2 recurrence; Qin et al., "HGRN2: Gated Linear
// RNNs with State Expansion").  u, z and v are slices of the projections' rows; everything between their load and the
// store of the normed output is 32-bit, the state included.
//
// What a request carries lies in its row of a 32-bit state array [slots][row_floats], the matrices as [head][column j of S,
// vdim][dim].  A new request's row is zero.  f_t is formed as 1 - k_t everywhere (the rows stay within the values' range,
// so an error of 2^-25 of f weighs no more than a rounding of S).
//
// Two forms.  fading_walk_kernel walks a request's tokens in order (decode steps, short portions).  Long portions are cut
// into chunks of 64 tokens that run side by side, in three kernels of matrix products in true 32-bit
// (v_mfma_f32_16x16x4_f32), for keys of up to 128 and values of up to 256 entries:
//   fading_local     a chunk's own matrix U = sum_s (prod_(r>s) f_r) k_s v_s^T and the products A of its factors;
//   fading_chunks    a request's chunks in order, S <- A S + U from the state row; the workspace keeps what each starts from;
//   fading_outputs   o_t = (prod_(r<=t) f_r q_t) S_c + sum_(s<=t) P[t][s] v_s and the norm behind it.
// The scores P[t][s] = sum_i q_t[i] k_s[i] prod_(s<r<=t) f_r[i] are no product of two matrices, and their factors cannot be
// split at one point of a chunk (a quotient of products would over- or underflow).  A chunk is cut into four blocks of 16
// tokens: between blocks the factor splits at the borders, q_t (prod from its block's start) . (whole blocks between) .
// k_s (prod to its block's end), every piece a product of numbers up to 1; inside a block the vector units form the scores
// directly, a running product a key.
#include "api.h"
#include "common.h"

#define FS_R 8
#define FS_THREADS 256
#define FS_CHUNK 64
#define FS_SUB 16
#define FS_V_LD 36
#define FS_MAX_DIM 128
#define FS_MAX_VDIM 256

typedef float fs_f32x4 __attribute__((ext_vector_type(4)));

struct FadingArgs {
    void* out;                        // [n][H * vdim], normed (chunks), or 32-bit as it is (walk)
    float* state; long long row_floats, s_off;
    const void* proj; long long ld; int q_off, f_off, v_off;
    const float *f_bias, *lower;      // [H * dim]
    const float* norm_w; float eps;   // [vdim]
    const int *cu_tokens, *state_slots;
    int H, dim, vdim, cols, stage, wide, vec;
    int chunk0, chunks;               // chunks of this pass: the first one's number in its request, how many a request
    float *chunk_s, *chunk_a;         // [seqs][chunks][H][vdim][dim], [seqs][chunks][H][dim]
};

__device__ __forceinline__ float fs_open(float z, float b, float l) { return (1.0f - l) / (1.0f + expf(z + b)); }
__device__ __forceinline__ float fs_silu(float u) { return u / (1.0f + expf(-u)); }

// ---- token by token ---------------------------------------------------------------------------------------------------
// A block owns a (request, head, tile of S's columns); a column is shared by P neighbouring lanes, each with FS_R of its
// entries in registers; the operands of a stage of tokens come into shared memory together.
template <typename T, int P>
__global__ __launch_bounds__(FS_THREADS) void fading_walk_kernel(const FadingArgs a) {
    extern __shared__ __attribute__((aligned(16))) float fs_stage[];
    constexpr int dimp = P * FS_R;
    float* const q_s = fs_stage;
    float* const k_s = q_s + (size_t)a.stage * dimp;
    float* const v_s = k_s + (size_t)a.stage * dimp;
    const int p = threadIdx.x % P, jj = threadIdx.x / P;
    const int h = blockIdx.y, seq = blockIdx.z;
    const int j0 = blockIdx.x * a.cols, j = j0 + jj;
    const bool live = j < a.vdim;
    const int first = a.cu_tokens[seq], last = a.cu_tokens[seq + 1];
    const int i0 = p * FS_R;
    const T* q = (const T*)a.proj + a.q_off + (long long)h * a.dim;
    const T* z = (const T*)a.proj + a.f_off + (long long)h * a.dim;
    const T* v = (const T*)a.proj + a.v_off + (long long)h * a.vdim;
    float* srow = a.state + (long long)a.state_slots[seq] * a.row_floats + a.s_off + ((long long)h * a.vdim + (live ? j : 0)) * a.dim + i0;
    const bool wide = a.wide && i0 + FS_R <= a.dim;
    float S[FS_R];
    if (live && wide) {
        const float4 lo = *(const float4*)srow, hi = *(const float4*)(srow + 4);
        S[0] = lo.x; S[1] = lo.y; S[2] = lo.z; S[3] = lo.w; S[4] = hi.x; S[5] = hi.y; S[6] = hi.z; S[7] = hi.w;
    } else {
#pragma unroll
        for (int r = 0; r < FS_R; ++r) S[r] = (live && i0 + r < a.dim) ? srow[r] : 0.f;
    }
    for (int t0 = first; t0 < last; t0 += a.stage) {
        const int nt = last - t0 < a.stage ? last - t0 : a.stage;
        __syncthreads();                                          // (the stage before is used up)
        for (int e = threadIdx.x; e < nt * dimp; e += FS_THREADS) {
            const int tt = e / dimp, i = e - tt * dimp;
            float qv = 0.f, kv = 0.f;
            if (i < a.dim) {
                qv = fs_silu(ld(q + (long long)(t0 + tt) * a.ld + i));
                kv = fs_open(ld(z + (long long)(t0 + tt) * a.ld + i), a.f_bias[h * a.dim + i], a.lower[h * a.dim + i]);
            }
            q_s[e] = qv;
            k_s[e] = kv;
        }
        for (int e = threadIdx.x; e < nt * a.cols; e += FS_THREADS) {
            const int tt = e / a.cols, jv = j0 + e - tt * a.cols;
            v_s[e] = jv < a.vdim ? ld(v + (long long)(t0 + tt) * a.ld + jv) : 0.f;
        }
        __syncthreads();
#pragma unroll 2
        for (int tt = 0; tt < nt; ++tt) {
            const float4 qa = *(const float4*)(q_s + tt * dimp + i0), qb = *(const float4*)(q_s + tt * dimp + i0 + 4);
            const float4 ka = *(const float4*)(k_s + tt * dimp + i0), kb = *(const float4*)(k_s + tt * dimp + i0 + 4);
            const float qc[FS_R] = {qa.x, qa.y, qa.z, qa.w, qb.x, qb.y, qb.z, qb.w};
            const float kc[FS_R] = {ka.x, ka.y, ka.z, ka.w, kb.x, kb.y, kb.z, kb.w};
            const float vc = v_s[tt * a.cols + jj];
            float part = 0.f;
#pragma unroll
            for (int r = 0; r < FS_R; ++r) {
                S[r] = fmaf(1.0f - kc[r], S[r], kc[r] * vc);
                part = fmaf(S[r], qc[r], part);
            }
#pragma unroll
            for (int o = P / 2; o > 0; o >>= 1) part += __shfl_xor(part, o, IA_WAVE);
            if (p == 0 && live) ((float*)a.out)[((long long)(t0 + tt) * a.H + h) * a.vdim + j] = part;
        }
    }
    if (live && wide) {
        *(float4*)srow = make_float4(S[0], S[1], S[2], S[3]);
        *(float4*)(srow + 4) = make_float4(S[4], S[5], S[6], S[7]);
    } else if (live) {
#pragma unroll
        for (int r = 0; r < FS_R; ++r)
            if (i0 + r < a.dim) srow[r] = S[r];
    }
}

// ---- chunks side by side ----------------------------------------------------------------------------------------------
// Rows of a chunk into shared memory: dst[tt][i] = fn(src[(first + tt) * ld + i], i) for tt < nt, i < dim, zeros up to 64
// rows and d16 columns.  Four pieces of a thread are asked for before the first is used.
__device__ __forceinline__ void fs_load(const float* p, float (&v)[8]) {
    const float4 q = *(const float4*)p;
    v[0] = q.x; v[1] = q.y; v[2] = q.z; v[3] = q.w;
}
__device__ __forceinline__ void fs_load(const bf16_t* p, float (&v)[8]) {
    const uint4 q = *(const uint4*)p;
    const uint32_t w[4] = {q.x, q.y, q.z, q.w};
#pragma unroll
    for (int e = 0; e < 4; ++e) {
        v[2 * e] = __uint_as_float(w[e] << 16);
        v[2 * e + 1] = __uint_as_float(w[e] & 0xffff0000u);
    }
}

template <typename T, typename F>
__device__ __forceinline__ void fs_stage_rows(float* __restrict__ dst, int ld_s, const T* __restrict__ src, long long ld_g, int first,
                                              int nt, int dim, int d16, bool vec, F fn) {
    constexpr int E = 16 / (int)sizeof(T);
    if (vec) {                                             // (dim is a multiple of E, the rows start at multiples of 16 bytes)
        const int per_row = dim / E, total = FS_CHUNK * per_row;
        for (int b = 0; b < total; b += 4 * FS_THREADS) {
            float v[4][8];
#pragma unroll
            for (int it = 0; it < 4; ++it) {
                const int idx = b + it * FS_THREADS + threadIdx.x;
                const int tt = idx / per_row, piece = idx - tt * per_row;
                if (idx < total && tt < nt) fs_load(src + (long long)(first + tt) * ld_g + piece * E, v[it]);
            }
#pragma unroll
            for (int it = 0; it < 4; ++it) {
                const int idx = b + it * FS_THREADS + threadIdx.x;
                const int tt = idx / per_row, piece = idx - tt * per_row;
                if (idx >= total) continue;
                float* d = dst + tt * ld_s + piece * E;
#pragma unroll
                for (int e = 0; e < E; e += 4) {
                    float4 w = make_float4(0.f, 0.f, 0.f, 0.f);
                    if (tt < nt) w = make_float4(fn(v[it][e], piece * E + e), fn(v[it][e + 1], piece * E + e + 1),
                                                 fn(v[it][e + 2], piece * E + e + 2), fn(v[it][e + 3], piece * E + e + 3));
                    *(float4*)(d + e) = w;
                }
            }
        }
        if (d16 > dim)
            for (int e = threadIdx.x; e < FS_CHUNK * (d16 - dim); e += FS_THREADS)
                dst[e / (d16 - dim) * ld_s + dim + e % (d16 - dim)] = 0.f;
        return;
    }
    for (int e = threadIdx.x; e < FS_CHUNK * d16; e += FS_THREADS) {
        const int tt = e / d16, i = e - tt * d16;
        dst[tt * ld_s + i] = tt < nt && i < dim ? fn(ld(src + (long long)(first + tt) * ld_g + i), i) : 0.f;
    }
}

// 32 columns of v: v_s[tt][c] (zeros for tokens the chunk does not have and columns beyond vdim)
template <typename T>
__device__ __forceinline__ void fs_stage_values(float* __restrict__ v_s, const T* __restrict__ v, long long ld_g, int first, int nt,
                                                int j0, int vdim) {
    const int j = j0 + (threadIdx.x & 31);
    float vv[8];
#pragma unroll
    for (int it = 0; it < 8; ++it) {
        const int tt = (threadIdx.x >> 5) + 8 * it;
        vv[it] = tt < nt && j < vdim ? ld(v + (long long)(first + tt) * ld_g + j) : 0.f;
    }
#pragma unroll
    for (int it = 0; it < 8; ++it) v_s[((threadIdx.x >> 5) + 8 * it) * FS_V_LD + (threadIdx.x & 31)] = vv[it];
}

// A block of four waves owns a (chunk, head).
template <typename T>
__global__ __launch_bounds__(FS_THREADS) void fading_local_kernel(const FadingArgs a, int ld_s) {
    extern __shared__ __attribute__((aligned(16))) float fs_shared[];
    const int d16 = (a.dim + 15) / 16 * 16;
    float* const k_s = fs_shared;                          // [64][ld_s]
    float* const v_s = k_s + FS_CHUNK * ld_s;              // [64][FS_V_LD]
    float* const m_s = v_s + FS_CHUNK * FS_V_LD;           // [4][d16]: the products of the blocks' factors
    const int h = blockIdx.y;
    const int seq = blockIdx.z / a.chunks, c = blockIdx.z - seq * a.chunks;
    const int first = a.cu_tokens[seq] + (a.chunk0 + c) * FS_CHUNK, end = a.cu_tokens[seq + 1];
    if (first >= end) return;                              // (the whole block: this request has fewer chunks)
    const int nt = end - first < FS_CHUNK ? end - first : FS_CHUNK;
    const float *fb = a.f_bias + h * a.dim, *lo = a.lower + h * a.dim;
    const T* v = (const T*)a.proj + a.v_off + (long long)h * a.vdim;
    fs_stage_rows<T>(k_s, ld_s, (const T*)a.proj + a.f_off + (long long)h * a.dim, a.ld, first, nt, a.dim, d16, a.vec != 0,
                     [&](float z, int i) { return fs_open(z, fb[i], lo[i]); });
    __syncthreads();
    // (tokens the chunk does not have are zeros: their factor is 1)
    for (int e = threadIdx.x; e < 4 * d16; e += FS_THREADS) {
        const int sub = e / d16, i = e - sub * d16;
        float kk[FS_SUB], run = 1.f;
#pragma unroll
        for (int s = 0; s < FS_SUB; ++s) kk[s] = k_s[(FS_SUB * sub + s) * ld_s + i];
#pragma unroll
        for (int s = FS_SUB - 1; s >= 0; --s) {
            k_s[(FS_SUB * sub + s) * ld_s + i] = kk[s] * run;
            run *= 1.0f - kk[s];
        }
        m_s[e] = run;
    }
    __syncthreads();
    const long long unit = (long long)blockIdx.z * a.H + h;
    for (int i = threadIdx.x; i < a.dim; i += FS_THREADS)
        a.chunk_a[unit * a.dim + i] = m_s[i] * m_s[d16 + i] * m_s[2 * d16 + i] * m_s[3 * d16 + i];
    float* const u_out = a.chunk_s + unit * a.vdim * a.dim;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int r16 = lane & 15, kq = lane >> 4;
    const int row_tiles = d16 / 16;
    for (int j0 = 0; j0 < a.vdim; j0 += 32) {
        if (j0 > 0) __syncthreads();                       // (the columns before are used up)
        fs_stage_values<T>(v_s, v, a.ld, first, nt, j0, a.vdim);
        __syncthreads();
        for (int mt = wave; mt < row_tiles; mt += 4) {
            const int ii = 16 * mt + r16;
            const float m1 = m_s[d16 + ii], m2 = m_s[2 * d16 + ii], m3 = m_s[3 * d16 + ii];
            const float later[4] = {m1 * m2 * m3, m2 * m3, m3, 1.0f};
            fs_f32x4 acc[2] = {(fs_f32x4){0.f, 0.f, 0.f, 0.f}, (fs_f32x4){0.f, 0.f, 0.f, 0.f}};
            const float* ka = k_s + kq * ld_s + ii;
            const float* vb = v_s + kq * FS_V_LD + r16;
#pragma unroll
            for (int k0 = 0; k0 < FS_CHUNK; k0 += 4) {
                const float av = ka[k0 * ld_s] * later[k0 / FS_SUB];
                acc[0] = __builtin_amdgcn_mfma_f32_16x16x4f32(av, vb[k0 * FS_V_LD], acc[0], 0, 0, 0);
                acc[1] = __builtin_amdgcn_mfma_f32_16x16x4f32(av, vb[k0 * FS_V_LD + 16], acc[1], 0, 0, 0);
            }
#pragma unroll
            for (int c2 = 0; c2 < 2; ++c2) {
                const int col = j0 + 16 * c2 + r16;
                if (col >= a.vdim) continue;
                const int i = 16 * mt + 4 * kq;
                float* at = u_out + (long long)col * a.dim + i;
                if (a.wide && i + 4 <= a.dim) *(float4*)at = make_float4(acc[c2][0], acc[c2][1], acc[c2][2], acc[c2][3]);
                else {
#pragma unroll
                    for (int r = 0; r < 4; ++r)
                        if (i + r < a.dim) at[r] = acc[c2][r];
                }
            }
        }
    }
}

// A request's chunks in order, one thread an entry of the heads' matrices; eight chunks' entries are asked for at a time.
__global__ void fading_chunks_kernel(const FadingArgs a) {
    const long long e = (long long)blockIdx.x * blockDim.x + threadIdx.x;
    const int per_head = a.vdim * a.dim;
    const long long per_seq = (long long)a.H * per_head;
    if (e >= per_seq) return;
    const int seq = blockIdx.y;
    const int h = (int)(e / per_head), i = (int)(e % a.dim);
    int n = (a.cu_tokens[seq + 1] - a.cu_tokens[seq] + FS_CHUNK - 1) / FS_CHUNK - a.chunk0;
    n = n < a.chunks ? n : a.chunks;
    if (n <= 0) return;
    float* srow = a.state + (long long)a.state_slots[seq] * a.row_floats + a.s_off + e;
    float S = *srow;
    for (int c0 = 0; c0 < n; c0 += 8) {
        float u[8], f[8];
#pragma unroll
        for (int q = 0; q < 8; ++q) {
            if (c0 + q >= n) continue;
            const long long unit = (long long)seq * a.chunks + c0 + q;
            u[q] = a.chunk_s[unit * per_seq + e];
            f[q] = a.chunk_a[(unit * a.H + h) * a.dim + i];
        }
#pragma unroll
        for (int q = 0; q < 8; ++q) {
            if (c0 + q >= n) continue;
            a.chunk_s[((long long)seq * a.chunks + c0 + q) * per_seq + e] = S;
            S = fmaf(f[q], S, u[q]);
        }
    }
    *srow = S;
}

// A block of four waves owns a (chunk, head); wave w owns tokens 16 w .. 16 w + 15.  Shared memory: the queries, whose
// rows the scores replace once a wave has its own in registers; the keys, whose place the columns of v and of the matrix
// the chunk starts from take once the scores are formed.  NT: pairs of 16-column tiles that a wave keeps in registers.
template <typename T, int NT>
__global__ __launch_bounds__(FS_THREADS, 2) void fading_outputs_kernel(const FadingArgs a, int ld_s, int q_floats, int k_floats) {
    extern __shared__ __attribute__((aligned(16))) float fs_shared[];
    const int d16 = (a.dim + 15) / 16 * 16;
    float* const q_s = fs_shared;                          // [64][ld_s]
    float* const k_s = q_s + q_floats;                     // [64][ld_s]
    float* const m_s = k_s + k_floats;                     // [4][d16]
    float* const p_s = q_s;                                // [64][p_ld], in the queries' rows (or rows of 68 where those are shorter)
    const int p_ld = ld_s >= FS_CHUNK + 4 ? ld_s : FS_CHUNK + 4;
    float* const v_s = k_s;                                // [64][FS_V_LD]
    float* const c_s = v_s + FS_CHUNK * FS_V_LD;           // [32][ld_s]
    const int h = blockIdx.y;
    const int seq = blockIdx.z / a.chunks, c = blockIdx.z - seq * a.chunks;
    const int first = a.cu_tokens[seq] + (a.chunk0 + c) * FS_CHUNK, end = a.cu_tokens[seq + 1];
    if (first >= end) return;                              // (the whole block)
    const int nt = end - first < FS_CHUNK ? end - first : FS_CHUNK;
    const float *fb = a.f_bias + h * a.dim, *lo = a.lower + h * a.dim;
    const T* v = (const T*)a.proj + a.v_off + (long long)h * a.vdim;
    fs_stage_rows<T>(q_s, ld_s, (const T*)a.proj + a.q_off + (long long)h * a.dim, a.ld, first, nt, a.dim, d16, a.vec != 0,
                     [&](float u, int) { return fs_silu(u); });
    fs_stage_rows<T>(k_s, ld_s, (const T*)a.proj + a.f_off + (long long)h * a.dim, a.ld, first, nt, a.dim, d16, a.vec != 0,
                     [&](float z, int i) { return fs_open(z, fb[i], lo[i]); });
    __syncthreads();
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int r16 = lane & 15, kq = lane >> 4;
    // ---- the scores inside the wave's block of 16 tokens: lane (s, part) follows key s through the block, a quarter of
    // the channels a lane, w = k_s prod_(s<r<=t) f_r
    float inside[FS_SUB];
    {
        const float* q0 = q_s + FS_SUB * wave * ld_s + 4 * kq;
        const float* k0 = k_s + FS_SUB * wave * ld_s + 4 * kq;
        float w[FS_MAX_DIM / 16][4];
#pragma unroll
        for (int j = 0; j < FS_MAX_DIM / 16; ++j) {
            if (16 * j < d16) {
                const float4 kk = *(const float4*)(k0 + r16 * ld_s + 16 * j);
                w[j][0] = kk.x; w[j][1] = kk.y; w[j][2] = kk.z; w[j][3] = kk.w;
            }
        }
#pragma unroll
        for (int t = 0; t < FS_SUB; ++t) {
            float acc = 0.f;
            const bool behind = t > r16;
#pragma unroll
            for (int j = 0; j < FS_MAX_DIM / 16; ++j) {
                if (16 * j >= d16) continue;
                const float4 kt = *(const float4*)(k0 + t * ld_s + 16 * j), qt = *(const float4*)(q0 + t * ld_s + 16 * j);
                const float f[4] = {1.0f - kt.x, 1.0f - kt.y, 1.0f - kt.z, 1.0f - kt.w}, qq[4] = {qt.x, qt.y, qt.z, qt.w};
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    w[j][e] = behind ? w[j][e] * f[e] : w[j][e];
                    acc = fmaf(qq[e], w[j][e], acc);
                }
            }
            acc += __shfl_xor(acc, 16, IA_WAVE);
            acc += __shfl_xor(acc, 32, IA_WAVE);
            inside[t] = t >= r16 ? acc : 0.f;
        }
    }
    __builtin_amdgcn_wave_barrier();
    asm volatile("" ::: "memory");
    // ---- the block's own products: q_t from the block's start, k_s to its end (the wave's own rows: no barrier)
    for (int i = lane; i < d16; i += IA_WAVE) {
        float kk[FS_SUB], run = 1.f;
#pragma unroll
        for (int s = 0; s < FS_SUB; ++s) kk[s] = k_s[(FS_SUB * wave + s) * ld_s + i];
#pragma unroll
        for (int s = 0; s < FS_SUB; ++s) {
            run *= 1.0f - kk[s];
            q_s[(FS_SUB * wave + s) * ld_s + i] *= run;
        }
        m_s[wave * d16 + i] = run;
        run = 1.f;
#pragma unroll
        for (int s = FS_SUB - 1; s >= 0; --s) {
            k_s[(FS_SUB * wave + s) * ld_s + i] = kk[s] * run;
            run *= 1.0f - kk[s];
        }
    }
    __syncthreads();
    float aq[FS_MAX_DIM / 4];
#pragma unroll
    for (int kk = 0; kk < FS_MAX_DIM / 4; ++kk) aq[kk] = 4 * kk < d16 ? q_s[(FS_SUB * wave + r16) * ld_s + 4 * kk + kq] : 0.f;
    if (p_ld != ld_s) __syncthreads();                     // (rows of scores that do not lie in their own queries' rows)
    __builtin_amdgcn_wave_barrier();
    asm volatile("" ::: "memory");
    float* const mine = p_s + FS_SUB * wave * p_ld;
#pragma unroll
    for (int t = 0; t < FS_SUB; ++t)
        if ((t >> 2) == kq) mine[t * p_ld + FS_SUB * wave + r16] = inside[t];
    for (int cb = wave - 1; cb >= 0; --cb) {
        fs_f32x4 acc = (fs_f32x4){0.f, 0.f, 0.f, 0.f};
        const float* kb = k_s + (FS_SUB * cb + r16) * ld_s + kq;
#pragma unroll
        for (int kk = 0; kk < FS_MAX_DIM / 4; ++kk)
            if (4 * kk < d16) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(aq[kk], kb[4 * kk], acc, 0, 0, 0);
#pragma unroll
        for (int r = 0; r < 4; ++r) mine[(4 * kq + r) * p_ld + FS_SUB * cb + r16] = acc[r];
#pragma unroll
        for (int kk = 0; kk < FS_MAX_DIM / 4; ++kk)
            if (4 * kk < d16) aq[kk] *= m_s[cb * d16 + 4 * kk + kq];
    }
    // ---- the outputs, 32 columns at a time
    const float* start = a.chunk_s + ((long long)blockIdx.z * a.H + h) * a.vdim * a.dim;
    fs_f32x4 acc[NT][2];
#pragma unroll
    for (int jt = 0; jt < NT; ++jt) {
        acc[jt][0] = acc[jt][1] = (fs_f32x4){0.f, 0.f, 0.f, 0.f};
        const int j0 = 32 * jt;
        if (j0 >= a.vdim) continue;
        __syncthreads();                                   // (the keys, or the columns before, are used up)
        fs_stage_values<T>(v_s, v, a.ld, first, nt, j0, a.vdim);
        const int here = a.vdim - j0 < 32 ? a.vdim - j0 : 32;
        if (a.wide) {
            const int per_row = d16 / 4;
            for (int idx = threadIdx.x; idx < 32 * per_row; idx += FS_THREADS) {
                const int jj = idx / per_row, piece = idx - jj * per_row;
                const float4 z = jj < here && 4 * piece < a.dim ? *(const float4*)(start + (long long)(j0 + jj) * a.dim + 4 * piece)
                                                                : make_float4(0.f, 0.f, 0.f, 0.f);
                *(float4*)(c_s + jj * ld_s + 4 * piece) = z;
            }
        } else {
            for (int e = threadIdx.x; e < 32 * d16; e += FS_THREADS) {
                const int jj = e / d16, i = e - jj * d16;
                c_s[jj * ld_s + i] = (jj < here && i < a.dim) ? start[(long long)(j0 + jj) * a.dim + i] : 0.f;
            }
        }
        __syncthreads();
        const float* sb = c_s + r16 * ld_s + kq;
#pragma unroll
        for (int kk = 0; kk < FS_MAX_DIM / 4; ++kk) {
            if (4 * kk >= d16) continue;
            acc[jt][0] = __builtin_amdgcn_mfma_f32_16x16x4f32(aq[kk], sb[4 * kk], acc[jt][0], 0, 0, 0);
            acc[jt][1] = __builtin_amdgcn_mfma_f32_16x16x4f32(aq[kk], sb[16 * ld_s + 4 * kk], acc[jt][1], 0, 0, 0);
        }
        const float* pa = mine + r16 * p_ld + kq;
        const float* vb = v_s + kq * FS_V_LD + r16;
#pragma unroll 4
        for (int k0 = 0; k0 < FS_SUB * (wave + 1); k0 += 4) {
            const float av = pa[k0];
            acc[jt][0] = __builtin_amdgcn_mfma_f32_16x16x4f32(av, vb[k0 * FS_V_LD], acc[jt][0], 0, 0, 0);
            acc[jt][1] = __builtin_amdgcn_mfma_f32_16x16x4f32(av, vb[k0 * FS_V_LD + 16], acc[jt][1], 0, 0, 0);
        }
    }
    // ---- the norm over a head's columns, row by row (the 16 lanes of a row's values hold its columns)
    float rs[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int jt = 0; jt < NT; ++jt)
#pragma unroll
        for (int c2 = 0; c2 < 2; ++c2)
#pragma unroll
            for (int r = 0; r < 4; ++r) rs[r] = fmaf(acc[jt][c2][r], acc[jt][c2][r], rs[r]);   // (columns beyond vdim are zero)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
#pragma unroll
        for (int o = 8; o > 0; o >>= 1) rs[r] += __shfl_xor(rs[r], o, IA_WAVE);
        rs[r] = 1.0f / sqrtf(rs[r] / (float)a.vdim + a.eps);
    }
#pragma unroll
    for (int jt = 0; jt < NT; ++jt)
#pragma unroll
        for (int c2 = 0; c2 < 2; ++c2) {
            const int col = 32 * jt + 16 * c2 + r16;
            if (col >= a.vdim) continue;
            const float w = a.norm_w[col];
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int tt = FS_SUB * wave + 4 * kq + r;
                if (tt < nt) st((T*)a.out + ((long long)(first + tt) * a.H + h) * a.vdim + col, acc[jt][c2][r] * rs[r] * w);
            }
        }
}

// Floats of workspace for passes of `chunks` chunks a request.
extern "C" long long ia_fading_scan_workspace(int n_seqs, int chunks, int H, int dim, int vdim) {
    return (long long)n_seqs * chunks * ((long long)H * vdim * dim + (long long)H * dim);
}

static int fading_shared(const void* fn, int bytes, int& asked, const char* who) {
    if (bytes > asked && bytes > 64 * 1024) {
        const hipError_t e = hipFuncSetAttribute(fn, hipFuncAttributeMaxDynamicSharedMemorySize, 96 * 1024);
        IA_CHECK(e == hipSuccess, "%s: cannot ask for %d bytes of shared memory: %s", who, bytes, hipGetErrorString(e));
        asked = 96 * 1024;
    }
    IA_CHECK(bytes <= 96 * 1024, "%s: %d bytes of shared memory", who, bytes);
    return 0;
}

// chunks 0: every request's tokens are walked from its state row; out is 32-bit and not normed.  chunks > 0: chunks of 64
// tokens side by side, `chunks` of a request at a time (max_q_len: the most tokens a request brings); out is normed, in the
// precision of proj.  q, the gate's logits and v lie at q_off, f_off and v_off of proj's rows.
extern "C" int ia_fading_scan(void* out, float* state, long long row_floats, long long s_off, const void* proj, long long ld, int q_off,
                              int f_off, int v_off, const float* f_bias, const float* lower, const float* norm_w, float eps,
                              const int* cu_tokens, const int* state_slots, int n_seqs, int H, int dim, int vdim, int max_q_len,
                              int chunks, float* workspace, int dtype, hipStream_t stream) {
    IA_CHECK(n_seqs >= 0 && H > 0 && dim > 0 && vdim > 0 && max_q_len >= 1, "fading_scan: bad sizes heads=%d dim=%d vdim=%d", H, dim, vdim);
    IA_CHECK(dim <= FS_R * IA_WAVE, "fading_scan: a key size of %d is beyond %d", dim, FS_R * IA_WAVE);
    IA_CHECK(s_off >= 0 && s_off + (long long)H * vdim * dim <= row_floats, "fading_scan: the matrices do not fit the state row");
    IA_CHECK(q_off >= 0 && q_off + (long long)H * dim <= ld && f_off >= 0 && f_off + (long long)H * dim <= ld && v_off >= 0 &&
             v_off + (long long)H * vdim <= ld, "fading_scan: q, f or v lie outside their rows");
    IA_CHECK(dtype == IA_F32 || dtype == IA_BF16, "fading_scan: unknown dtype %d", dtype);
    if (n_seqs == 0) return 0;
    FadingArgs a;
    a.out = out; a.state = state; a.row_floats = row_floats; a.s_off = s_off;
    a.proj = proj; a.ld = ld; a.q_off = q_off; a.f_off = f_off; a.v_off = v_off;
    a.f_bias = f_bias; a.lower = lower; a.norm_w = norm_w; a.eps = eps; a.cu_tokens = cu_tokens; a.state_slots = state_slots;
    a.H = H; a.dim = dim; a.vdim = vdim; a.cols = 0; a.stage = 0; a.chunk0 = 0; a.chunks = 0; a.chunk_s = a.chunk_a = nullptr;
    a.wide = dim % 4 == 0 && s_off % 4 == 0 && row_floats % 4 == 0 && (((uintptr_t)state | (uintptr_t)workspace) & 15) == 0;
    const int per = dtype == IA_F32 ? 4 : 8;
    a.vec = dim % per == 0 && q_off % per == 0 && f_off % per == 0 && ld % per == 0 && ((uintptr_t)proj & 15) == 0;
    if (chunks == 0) {
        int P = 1;
        while (P * FS_R < dim) P *= 2;
        a.cols = FS_THREADS / P;
        const int per_token = 2 * P * FS_R + a.cols;
        int stage = 32 * 1024 / 4 / per_token;
        stage = stage > 32 ? 32 : stage < 2 ? 2 : stage;
        a.stage = stage < max_q_len ? stage : max_q_len;
        const size_t shm = (size_t)a.stage * per_token * sizeof(float);
        const dim3 grid((unsigned)((vdim + a.cols - 1) / a.cols), (unsigned)H, (unsigned)n_seqs);
        IA_CHECK(H <= 65535 && n_seqs <= 65535, "fading_scan: %d heads of %d requests exceed the grid", H, n_seqs);
#define FS_WALK(PP)                                                                                         \
    do {                                                                                                    \
        if (dtype == IA_F32) fading_walk_kernel<float, PP><<<grid, FS_THREADS, shm, stream>>>(a);           \
        else fading_walk_kernel<bf16_t, PP><<<grid, FS_THREADS, shm, stream>>>(a);                          \
    } while (0)
        switch (P) {
            case 1: FS_WALK(1); break;
            case 2: FS_WALK(2); break;
            case 4: FS_WALK(4); break;
            case 8: FS_WALK(8); break;
            case 16: FS_WALK(16); break;
            case 32: FS_WALK(32); break;
            default: FS_WALK(64); break;
        }
#undef FS_WALK
        IA_LAUNCH_CHECK("fading_scan");
        return 0;
    }
    IA_CHECK(dim <= FS_MAX_DIM && vdim <= FS_MAX_VDIM && workspace != nullptr && norm_w != nullptr && chunks > 0,
             "fading_scan: chunks take keys up to %d, values up to %d, a workspace and the norm's weight", FS_MAX_DIM, FS_MAX_VDIM);
    IA_CHECK((long long)n_seqs * chunks <= 65535 && H <= 65535, "fading_scan: %d requests x %d chunks exceed the grid", n_seqs, chunks);
    const int d16 = (dim + 15) / 16 * 16, ld_s = d16 + 4;
    const int lshm = (FS_CHUNK * ld_s + FS_CHUNK * FS_V_LD + 4 * d16) * 4;
    const int q_floats = FS_CHUNK * (ld_s > FS_CHUNK + 4 ? ld_s : FS_CHUNK + 4);
    const int tiles = FS_CHUNK * FS_V_LD + 32 * ld_s;
    const int k_floats = FS_CHUNK * ld_s > tiles ? FS_CHUNK * ld_s : tiles;
    const int oshm = (q_floats + k_floats + 4 * d16) * 4;
    a.chunks = chunks;
    a.chunk_s = workspace;
    a.chunk_a = workspace + (long long)n_seqs * chunks * H * vdim * dim;
    const dim3 cgrid(1, (unsigned)H, (unsigned)(n_seqs * chunks));
    const dim3 sgrid((unsigned)(((long long)H * vdim * dim + 255) / 256), (unsigned)n_seqs);
    static int asked[2][2];
    for (a.chunk0 = 0; (long long)a.chunk0 * FS_CHUNK < max_q_len; a.chunk0 += chunks) {
        if (dtype == IA_F32) fading_local_kernel<float><<<cgrid, FS_THREADS, lshm, stream>>>(a, ld_s);
        else fading_local_kernel<bf16_t><<<cgrid, FS_THREADS, lshm, stream>>>(a, ld_s);
        fading_chunks_kernel<<<sgrid, 256, 0, stream>>>(a);
#define FS_OUT(TT, NT, I, J)                                                                                              \
    do {                                                                                                                  \
        if (fading_shared((const void*)fading_outputs_kernel<TT, NT>, oshm, asked[I][J], "fading_scan")) return 1;        \
        fading_outputs_kernel<TT, NT><<<cgrid, FS_THREADS, oshm, stream>>>(a, ld_s, q_floats, k_floats);                  \
    } while (0)
        if (dtype == IA_F32 && vdim <= 128) FS_OUT(float, 4, 0, 0);
        else if (dtype == IA_F32) FS_OUT(float, 8, 0, 1);
        else if (vdim <= 128) FS_OUT(bf16_t, 4, 1, 0);
        else FS_OUT(bf16_t, 8, 1, 1);
#undef FS_OUT
    }
    IA_LAUNCH_CHECK("fading_scan (chunks)");
    return 0;
}
