// The mLSTM recurrence over long segments (mlstm_chunks.hip holds the equations and the order of the three steps) for bfloat16 rows:
// q, k and v are bfloat16 as the projection leaves them, so every product has one side that is a bfloat16 already.  The other side
// (the state, the weights of a chunk's second sum, the values times their weights) is float and enters v_mfma_f32_16x16x32_bf16 as
// three bfloat16 terms, x = hi + mid + lo with 8 bits each: a product of a bfloat16 and a float to 24 bits, summed in float.
//
// Operands of 32 entries of the summed index: lane (r, q) holds the entries 4 q .. 4 q + 3 of both halves of 16, which is how the
// results of two 16 x 16 products lie, so a state or a tile of weights goes from one product into the next without a move.
// Columns of k and v come out of their rows in LDS through the transposing read (four tokens of a column a lane).
#include "mlstm.h"

typedef __attribute__((ext_vector_type(4))) float f32x4;
typedef __attribute__((ext_vector_type(2))) float f32x2;
typedef __attribute__((ext_vector_type(2))) __bf16 bf16x2;
typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(4))) short s16x4;

#define MV_LD (MCOLS + 8)      // elements a row of values in LDS
#define MO_LD (MCOLS + 4)      // floats a row of results in LDS

struct MbTerms { uint4 t[3]; };

__device__ __forceinline__ uint32_t mb_pack(float a, float b) {
    const f32x2 v = {a, b};
    return __builtin_bit_cast(uint32_t, __builtin_convertvector(v, bf16x2));
}
// two floats as three pairs of bfloat16
__device__ __forceinline__ void mb_split2(float a, float b, uint32_t& hi, uint32_t& mid, uint32_t& lo) {
    hi = mb_pack(a, b);
    a -= __uint_as_float(hi << 16);
    b -= __uint_as_float(hi & 0xffff0000u);
    mid = mb_pack(a, b);
    a -= __uint_as_float(mid << 16);
    b -= __uint_as_float(mid & 0xffff0000u);
    lo = mb_pack(a, b);
}
__device__ __forceinline__ MbTerms mb_split(const f32x4& a, const f32x4& b) {
    MbTerms r;
    uint32_t* h = reinterpret_cast<uint32_t*>(&r.t[0]);
    uint32_t* m = reinterpret_cast<uint32_t*>(&r.t[1]);
    uint32_t* l = reinterpret_cast<uint32_t*>(&r.t[2]);
    mb_split2(a[0], a[1], h[0], m[0], l[0]);
    mb_split2(a[2], a[3], h[1], m[1], l[1]);
    mb_split2(b[0], b[1], h[2], m[2], l[2]);
    mb_split2(b[2], b[3], h[3], m[3], l[3]);
    return r;
}
__device__ __forceinline__ f32x4 mb_mfma(const uint4& a, const uint4& b, f32x4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
}
// the small terms first
__device__ __forceinline__ f32x4 mb_mfma_b(const uint4& a, const MbTerms& b, f32x4 c) { return mb_mfma(a, b.t[0], mb_mfma(a, b.t[1], mb_mfma(a, b.t[2], c))); }

// four rows of 16 columns (rows `ld` elements apart from `at` on): lane (r, q) of a quarter wave gets rows 0 .. 3 of column r
__device__ __forceinline__ uint2 mb_columns(const bf16* at, int ld, int r) {
    const bf16* p = at + (r >> 2) * ld + (r & 3) * 4;
    const s16x4 v = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)p);
    return __builtin_bit_cast(uint2, v);
}
// ... of the 32 tokens from row t0 on, as an operand
__device__ __forceinline__ uint4 mb_operand(const bf16* at, int ld, int r, int q) {
    const uint2 a = mb_columns(at + 4 * q * ld, ld, r), b = mb_columns(at + (16 + 4 * q) * ld, ld, r);
    return make_uint4(a.x, a.y, b.x, b.y);
}
__device__ __forceinline__ void mb_unpack(uint32_t p, float& a, float& b) {
    a = __uint_as_float(p << 16);
    b = __uint_as_float(p & 0xffff0000u);
}

// rows of MC tokens with `nc` columns each, filled up with zeros to W columns and MC rows
template <int W>
__device__ __forceinline__ void mb_stage(int tid, bf16* __restrict__ dst, int ld, const bf16* __restrict__ src, long stride, int n, int nc, bool vec) {
    if (vec) {
#pragma unroll
        for (int i = tid; i < MC * (W / 8); i += MW * 64) {
            const int t = i / (W / 8), c = (i % (W / 8)) * 8;
            uint4 v = make_uint4(0u, 0u, 0u, 0u);
            if (t < n && c < nc) v = *reinterpret_cast<const uint4*>(src + (size_t)t * stride + c);
            *reinterpret_cast<uint4*>(&dst[t * ld + c]) = v;
        }
        return;
    }
#pragma unroll 1
    for (int i = tid; i < MC * W; i += MW * 64) {
        const int t = i / W, c = i % W;
        dst[t * ld + c] = (t < n && c < nc) ? src[(size_t)t * stride + c] : from_f32<bf16>(0.f);
    }
}

// the state's tiles over a chunk: S = keep S + K^T (put V); v: the wave's columns as operands of tokens 0 .. 31 and 32 .. 63
template <int KT>
__device__ __forceinline__ void mb_carry(f32x4 (&S)[KT], const bf16* __restrict__ Ks, const uint4 (&v)[2], const float* __restrict__ put, float keep,
                                         int r, int q) {
    constexpr int LD = KT * 16 + 8;
#pragma unroll
    for (int m = 0; m < KT; ++m) S[m] = S[m] * keep;
#pragma unroll
    for (int b = 0; b < 2; ++b) {
        const float4 p0 = *reinterpret_cast<const float4*>(&put[32 * b + 4 * q]), p1 = *reinterpret_cast<const float4*>(&put[32 * b + 16 + 4 * q]);
        float u[8];
        mb_unpack(v[b].x, u[0], u[1]);
        mb_unpack(v[b].y, u[2], u[3]);
        mb_unpack(v[b].z, u[4], u[5]);
        mb_unpack(v[b].w, u[6], u[7]);
        const f32x4 w0 = f32x4{u[0] * p0.x, u[1] * p0.y, u[2] * p0.z, u[3] * p0.w}, w1 = f32x4{u[4] * p1.x, u[5] * p1.y, u[6] * p1.z, u[7] * p1.w};
        const MbTerms w = mb_split(w0, w1);
#pragma unroll
        for (int m = 0; m < KT; ++m) S[m] = mb_mfma_b(mb_operand(Ks + 32 * b * LD + 16 * m, LD, r, q), w, S[m]);
    }
}

// n, a part of the tokens a thread: thread (part, d) of the block adds the tokens 16 part .. of entry d
template <int KT>
__device__ __forceinline__ float mb_carry_n(float n, const bf16* __restrict__ Ks, const float* __restrict__ put, float keep) {
    constexpr int LD = KT * 16 + 8;
    const int d = threadIdx.x & 127, part = threadIdx.x >> 7;
    if (d >= KT * 16) return 0.f;
    n *= keep;
#pragma unroll
    for (int i = 0; i < 16; ++i) n = fmaf(to_f32(Ks[(part * 16 + i) * LD + d]), put[part * 16 + i], n);
    return n;
}

__device__ __forceinline__ double mb_scan_max(double v, int lane) {
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
        const double up = __shfl_up(v, off, 64);
        if (lane >= off) v = fmax(v, up);
    }
    return v;
}

// KS: key entries / 32.  ws_g: (a_t, L_t) of every (token, head), counted from the token's piece.
template <int KS>
__global__ void __launch_bounds__(MW * 64, 4)
mlstm_states_mfma_kernel(float4* __restrict__ ws_s, float* __restrict__ ws_n, double* __restrict__ ws_m, double2* __restrict__ ws_g, MlRows a,
                         const int* __restrict__ seg_offsets, int R, int H, int dk, int dv, int CT, int piece, int min_len, int vec) {
    constexpr int KT = 2 * KS, DK = 32 * KS, LD = DK + 8;
    __shared__ __attribute__((aligned(16))) bf16 Ks[MC * LD];
    __shared__ __attribute__((aligned(16))) bf16 Vs[MC * MV_LD];
    __shared__ __attribute__((aligned(16))) float put[MC];
    __shared__ float keep;
    __shared__ float nred[4][128];
    const int h = blockIdx.x % H, cg = blockIdx.x / H, slot = blockIdx.y;
    int p;
    const int seg = ml_find(seg_offsets, R, piece, slot, p);
    if (seg < 0) return;
    const int len = seg_offsets[seg + 1] - seg_offsets[seg];
    if (len < min_len) return;                         // (the step kernel's)
    const int p0 = seg_offsets[seg] + p * piece, plen = min(piece, len - p * piece);
    const int tid = threadIdx.x, lane = tid & 63, r = lane & 15, q = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int ct = cg * MW + wave;
    const bf16* base = (const bf16*)a.rows;
    f32x4 S[KT];
#pragma unroll
    for (int m = 0; m < KT; ++m) S[m] = f32x4{0.f, 0.f, 0.f, 0.f};
    float n = 0.f;
    double L = 0.0, M = -INFINITY;
    for (int c0 = 0; c0 < plen; c0 += MC) {
        const int t0 = p0 + c0, cn = min(MC, plen - c0);
        const bf16* row = base + (size_t)t0 * a.stride;
        float zi = 0.f, zf = 0.f;
        if (wave == 0) ml_raw_gates<bf16>(a, (size_t)t0 + (lane < cn ? lane : cn - 1), h, zi, zf);
        __syncthreads();                               // the last chunk's readers are done
        mb_stage<DK>(tid, Ks, LD, row + (size_t)(H + h) * dk, a.stride, cn, dk, vec & 1);
        mb_stage<MCOLS>(tid, Vs, MV_LD, row + (size_t)2 * H * dk + (size_t)h * dv + cg * MCOLS, a.stride, cn, dv - cg * MCOLS, vec & 2);
        if (wave == 0) {
            const float li = ml_capped(zi, a.cap), lf = ml_log_sigmoid(ml_capped(zf, a.cap));
            double Lt = lane < cn ? (double)lf : 0.0;
#pragma unroll
            for (int off = 1; off < 64; off <<= 1) {
                const double up = __shfl_up(Lt, off, 64);
                if (lane >= off) Lt += up;
            }
            Lt += L;
            const double at = lane < cn ? (double)li - Lt : -INFINITY;
            double Mend = at;
#pragma unroll
            for (int off = 1; off < 64; off <<= 1) Mend = fmax(Mend, __shfl_xor(Mend, off, 64));
            Mend = fmax(Mend, M);
            put[lane] = lane < cn ? expf((float)(at - Mend)) : 0.f;
            if (cg == 0 && lane < cn) ws_g[(size_t)(t0 + lane) * H + h] = make_double2(at, Lt);
            if (lane == 0) keep = expf((float)(M - Mend));
            M = Mend;
            L = __shfl(Lt, 63, 64);
        }
        __syncthreads();
        if (ct < CT) {
            uint4 v[2];
#pragma unroll
            for (int b = 0; b < 2; ++b) v[b] = mb_operand(Vs + 32 * b * MV_LD + 16 * wave, MV_LD, r, q);
            mb_carry<KT>(S, Ks, v, put, keep, r, q);
        }
        if (cg == 0) n = mb_carry_n<KT>(n, Ks, put, keep);
    }
    const size_t sh = (size_t)slot * H + h;
    if (ct < CT) {
#pragma unroll
        for (int m = 0; m < KT; ++m) ws_s[((sh * CT + ct) * KT + m) * 64 + lane] = make_float4(S[m][0], S[m][1], S[m][2], S[m][3]);
    }
    if (cg != 0) return;                               // (a whole block)
    nred[threadIdx.x >> 7][threadIdx.x & 127] = n;
    __syncthreads();
    if (threadIdx.x < DK) ws_n[sh * DK + threadIdx.x] = (nred[0][threadIdx.x] + nred[1][threadIdx.x]) + (nred[2][threadIdx.x] + nred[3][threadIdx.x]);
    if (threadIdx.x == 0) {
        ws_m[sh * 3] = L;
        ws_m[sh * 3 + 1] = M;
    }
}

// NORM: a block holds all columns of the head and ends with the output norm, weight and gate
template <int KS, bool NORM>
__global__ void __launch_bounds__(MW * 64, 4)
mlstm_outputs_mfma_kernel(float* __restrict__ out, void* __restrict__ y, const float4* __restrict__ ws_s, const float* __restrict__ ws_n,
                          const double* __restrict__ ws_m, const double2* __restrict__ ws_g, MlRows a, float* __restrict__ pool_m,
                          const int* __restrict__ state_out, const int* __restrict__ seg_offsets, int R, int H, int dk, int dv, int CT, int piece,
                          int min_len, int y_stride, int y_dt, int vec) {
    constexpr int KT = 2 * KS, DK = 32 * KS, LD = DK + 8;
    constexpr int QK = 2 * MC * LD * (int)sizeof(bf16), OB = MC * MO_LD * (int)sizeof(float);
    __shared__ __attribute__((aligned(16))) char buf[QK > OB ? QK : OB];     // q and k rows of a chunk, then its results
    __shared__ __attribute__((aligned(16))) bf16 Vs[MC * MV_LD];
    // the weights of the second sum as operands: (row tile, pair of column tiles) 0: (0, 0), 1: (1, 0), 2, 3: (2, 0 | 1), 4, 5: (3, 0 | 1)
    __shared__ __attribute__((aligned(16))) uint4 Ps[6][3][64];
    __shared__ double As[MC], Ms[MC];
    __shared__ __attribute__((aligned(16))) float put[MC], start[MC], floor_[MC];
    __shared__ float keep;
    __shared__ float nred[4][128];
    __shared__ float rs[4][MC], nq[MC];
    bf16* Qs = reinterpret_cast<bf16*>(buf);
    bf16* Ks = Qs + MC * LD;
    float* Os = reinterpret_cast<float*>(buf);
    const int h = blockIdx.x % H, cg = blockIdx.x / H, slot = blockIdx.y;
    int p;
    const int seg = ml_find(seg_offsets, R, piece, slot, p);
    if (seg < 0) return;
    const int len = seg_offsets[seg + 1] - seg_offsets[seg];
    if (len < min_len) return;
    const int p0 = seg_offsets[seg] + p * piece, plen = min(piece, len - p * piece);
    int tid = threadIdx.x;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int ct = cg * MW + wave;
    const bf16* base = (const bf16*)a.rows;
    const size_t sh = (size_t)slot * H + h;
    f32x4 S[KT];
#pragma unroll
    for (int m = 0; m < KT; ++m) {
        const float4 t = ws_s[((sh * CT + (ct < CT ? ct : 0)) * KT + m) * 64 + (tid & 63)];
        S[m] = f32x4{t.x, t.y, t.z, t.w};
    }
    float n = tid < DK && tid < 128 ? ws_n[sh * DK + tid] : 0.f;       // (part 0 starts from the whole, the others from nothing)
    double M = ws_m[sh * 3 + 2], m_last = 0.0;
    for (int c0 = 0; c0 < plen; c0 += MC) {
        // (opaque: every address that follows from the thread's number would else be formed before the loop and held in registers)
        asm volatile("" : "+v"(tid));
        const int lane = tid & 63, r = lane & 15, q = lane >> 4;
        const int t0 = p0 + c0, cn = min(MC, plen - c0);
        const bf16* row = base + (size_t)t0 * a.stride;
        double2 al = make_double2(0.0, 0.0);
        if (wave == 0) al = ws_g[(size_t)(t0 + (lane < cn ? lane : cn - 1)) * H + h];
        __syncthreads();                               // the last chunk's readers are done
        mb_stage<DK>(tid, Qs, LD, row + (size_t)h * dk, a.stride, cn, dk, vec & 1);
        mb_stage<DK>(tid, Ks, LD, row + (size_t)(H + h) * dk, a.stride, cn, dk, vec & 1);
        mb_stage<MCOLS>(tid, Vs, MV_LD, row + (size_t)2 * H * dk + (size_t)h * dv + cg * MCOLS, a.stride, cn, dv - cg * MCOLS, vec & 2);
        nred[tid >> 7][tid & 127] = n;
        if (wave == 0) {
            const double at = lane < cn ? al.x : -INFINITY;
            const double Mt = fmax(mb_scan_max(at, lane), M), Mend = __shfl(Mt, 63, 64);
            As[lane] = at;
            Ms[lane] = Mt;
            put[lane] = lane < cn ? expf((float)(at - Mend)) : 0.f;
            start[lane] = expf((float)(M - Mt));
            floor_[lane] = expf(-(float)(al.y + Mt));
            if (lane == 0) keep = expf((float)(M - Mend));
            M = Mend;
            m_last = __shfl(al.y, 63, 64) + Mend;
        }
        __syncthreads();
        // ---- weights exp(a_i - M_t) (k_i . q_t) as [i, t], by tiles at and below the diagonal, and their sums over i
        for (int tile = wave; tile < 10; tile += MW) {
            const int rt = tile < 1 ? 0 : (tile < 3 ? 1 : (tile < 6 ? 2 : 3)), kt = tile - rt * (rt + 1) / 2;
            f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int s = 0; s < KS; ++s)
                acc = mb_mfma(*reinterpret_cast<const uint4*>(&Ks[(16 * kt + r) * LD + 32 * s + 8 * q]),
                              *reinterpret_cast<const uint4*>(&Qs[(16 * rt + r) * LD + 32 * s + 8 * q]), acc);
            const double Mt = Ms[16 * rt + r];
            float w[4], sum = 0.f;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int i = 16 * kt + 4 * q + e;
                w[e] = i <= 16 * rt + r ? expf((float)(As[i] - Mt)) * acc[e] : 0.f;
                sum += w[e];
            }
            sum += __shfl_xor(sum, 16, 64);
            sum += __shfl_xor(sum, 32, 64);
            if (q == 0) rs[kt][16 * rt + r] = sum;
            uint2 t[3];
            mb_split2(w[0], w[1], t[0].x, t[1].x, t[2].x);
            mb_split2(w[2], w[3], t[0].y, t[1].y, t[2].y);
            const int set = (rt < 2 ? rt : 2 * rt - 2) + (kt >> 1);
#pragma unroll
            for (int i = 0; i < 3; ++i) {
                uint2* at = reinterpret_cast<uint2*>(&Ps[set][i][lane]);
                at[kt & 1] = t[i];
                if (kt == rt && !(kt & 1)) at[1] = make_uint2(0u, 0u);     // (the tile beside it lies above the diagonal)
            }
        }
        {   // n . q_t before the chunk, eight lanes a token
            const int t = tid >> 3, part = tid & 7;
            float s = 0.f;
#pragma unroll 4
            for (int d = part * (DK / 8); d < (part + 1) * (DK / 8); ++d)
                s = fmaf((nred[0][d] + nred[1][d]) + (nred[2][d] + nred[3][d]), to_f32(Qs[t * LD + d]), s);
            s += __shfl_xor(s, 1, 64);
            s += __shfl_xor(s, 2, 64);
            s += __shfl_xor(s, 4, 64);
            if (part == 0) nq[t] = s;
        }
        __syncthreads();
        // ---- exp(m_s - M_t) q S + P V
        f32x4 x[4];
#pragma unroll
        for (int rt = 0; rt < 4; ++rt) x[rt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < KS; ++s) {
            const MbTerms b = mb_split(S[2 * s], S[2 * s + 1]);
#pragma unroll
            for (int rt = 0; rt < 4; ++rt) {
                const uint2 lo = *reinterpret_cast<const uint2*>(&Qs[(16 * rt + r) * LD + 32 * s + 4 * q]),
                            hi = *reinterpret_cast<const uint2*>(&Qs[(16 * rt + r) * LD + 32 * s + 16 + 4 * q]);
                x[rt] = mb_mfma_b(make_uint4(lo.x, lo.y, hi.x, hi.y), b, x[rt]);
            }
            __builtin_amdgcn_sched_barrier(0);         // (the terms of one step's state at a time in registers)
        }
        uint4 v[2];
#pragma unroll
        for (int b = 0; b < 2; ++b) v[b] = mb_operand(Vs + 32 * b * MV_LD + 16 * wave, MV_LD, r, q);
#pragma unroll
        for (int rt = 0; rt < 4; ++rt) {
            const float4 st = *reinterpret_cast<const float4*>(&start[16 * rt + 4 * q]);
            x[rt] = f32x4{x[rt][0] * st.x, x[rt][1] * st.y, x[rt][2] * st.z, x[rt][3] * st.w};
#pragma unroll
            for (int b = 0; b <= rt / 2; ++b) {
                const int set = (rt < 2 ? rt : 2 * rt - 2) + b;
                x[rt] = mb_mfma(Ps[set][2][lane], v[b], x[rt]);
                x[rt] = mb_mfma(Ps[set][1][lane], v[b], x[rt]);
                x[rt] = mb_mfma(Ps[set][0][lane], v[b], x[rt]);
            }
        }
        if (c0 + MC < plen) {
            mb_carry<KT>(S, Ks, v, put, keep, r, q);
            n = mb_carry_n<KT>(n, Ks, put, keep);
        }
        __syncthreads();                               // q and k are done with: their place takes the results
#pragma unroll
        for (int rt = 0; rt < 4; ++rt)
#pragma unroll
            for (int e = 0; e < 4; ++e) Os[(16 * rt + 4 * q + e) * MO_LD + 16 * wave + r] = x[rt][e];
        __syncthreads();
        // ---- rows: eight threads a token, 16 columns each
        const int t = tid >> 3, cb = (tid & 7) * 16, nc = min(dv - cg * MCOLS, MCOLS);
        float d = start[t] * nq[t];
        for (int j = 0; j <= t / 16; ++j) d += rs[j][t];
        const float to_o = a.scale / (fmaxf(fabsf(d * a.scale), floor_[t]) + 1e-6f);
        if constexpr (NORM) {
            float ov[16];
#pragma unroll
            for (int i = 0; i < 16; i += 4) {
                const float4 f = *reinterpret_cast<const float4*>(&Os[t * MO_LD + cb + i]);
                ov[i] = f.x * to_o; ov[i + 1] = f.y * to_o; ov[i + 2] = f.z * to_o; ov[i + 3] = f.w * to_o;
            }
            float ss = 0.f;
#pragma unroll
            for (int i = 0; i < 16; ++i) ss = cb + i < nc ? fmaf(ov[i], ov[i], ss) : ss;
            ss += __shfl_xor(ss, 1, 64);
            ss += __shfl_xor(ss, 2, 64);
            ss += __shfl_xor(ss, 4, 64);
            const float rstd = 1.0f / sqrtf(ss / (float)dv + a.eps);
            if (t < cn) {
                const int j0 = h * dv + cb;
                const bf16* gp = row + (size_t)t * a.stride + a.g_off + j0;
                if (vec & 4) {       // (everything bfloat16, in pieces of eight)
#pragma unroll
                    for (int i = 0; i < 16; i += 8)
                        if (cb + i < nc) {
                            const uint4 g = *reinterpret_cast<const uint4*>(gp + i), w = *reinterpret_cast<const uint4*>((const bf16*)a.norm_w + j0 + i);
                            const uint32_t gw[4] = {g.x, g.y, g.z, g.w}, ww[4] = {w.x, w.y, w.z, w.w};
                            uint32_t z[4];
#pragma unroll
                            for (int e = 0; e < 4; ++e) {
                                float g0, g1, w0, w1;
                                mb_unpack(gw[e], g0, g1);
                                mb_unpack(ww[e], w0, w1);
                                z[e] = mb_pack(ov[i + 2 * e] * rstd * w0 * ml_sigmoid(g0), ov[i + 2 * e + 1] * rstd * w1 * ml_sigmoid(g1));
                            }
                            *reinterpret_cast<uint4*>((bf16*)y + (size_t)(t0 + t) * y_stride + j0 + i) = make_uint4(z[0], z[1], z[2], z[3]);
                        }
                } else {
#pragma unroll 1
                    for (int i = 0; i < 16; ++i)
                        if (cb + i < nc) {
                            const float z = Os[t * MO_LD + cb + i] * to_o * rstd * ml_any(a.norm_w, a.w_dt, j0 + i) * ml_sigmoid(to_f32(gp[i]));
                            if (y_dt == ILM_DTYPE_F32) ((float*)y)[(size_t)(t0 + t) * y_stride + j0 + i] = z;
                            else ((bf16*)y)[(size_t)(t0 + t) * y_stride + j0 + i] = from_f32<bf16>(z);
                        }
                }
            }
        } else if (t < cn) {
            float* op = out + ((size_t)(t0 + t) * H + h) * dv + cg * MCOLS + cb;
#pragma unroll 1
            for (int i = 0; i < 16; ++i)
                if (cb + i < nc) op[i] = Os[t * MO_LD + cb + i] * to_o;
        }
    }
    if (cg == 0 && tid == 0 && (p + 1) * piece >= len) pool_m[(size_t)state_out[seg] * H + h] = (float)m_last;
}

static int mb_key_steps(int dk) { return (dk + 31) / 32; }

long ml_chunks_bf16_ws(int dk, int dv) { return (long)((dv + 15) / 16) * 16 * 32 * mb_key_steps(dk) + 32 * mb_key_steps(dk) + 6; }

int ml_chunks_bf16(const MlLaunch& l, hipStream_t stream) {
    const int KS = mb_key_steps(l.dk), CT = (l.dv + 15) / 16, groups = (CT + MW - 1) / MW, slots = l.T / l.piece + l.R;
    const size_t sh = (size_t)slots * l.H;
    float4* ws_s = (float4*)l.ws;
    float* ws_n = (float*)(ws_s + sh * CT * 2 * KS * 64);
    double* ws_m = (double*)(ws_n + sh * 32 * KS);
    double2* ws_g = (double2*)(ws_m + (3 * sh + 1) / 2 * 2);
    const dim3 grid(l.H * groups, slots);
    // 1: q and k in pieces of eight, 2: v, 4: gate, weight and result
    const int vec = (l.dk % 8 == 0 ? 1 : 0) | (l.dv % 8 == 0 && (2 * l.H * l.dk) % 8 == 0 ? 2 : 0)
                    | (l.dv % 8 == 0 && l.rows.g_off % 8 == 0 && l.y_stride % 8 == 0 && l.y_dt == ILM_DTYPE_BF16 && l.rows.w_dt == ILM_DTYPE_BF16
                       && (((uintptr_t)l.y | (uintptr_t)l.rows.norm_w) & 15) == 0 ? 4 : 0);
#define MB_CASE(KS_)                                                                                                                      \
    case KS_:                                                                                                                             \
        mlstm_states_mfma_kernel<KS_><<<grid, MW * 64, 0, stream>>>(ws_s, ws_n, ws_m, ws_g, l.rows, l.seg_offsets, l.R, l.H, l.dk, l.dv, CT,  \
                                                                    l.piece, l.min_len, vec);                                             \
        ILM_LAUNCH_CHECK("mlstm_chunks (states)");                                                                                        \
        if (ml_combine(2 * KS_, ws_s, ws_n, ws_m, l.pool, l.pool_m, l.state_in, l.state_out, l.seg_offsets, l.R, l.H, l.dk, l.dv, CT, l.piece,  \
                       l.min_len, stream)) return -1;                                                                                     \
        if (l.y != nullptr)                                                                                                               \
            mlstm_outputs_mfma_kernel<KS_, true><<<grid, MW * 64, 0, stream>>>(nullptr, l.y, ws_s, ws_n, ws_m, ws_g, l.rows, l.pool_m, l.state_out, \
                                                                               l.seg_offsets, l.R, l.H, l.dk, l.dv, CT, l.piece, l.min_len,   \
                                                                               l.y_stride, l.y_dt, vec);                                  \
        else                                                                                                                              \
            mlstm_outputs_mfma_kernel<KS_, false><<<grid, MW * 64, 0, stream>>>((float*)l.o, nullptr, ws_s, ws_n, ws_m, ws_g, l.rows, l.pool_m, \
                                                                                l.state_out, l.seg_offsets, l.R, l.H, l.dk, l.dv, CT, l.piece,  \
                                                                                l.min_len, l.y_stride, l.y_dt, vec);                      \
        break
    switch (KS) {
        MB_CASE(1); MB_CASE(2); MB_CASE(3); MB_CASE(4);
        default: ILM_REQUIRE(false, "mlstm_chunks: keys of %d", l.dk);
    }
#undef MB_CASE
    ILM_LAUNCH_CHECK("mlstm_chunks (outputs)");
    return 0;
}
