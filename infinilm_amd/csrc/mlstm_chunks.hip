// The mLSTM recurrence (mlstm.hip) over long segments.
//
//   ilm_mlstm_chunks   long segments (portions of prompts).  With L_t the sum of the log forget gates from a fixed start,
//       a_j = li_j - L_j and M_t = max(m_start, max_{j <= t} a_j), m_t = L_t + M_t, and token j has at token t the weight exp(a_j - M_t), the state at
//       the start exp(m_start - M_t): differences that never exceed zero.  They are taken in double, so that a weight keeps its float precision
//       however much has been forgotten in between.  A segment is cut into pieces, a piece into chunks of MC = 64 tokens:
//         states    for every piece and head side by side: what its tokens alone would leave behind, S' = sum_j exp(a_j - M) k_j v_j^T
//         combine   element by element along a segment's pieces: the state each piece starts from, and the segment's last state
//         outputs   for every piece and head side by side: chunk by chunk o = exp(m_s - M) q S_s + sum_j exp(a_j - M) (k_j . q) v_j,
//                   the chunk's sums on the matrix cores, and the state carried on to the piece's next chunk.
//       Piece p of segment r has the workspace slot floor(first row of r / piece) + r + p.
//
// Here on the float matrix instruction (v_mfma_f32_16x16x4_f32: IEEE float products and sums): float rows, and keys above 128.
// bfloat16 rows with keys up to 128 take the kernels of mlstm_mfma.hip.
#include "mlstm.h"

typedef __attribute__((ext_vector_type(4))) float f32x4;

// ---- long segments in pieces ------------------------------------------------------------------------------------------------
__device__ __forceinline__ f32x4 ml_mfma(float x, float y, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(x, y, c, 0, 0, 0); }
// D += A[16 x 16] B[16 x 16]: lane (r, q) brings A[r][4q .. 4q + 3] and holds B and D as rows 4q .. 4q + 3 of column r
__device__ __forceinline__ f32x4 ml_mma(const float4& x, const f32x4& b, f32x4 c) {
    c = ml_mfma(x.x, b[0], c);
    c = ml_mfma(x.y, b[1], c);
    c = ml_mfma(x.z, b[2], c);
    return ml_mfma(x.w, b[3], c);
}
// D += A[16 x 16] B^T: both sides as rows, lane (r, q) brings A[r][4q ..] and B[r][4q ..]
__device__ __forceinline__ f32x4 ml_mmt(const float4& x, const float4& b, f32x4 c) {
    c = ml_mfma(x.x, b.x, c);
    c = ml_mfma(x.y, b.y, c);
    c = ml_mfma(x.z, b.z, c);
    return ml_mfma(x.w, b.w, c);
}

// A chunk's gates, made by one wave (lane t = token t of the chunk, n tokens exist): L and M carried on, a_t, M_t and what follows from them.
struct MlChunk {
    double a[MC], M[MC];
    float start[MC];       // exp(M before the chunk - M_t)
    float floor_[MC];      // exp(-m_t)
    float put[MC];         // exp(a_t - M at the chunk's end)
    float keep;            // exp(M before the chunk - M at its end)
};

template <typename T, bool OUT>
__device__ __forceinline__ void ml_chunk_gates(const MlRows& rows, int t0, int n, int h, int lane, double& L, double& M, MlChunk& c) {
    float li = 0.f, lf = 0.f;
    ml_gates<T>(rows, (size_t)t0 + (lane < n ? lane : n - 1), h, li, lf);
    double Lt = lane < n ? (double)lf : 0.0;
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
        const double up = __shfl_up(Lt, off, 64);
        if (lane >= off) Lt += up;
    }
    Lt += L;
    const double at = lane < n ? (double)li - Lt : -INFINITY;
    double Mt = at;
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
        const double up = __shfl_up(Mt, off, 64);
        if (lane >= off) Mt = fmax(Mt, up);
    }
    Mt = fmax(Mt, M);
    const double Mend = __shfl(Mt, 63, 64), Lend = __shfl(Lt, 63, 64);
    c.put[lane] = lane < n ? expf((float)(at - Mend)) : 0.f;
    if (OUT) {
        c.a[lane] = at;
        c.M[lane] = Mt;
        c.start[lane] = expf((float)(M - Mt));
        c.floor_[lane] = expf(-(float)(Lt + Mt));
    }
    if (lane == 0) c.keep = expf((float)(M - Mend));
    M = Mend;
    L = Lend;
}

// rows of MC tokens, KT * 16 entries a token filled up with zeros, from dk columns at `col`, as floats with a stride of LDS_ floats
template <typename T, int KT>
__device__ __forceinline__ void ml_stage(float* __restrict__ dst, const T* __restrict__ rows, size_t stride, int n, int dk) {
    constexpr int DK = KT * 16, LD = DK + 4;
    const bool v4 = dk % 4 == 0;
    for (int i = threadIdx.x; i < MC * (DK / 4); i += MW * 64) {
        const int t = i / (DK / 4), c = (i % (DK / 4)) * 4;
        float v[4] = {0.f, 0.f, 0.f, 0.f};
        if (t < n) {
            const T* at = rows + (size_t)t * stride + c;
            if (v4) {
                if (c < dk) ml_ld4(at, v);
            } else {
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    if (c + e < dk) v[e] = ml_ld(at + e);
            }
        }
        *reinterpret_cast<float4*>(&dst[t * LD + c]) = make_float4(v[0], v[1], v[2], v[3]);
    }
}

// a wave's 16 columns of v of a chunk: rows 16 j + 4 q + e of column r
template <typename T>
__device__ __forceinline__ void ml_values(f32x4 (&v)[4], const T* __restrict__ rows, size_t stride, int n, int col, int dv, int q) {
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int t = 16 * j + 4 * q + e;
            const float x = ml_ld(rows + (size_t)(t < n ? t : n - 1) * stride + (col < dv ? col : dv - 1));
            v[j][e] = (t < n && col < dv) ? x : 0.f;
        }
}

// the state's tiles carried over a chunk: S = keep S + K^T (put V)
template <int KT>
__device__ __forceinline__ void ml_carry(f32x4 (&S)[KT], const float* __restrict__ Ks, const f32x4 (&v)[4], const MlChunk& c, int r, int q) {
    constexpr int LD = KT * 16 + 4;
    f32x4 w[4];
    const float keep = c.keep;
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int e = 0; e < 4; ++e) w[j][e] = v[j][e] * c.put[16 * j + 4 * q + e];
#pragma unroll
    for (int m = 0; m < KT; ++m) {
        f32x4 s = S[m] * keep;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            float4 k;
            k.x = Ks[(16 * j + 4 * q) * LD + 16 * m + r];
            k.y = Ks[(16 * j + 4 * q + 1) * LD + 16 * m + r];
            k.z = Ks[(16 * j + 4 * q + 2) * LD + 16 * m + r];
            k.w = Ks[(16 * j + 4 * q + 3) * LD + 16 * m + r];
            s = ml_mma(k, w[j], s);
        }
        S[m] = s;
    }
}

// n, a part of the tokens a thread: thread (part, d) adds the tokens of its part to entry d
template <int KT>
struct MlN {
    static constexpr int WIDTH = KT <= 8 ? 128 : 256, PARTS = MW * 64 / WIDTH, TOKENS = MC / PARTS;
};
template <int KT>
__device__ __forceinline__ float ml_carry_n(float n, const float* __restrict__ Ks, const MlChunk& c) {
    constexpr int LD = KT * 16 + 4;
    const int d = threadIdx.x % MlN<KT>::WIDTH, part = threadIdx.x / MlN<KT>::WIDTH;
    if (d >= KT * 16) return 0.f;
    n *= c.keep;
#pragma unroll 8
    for (int i = 0; i < MlN<KT>::TOKENS; ++i) {
        const int t = part * MlN<KT>::TOKENS + i;
        n = fmaf(Ks[t * LD + d], c.put[t], n);
    }
    return n;
}

// workspace: state tiles [slot, H, columns / 16, KT, 64] float4 | n [slot, H, DK] float | (L, M, m at the start) [slot, H, 3] double
template <typename T, int KT>
__global__ void __launch_bounds__(MW * 64, 2)
mlstm_states_kernel(float4* __restrict__ ws_s, float* __restrict__ ws_n, double* __restrict__ ws_m, MlRows a, const int* __restrict__ seg_offsets,
                    int R, int H, int dk, int dv, int CT, int piece, int min_len) {
    constexpr int DK = KT * 16, LD = DK + 4;
    __shared__ __attribute__((aligned(16))) float Ks[MC * LD];
    __shared__ MlChunk ch;
    __shared__ float nred[MlN<KT>::PARTS][MlN<KT>::WIDTH];
    const int h = blockIdx.x % H, cg = blockIdx.x / H, slot = blockIdx.y;
    int p;
    const int seg = ml_find(seg_offsets, R, piece, slot, p);
    if (seg < 0) return;
    const int len = seg_offsets[seg + 1] - seg_offsets[seg];
    if (len < min_len) return;                         // (the step kernel's)
    const int p0 = seg_offsets[seg] + p * piece, plen = min(piece, len - p * piece);
    const int lane = threadIdx.x & 63, r = lane & 15, q = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int ct = cg * MW + wave, col = 16 * ct + r;
    const T* base = (const T*)a.rows;
    f32x4 S[KT];
#pragma unroll
    for (int m = 0; m < KT; ++m) S[m] = f32x4{0.f, 0.f, 0.f, 0.f};
    float n = 0.f;
    double L = 0.0, M = -INFINITY;
    for (int c0 = 0; c0 < plen; c0 += MC) {
        const int t0 = p0 + c0, cn = min(MC, plen - c0);
        const T* row = base + (size_t)t0 * a.stride;
        f32x4 v[4];
        ml_values<T>(v, row + (size_t)2 * H * dk + (size_t)h * dv, a.stride, cn, col, dv, q);
        __syncthreads();                               // the last chunk's readers are done
        ml_stage<T, KT>(Ks, row + (size_t)(H + h) * dk, a.stride, cn, dk);
        if (wave == 0) ml_chunk_gates<T, false>(a, t0, cn, h, lane, L, M, ch);
        __syncthreads();
        if (ct < CT) ml_carry<KT>(S, Ks, v, ch, r, q);
        if (cg == 0) n = ml_carry_n<KT>(n, Ks, ch);
    }
    const size_t sh = (size_t)slot * H + h;
    if (ct < CT) {
#pragma unroll
        for (int m = 0; m < KT; ++m) ws_s[((sh * CT + ct) * KT + m) * 64 + lane] = make_float4(S[m][0], S[m][1], S[m][2], S[m][3]);
    }
    if (cg != 0) return;                               // (a whole block)
    const int d = threadIdx.x % MlN<KT>::WIDTH;
    nred[threadIdx.x / MlN<KT>::WIDTH][d] = n;
    __syncthreads();
    if (threadIdx.x < DK) {
        float sum = 0.f;
#pragma unroll
        for (int i = 0; i < MlN<KT>::PARTS; ++i) sum += nred[i][threadIdx.x];
        ws_n[sh * DK + threadIdx.x] = sum;
    }
    if (threadIdx.x == 0) {
        ws_m[sh * 3] = L;
        ws_m[sh * 3 + 1] = M;
    }
}

// Along a segment's pieces, four elements a thread: the state before each piece in the place of what the piece leaves behind, and the
// segment's last state into the pool.  Items: the state's tiles as they lie in the workspace, then n.
__global__ void __launch_bounds__(256)
mlstm_combine_kernel(float4* __restrict__ ws_s, float* __restrict__ ws_n, double* __restrict__ ws_m, float* __restrict__ pool,
                     const float* __restrict__ pool_m, const int* __restrict__ state_in, const int* __restrict__ state_out,
                     const int* __restrict__ seg_offsets, int KT, int H, int dk, int dv, int CT, int piece, int min_len) {
    const int DK = KT * 16;
    const int h = blockIdx.y, seg = blockIdx.z;
    const int s0 = seg_offsets[seg], len = seg_offsets[seg + 1] - s0;
    if (len <= 0 || len < min_len) return;
    const int item = blockIdx.x * 256 + threadIdx.x, tiles = CT * KT * 64;
    if (item >= tiles + DK / 4) return;
    const bool is_n = item >= tiles;
    int k0, col;
    if (is_n) {
        k0 = (item - tiles) * 4;
        col = dv;
    } else {
        const int ln = item & 63, m = (item >> 6) % KT, ct = (item >> 6) / KT;
        k0 = 16 * m + 4 * (ln >> 4);
        col = 16 * ct + (ln & 15);
    }
    const size_t hs = (size_t)dk * (dv + 1);
    const bool in = k0 < dk && (is_n || col < dv), v4 = dk % 4 == 0;
    const float* src = pool + ((size_t)state_in[seg] * H + h) * hs + (size_t)(in ? col : 0) * dk + (in ? k0 : 0);
    float s[4] = {0.f, 0.f, 0.f, 0.f};
    if (in) {
        if (v4) ml_ld4(src, s);
        else
#pragma unroll
            for (int e = 0; e < 4; ++e) s[e] = k0 + e < dk ? src[e] : 0.f;
    }
    double m = (double)pool_m[(size_t)state_in[seg] * H + h];
    const int pieces = (len + piece - 1) / piece;
    const size_t slot0 = (size_t)(s0 / piece + seg);
    const size_t step = (size_t)H * (is_n ? (size_t)(DK / 4) : (size_t)tiles);
    float4* at = is_n ? reinterpret_cast<float4*>(ws_n) + (slot0 * H + h) * (DK / 4) + (item - tiles) : ws_s + (slot0 * H + h) * tiles + item;
    const bool notes = is_n && k0 == 0;                // one thread a head also leaves m at every piece's start
    constexpr int AHEAD = 4;
    float4 nxt[AHEAD];
    double nl[AHEAD], nm[AHEAD];
    auto fetch = [&](int p, int i) {
        const int pc = p < pieces ? p : pieces - 1;
        nxt[i] = at[(size_t)pc * step];
        const double* wm = ws_m + ((slot0 + pc) * H + h) * 3;
        nl[i] = wm[0];
        nm[i] = wm[1];
    };
#pragma unroll
    for (int i = 0; i < AHEAD; ++i) fetch(i, i);
    for (int p0 = 0; p0 < pieces; p0 += AHEAD) {
        float4 cur[AHEAD];
        double cl[AHEAD], cm[AHEAD];
#pragma unroll
        for (int i = 0; i < AHEAD; ++i) { cur[i] = nxt[i]; cl[i] = nl[i]; cm[i] = nm[i]; }
        if (p0 + AHEAD < pieces) {
#pragma unroll
            for (int i = 0; i < AHEAD; ++i) fetch(p0 + AHEAD + i, i);
        }
#pragma unroll
        for (int i = 0; i < AHEAD; ++i) {
            const int p = p0 + i;
            if (p >= pieces) break;
            at[(size_t)p * step] = make_float4(s[0], s[1], s[2], s[3]);
            if (notes) ws_m[((slot0 + p) * H + h) * 3 + 2] = m;
            const double M = fmax(m, cm[i]);
            const float x = expf((float)(m - M)), z = expf((float)(cm[i] - M));
            s[0] = fmaf(z, cur[i].x, x * s[0]);
            s[1] = fmaf(z, cur[i].y, x * s[1]);
            s[2] = fmaf(z, cur[i].z, x * s[2]);
            s[3] = fmaf(z, cur[i].w, x * s[3]);
            m = cl[i] + M;
        }
    }
    if (!in) return;
    float* dst = pool + ((size_t)state_out[seg] * H + h) * hs + (size_t)col * dk + k0;
    if (v4) *reinterpret_cast<float4*>(dst) = make_float4(s[0], s[1], s[2], s[3]);
    else
#pragma unroll
        for (int e = 0; e < 4; ++e)
            if (k0 + e < dk) dst[e] = s[e];
}

int ml_combine(int KT, float4* ws_s, float* ws_n, double* ws_m, float* pool, const float* pool_m, const int* state_in, const int* state_out,
               const int* seg_offsets, int R, int H, int dk, int dv, int CT, int piece, int min_len, hipStream_t stream) {
    const dim3 grid((CT * KT * 64 + KT * 4 + 255) / 256, H, R);
    mlstm_combine_kernel<<<grid, 256, 0, stream>>>(ws_s, ws_n, ws_m, pool, pool_m, state_in, state_out, seg_offsets, KT, H, dk, dv, CT, piece, min_len);
    ILM_LAUNCH_CHECK("mlstm_chunks (combine)");
    return 0;
}

// NORM: a block holds all columns of the head and ends with the output norm, weight and gate
template <typename T, int KT, bool NORM>
__global__ void __launch_bounds__(MW * 64, 2)
mlstm_outputs_kernel(float* __restrict__ out, void* __restrict__ y, const float4* __restrict__ ws_s, const float* __restrict__ ws_n,
                     const double* __restrict__ ws_m, MlRows a, float* __restrict__ pool_m, const int* __restrict__ state_out,
                     const int* __restrict__ seg_offsets, int R, int H, int dk, int dv, int CT, int piece, int min_len, int y_stride, int y_dt) {
    constexpr int DK = KT * 16, LD = DK + 4, NP = MlN<KT>::PARTS, NW = MlN<KT>::WIDTH;
    __shared__ __attribute__((aligned(16))) float Ks[MC * LD];
    __shared__ __attribute__((aligned(16))) float Qs[MC * LD];
    __shared__ float4 Ps[10][64];                      // tiles (rt, ct), ct <= rt, of the second sum's weights as operands
    __shared__ MlChunk ch;
    __shared__ float nred[NP][NW];
    __shared__ float rs[4][MC];                        // the weights' sums by column tile
    __shared__ float nq[MC], to_o[MC], sq[MW][MC], rstd[MC];
    const int h = blockIdx.x % H, cg = blockIdx.x / H, slot = blockIdx.y;
    int p;
    const int seg = ml_find(seg_offsets, R, piece, slot, p);
    if (seg < 0) return;
    const int len = seg_offsets[seg + 1] - seg_offsets[seg];
    if (len < min_len) return;
    const int p0 = seg_offsets[seg] + p * piece, plen = min(piece, len - p * piece);
    const int tid = threadIdx.x, lane = tid & 63, r = lane & 15, q = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int ct = cg * MW + wave, col = 16 * ct + r;
    const bool col_ok = col < dv;
    const T* base = (const T*)a.rows;
    const size_t sh = (size_t)slot * H + h;
    f32x4 S[KT];
#pragma unroll
    for (int m = 0; m < KT; ++m) {
        const float4 t = ws_s[((sh * CT + (ct < CT ? ct : 0)) * KT + m) * 64 + lane];
        S[m] = f32x4{t.x, t.y, t.z, t.w};
    }
    const int nd = tid % NW;
    float n = tid < NW && nd < DK ? ws_n[sh * DK + nd] : 0.f;      // (part 0 starts from the whole, the others from nothing)
    double L = 0.0, M = ws_m[sh * 3 + 2];
    for (int c0 = 0; c0 < plen; c0 += MC) {
        const int t0 = p0 + c0, cn = min(MC, plen - c0);
        const T* row = base + (size_t)t0 * a.stride;
        f32x4 v[4];
        ml_values<T>(v, row + (size_t)2 * H * dk + (size_t)h * dv, a.stride, cn, col, dv, q);
        __syncthreads();                               // the last chunk's readers are done
        ml_stage<T, KT>(Qs, row + (size_t)h * dk, a.stride, cn, dk);
        ml_stage<T, KT>(Ks, row + (size_t)(H + h) * dk, a.stride, cn, dk);
        nred[tid / NW][nd] = n;
        if (wave == 0) ml_chunk_gates<T, true>(a, t0, cn, h, lane, L, M, ch);
        __syncthreads();
        // ---- weights exp(a_i - M_t) (k_i . q_t) as [i, t], by tiles at and below the diagonal, and their sums over i
        for (int tile = wave; tile < 10; tile += MW) {
            const int rt = tile < 1 ? 0 : (tile < 3 ? 1 : (tile < 6 ? 2 : 3)), kt = tile - rt * (rt + 1) / 2;
            f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int j = 0; j < KT; ++j)
                acc = ml_mmt(*reinterpret_cast<const float4*>(&Ks[(16 * kt + r) * LD + 16 * j + 4 * q]),
                             *reinterpret_cast<const float4*>(&Qs[(16 * rt + r) * LD + 16 * j + 4 * q]), acc);
            const double Mt = ch.M[16 * rt + r];
            float4 w;
            float* we = reinterpret_cast<float*>(&w);
            float sum = 0.f;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int i = 16 * kt + 4 * q + e;
                we[e] = i <= 16 * rt + r ? expf((float)(ch.a[i] - Mt)) * acc[e] : 0.f;
                sum += we[e];
            }
            sum += __shfl_xor(sum, 16, 64);
            sum += __shfl_xor(sum, 32, 64);
            if (q == 0) rs[kt][16 * rt + r] = sum;
            Ps[tile][lane] = w;
        }
        {   // n . q_t before the chunk, eight lanes a token
            const int t = tid >> 3, part = tid & 7;
            float s = 0.f;
            for (int d = part; d < DK; d += 8) {
                float nn = nred[0][d];
#pragma unroll
                for (int i = 1; i < NP; ++i) nn += nred[i][d];
                s = fmaf(nn, Qs[t * LD + d], s);
            }
            s += __shfl_xor(s, 1, 64);
            s += __shfl_xor(s, 2, 64);
            s += __shfl_xor(s, 4, 64);
            if (part == 0) nq[t] = s;
        }
        __syncthreads();
        if (tid < MC) {
            float d = ch.start[tid] * nq[tid];
            for (int j = 0; j <= tid / 16; ++j) d += rs[j][tid];
            to_o[tid] = a.scale / (fmaxf(fabsf(d * a.scale), ch.floor_[tid]) + 1e-6f);
        }
        // ---- exp(m_s - M_t) q S + P V
        f32x4 x[4];
#pragma unroll
        for (int rt = 0; rt < 4; ++rt) {
            f32x4 b0 = f32x4{0.f, 0.f, 0.f, 0.f}, b1 = b0;
#pragma unroll
            for (int m = 0; m < KT; ++m) {
                const float4 qa = *reinterpret_cast<const float4*>(&Qs[(16 * rt + r) * LD + 16 * m + 4 * q]);
                if (m & 1) b1 = ml_mma(qa, S[m], b1);
                else b0 = ml_mma(qa, S[m], b0);
            }
            b0 = b0 + b1;
#pragma unroll
            for (int e = 0; e < 4; ++e) b0[e] *= ch.start[16 * rt + 4 * q + e];
#pragma unroll
            for (int j = 0; j <= rt; ++j) b0 = ml_mma(Ps[rt * (rt + 1) / 2 + j][lane], v[j], b0);
            x[rt] = b0;
        }
        __syncthreads();
        if (NORM) {
            float g[4][4];
            const T* grow = row + a.g_off + (size_t)h * dv + (col_ok ? col : 0);
#pragma unroll
            for (int rt = 0; rt < 4; ++rt)
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const int t = 16 * rt + 4 * q + e;
                    g[rt][e] = ml_ld(grow + (size_t)(t < cn ? t : cn - 1) * a.stride);
                }
#pragma unroll
            for (int rt = 0; rt < 4; ++rt)
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const float ov = x[rt][e] * to_o[16 * rt + 4 * q + e];
                    x[rt][e] = ov;
                    float s = col_ok ? ov * ov : 0.f;
                    s += __shfl_xor(s, 1, 64);
                    s += __shfl_xor(s, 2, 64);
                    s += __shfl_xor(s, 4, 64);
                    s += __shfl_xor(s, 8, 64);
                    if (r == 0) sq[wave][16 * rt + 4 * q + e] = s;
                }
            __syncthreads();
            if (tid < MC) {
                float s = 0.f;
#pragma unroll
                for (int i = 0; i < MW; ++i) s += sq[i][tid];
                rstd[tid] = 1.0f / sqrtf(s / (float)dv + a.eps);
            }
            __syncthreads();
            if (col_ok) {
                const int j = h * dv + col;
                const float w = ml_any(a.norm_w, a.w_dt, j);
#pragma unroll
                for (int rt = 0; rt < 4; ++rt)
#pragma unroll
                    for (int e = 0; e < 4; ++e) {
                        const int t = 16 * rt + 4 * q + e;
                        if (t < cn) {
                            const float z = x[rt][e] * rstd[t] * w * ml_sigmoid(g[rt][e]);
                            if (y_dt == ILM_DTYPE_F32) ((float*)y)[(size_t)(t0 + t) * y_stride + j] = z;
                            else ((bf16*)y)[(size_t)(t0 + t) * y_stride + j] = from_f32<bf16>(z);
                        }
                    }
            }
        } else if (col_ok) {
#pragma unroll
            for (int rt = 0; rt < 4; ++rt)
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const int t = 16 * rt + 4 * q + e;
                    if (t < cn) out[((size_t)(t0 + t) * H + h) * dv + col] = x[rt][e] * to_o[t];
                }
        }
        if (c0 + MC < plen) {
            ml_carry<KT>(S, Ks, v, ch, r, q);
            n = ml_carry_n<KT>(n, Ks, ch);
        }
    }
    if (cg == 0 && tid == 0 && (p + 1) * piece >= len) pool_m[(size_t)state_out[seg] * H + h] = (float)(L + M);
}

#define ML_MAX_KT 16
static int ml_key_tiles(int dk) {      // (sizes above 128 in two steps)
    const int kt = (dk + 15) / 16;
    return kt <= 8 ? kt : (kt <= 12 ? 12 : 16);
}
static bool ml_on_bf16(int rows_dt, int dk) { return rows_dt == ILM_DTYPE_BF16 && dk <= 128; }
extern "C" int ilm_mlstm_chunk() { return MC; }
extern "C" int ilm_mlstm_chunk_max_dk() { return 16 * ML_MAX_KT; }
extern "C" int ilm_mlstm_chunk_cols() { return MCOLS; }
// floats of workspace a (slot, head) takes; four more are needed a (token, head)
extern "C" int ilm_mlstm_chunk_ws(int dk, int dv, int rows_dt) {
    if (ml_on_bf16(rows_dt, dk)) return (int)ml_chunks_bf16_ws(dk, dv);
    const int DK = ml_key_tiles(dk) * 16, CT = (dv + 15) / 16;
    return CT * 16 * DK + DK + 6;
}

// Segments of at least min_len tokens; the others are passed over.  piece: a multiple of 64; ws: (T / piece + R) * H *
// ilm_mlstm_chunk_ws floats and 4 * T * H more.  y != null: with the output norm (dv <= ilm_mlstm_chunk_cols()); else o [T, H dv] float.
extern "C" int ilm_mlstm_chunks(void* o, void* y, const void* rows, int row_stride, int rows_dt, const void* bias_i, const void* bias_f, int b_dt,
                                int i_off, int f_off, int g_off, float cap, float scale, void* pool, void* pool_m, const void* state_in,
                                const void* state_out, const void* seg_offsets, int R, int H, int dk, int dv, int T_, int min_len, int piece,
                                const void* norm_w, int w_dt, float eps, int y_stride, int y_dt, void* ws, hipStream_t stream) {
    ML_CHECK_ROWS("mlstm_chunks");
    ILM_REQUIRE(T_ > 0 && dk <= 16 * ML_MAX_KT && piece > 0 && piece % MC == 0, "mlstm_chunks: keys of %d (at most %d), pieces of %d", dk,
                16 * ML_MAX_KT, piece);
    ILM_REQUIRE((y != nullptr) != (o != nullptr) && (y == nullptr || dv <= MCOLS), "mlstm_chunks: one kind of result, a norm over at most %d columns", MCOLS);
    const int slots = T_ / piece + R, CT = (dv + 15) / 16, groups = (CT + MW - 1) / MW;
    ILM_REQUIRE(slots <= 65535 && ws != nullptr && ((uintptr_t)ws & 15) == 0, "mlstm_chunks: %d pieces in a step, at most 65535", slots);
    if (ml_on_bf16(rows_dt, dk)) {
        const MlLaunch l = {o, y, a, (float*)pool, (float*)pool_m, (const int*)state_in, (const int*)state_out, (const int*)seg_offsets, R, H, dk, dv,
                            T_, min_len, piece, y_stride, y_dt, ws};
        return ml_chunks_bf16(l, stream);
    }
    const int KT = ml_key_tiles(dk);
    const size_t sh = (size_t)slots * H;
    float4* ws_s = (float4*)ws;
    float* ws_n = (float*)(ws_s + sh * CT * KT * 64);
    double* ws_m = (double*)(ws_n + sh * KT * 16);
    const dim3 grid(H * groups, slots);
#define MLC_T(T__, KT_)                                                                                                                   \
    {                                                                                                                                     \
        mlstm_states_kernel<T__, KT_><<<grid, MW * 64, 0, stream>>>(ws_s, ws_n, ws_m, a, (const int*)seg_offsets, R, H, dk, dv, CT, piece, min_len); \
        ILM_LAUNCH_CHECK("mlstm_chunks (states)");                                                                                        \
        if (ml_combine(KT_, ws_s, ws_n, ws_m, (float*)pool, (const float*)pool_m, (const int*)state_in, (const int*)state_out,              \
                       (const int*)seg_offsets, R, H, dk, dv, CT, piece, min_len, stream)) return -1;                                       \
        if (y != nullptr)                                                                                                                 \
            mlstm_outputs_kernel<T__, KT_, true><<<grid, MW * 64, 0, stream>>>(nullptr, y, ws_s, ws_n, ws_m, a, (float*)pool_m, (const int*)state_out, \
                                                                               (const int*)seg_offsets, R, H, dk, dv, CT, piece, min_len, y_stride, y_dt); \
        else                                                                                                                              \
            mlstm_outputs_kernel<T__, KT_, false><<<grid, MW * 64, 0, stream>>>((float*)o, nullptr, ws_s, ws_n, ws_m, a, (float*)pool_m,     \
                                                                                (const int*)state_out, (const int*)seg_offsets, R, H, dk, dv, CT,  \
                                                                                piece, min_len, y_stride, y_dt);                           \
    }
#define MLC_CASE(KT_)             \
    case KT_:                     \
        MLC_T(float, KT_)         \
        break
#define MLC_BOTH(KT_)                                                                 \
    case KT_:                                                                         \
        if (rows_dt == ILM_DTYPE_F32) MLC_T(float, KT_) else MLC_T(bf16, KT_)          \
        break
    switch (KT) {
        MLC_CASE(1); MLC_CASE(2); MLC_CASE(3); MLC_CASE(4); MLC_CASE(5); MLC_CASE(6); MLC_CASE(7); MLC_CASE(8);
        MLC_BOTH(12); MLC_BOTH(16);
        default: ILM_REQUIRE(false, "mlstm_chunks: keys of %d", dk);
    }
#undef MLC_BOTH
#undef MLC_CASE
#undef MLC_T
    ILM_LAUNCH_CHECK("mlstm_chunks (outputs)");
    return 0;
}
