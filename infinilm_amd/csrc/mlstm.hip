// The matrix memory of an mLSTM: a linear attention whose state is written and forgotten through exponential gates, kept in
// range by a running maximum, and read through a denominator.  Per head, with the vectors of token t as rows and its log gates
//
//   li = cap tanh((raw_i + b_i) / cap),     lf = log sigmoid(cap tanh((raw_f + b_f) / cap))
//   m_t = max(lf + m_{t-1}, li)             (m_0 = 0)
//   S_t = exp(lf + m_{t-1} - m_t) S_{t-1} + exp(li - m_t) outer(k_t, v_t),      n_t likewise with k_t alone
//   o_t = q_t S_t / (max(|n_t . q_t|, exp(-m_t)) + 1e-6),                       q_t scaled by dk^(-1/2)
//
// and, where a block holds all columns of a head, y_t = o_t / sqrt(mean(o_t^2) + eps) * w * sigmoid(gate) in the activations'
// dtype.  Everything but the rows themselves is float.  Rows are those of one fused projection, [q: H dk | k: H dk | v: H dv | ...]
// with the raw gates and the output gate at offsets of their own.
//
// A request's state passes from step to step through rows of two pools, [H, dv + 1, dk] (the key index fastest; row dv is n) and
// [H] (m).
//
//   ilm_mlstm_step     token by token, a block a (request, head, columns).  A thread keeps ML_NK state entries of VC columns in
//       registers; n is one column more, whose value is 1, so that n . q comes out of the same sums.
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
#include "common.h"

typedef __attribute__((ext_vector_type(4))) float f32x4;

#define ML_NK 8

__device__ __forceinline__ float ml_ld(const float* p) { return *p; }
__device__ __forceinline__ float ml_ld(const bf16* p) { return to_f32(*p); }
__device__ __forceinline__ void ml_ld4(const float* p, float* v) {
    const float4 t = *reinterpret_cast<const float4*>(p);
    v[0] = t.x; v[1] = t.y; v[2] = t.z; v[3] = t.w;
}
__device__ __forceinline__ void ml_ld4(const bf16* p, float* v) {
    const uint2 t = *reinterpret_cast<const uint2*>(p);
    v[0] = __uint_as_float(t.x << 16); v[1] = __uint_as_float(t.x & 0xffff0000u);
    v[2] = __uint_as_float(t.y << 16); v[3] = __uint_as_float(t.y & 0xffff0000u);
}
__device__ __forceinline__ float ml_any(const void* p, int dt, size_t i) {
    return dt == ILM_DTYPE_F32 ? ((const float*)p)[i] : to_f32(((const bf16*)p)[i]);
}
__device__ __forceinline__ float ml_capped(float z, float cap) { return cap * tanhf(z / cap); }
__device__ __forceinline__ float ml_log_sigmoid(float z) { return -(log1pf(expf(-fabsf(z))) + fmaxf(-z, 0.f)); }
__device__ __forceinline__ float ml_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }

// what a launch knows of its rows
struct MlRows {
    const void* rows;       // [T, stride]
    const void *bias_i, *bias_f;
    const void *norm_w;     // [H dv]
    long stride;
    int i_off, f_off, g_off;    // columns of the raw gates and of the output gate
    int b_dt, w_dt;
    float cap, scale, eps;
};

template <typename T>
__device__ __forceinline__ void ml_gates(const MlRows& a, size_t t, int h, float& li, float& lf) {
    const T* row = (const T*)a.rows + t * a.stride;
    li = ml_capped(ml_ld(row + a.i_off + h) + ml_any(a.bias_i, a.b_dt, h), a.cap);
    lf = ml_log_sigmoid(ml_capped(ml_ld(row + a.f_off + h) + ml_any(a.bias_f, a.b_dt, h), a.cap));
}

// The columns of a block: slots 0 .. CB - 2 are columns of v, slot CB - 1 is n (written back only where the block holds the whole head).
template <typename T, int THREADS, int VC, bool NORM>
__global__ void __launch_bounds__(THREADS)
mlstm_step_kernel(float* __restrict__ o, void* __restrict__ y, MlRows a, float* __restrict__ pool, float* __restrict__ pool_m,
                  const int* __restrict__ state_in, const int* __restrict__ state_out, const int* __restrict__ seg_offsets, int H, int dk,
                  int dv, int KP, int max_len, int y_stride, int y_dt) {
    __shared__ float red[THREADS / 64];
    __shared__ float den[2];
    const int h = blockIdx.y, r = blockIdx.z;
    const int t0 = seg_offsets[r], t1 = seg_offsets[r + 1];
    if (t0 >= t1 || t1 - t0 > max_len) return;       // (longer segments are another kernel's)
    const int CB = (THREADS / KP) * VC;
    const int kp = threadIdx.x % KP, slot0 = (threadIdx.x / KP) * VC;
    const size_t hs = (size_t)dk * (dv + 1);
    const float* src = pool + ((size_t)state_in[r] * H + h) * hs;
    float m = pool_m[(size_t)state_in[r] * H + h];
    const bool v4 = dk % 4 == 0;
    // the thread's entries 4 p .. 4 p + 3 are k = kof[p] .. kof[p] + 3
    const int kof[2] = {4 * kp, 4 * (KP + kp)};
    int col[VC];
    float S[VC][ML_NK];
#pragma unroll
    for (int c = 0; c < VC; ++c) {
        const int s = slot0 + c, real = blockIdx.x * (CB - 1) + s;
        col[c] = s == CB - 1 ? dv : (real < dv ? real : -1);
#pragma unroll
        for (int p = 0; p < 2; ++p) {
            const bool ok = col[c] >= 0 && kof[p] < dk;
            const float* at = src + (size_t)(ok ? col[c] : 0) * dk + (ok ? kof[p] : 0);
            if (v4) {
                const float4 t = ok ? *reinterpret_cast<const float4*>(at) : make_float4(0.f, 0.f, 0.f, 0.f);
                S[c][4 * p] = t.x; S[c][4 * p + 1] = t.y; S[c][4 * p + 2] = t.z; S[c][4 * p + 3] = t.w;
            } else {
#pragma unroll
                for (int e = 0; e < 4; ++e) S[c][4 * p + e] = (ok && kof[p] + e < dk) ? at[e] : 0.f;
            }
        }
    }
    const T* base = (const T*)a.rows;
    for (int t = t0; t < t1; ++t) {
        const T* row = base + (size_t)t * a.stride;
        const T* qp = row + (size_t)h * dk;
        const T* kq = qp + (size_t)H * dk;
        const T* vp = row + (size_t)2 * H * dk + (size_t)h * dv;
        float q[ML_NK], k[ML_NK], v[VC];
#pragma unroll
        for (int p = 0; p < 2; ++p) {
            const bool in = kof[p] < dk;
            if (v4) {
                ml_ld4(qp + (in ? kof[p] : 0), q + 4 * p);
                ml_ld4(kq + (in ? kof[p] : 0), k + 4 * p);
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    q[4 * p + e] = in ? q[4 * p + e] : 0.f;
                    k[4 * p + e] = in ? k[4 * p + e] : 0.f;
                }
            } else {
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const bool ok = kof[p] + e < dk;
                    q[4 * p + e] = ok ? ml_ld(qp + kof[p] + e) : 0.f;
                    k[4 * p + e] = ok ? ml_ld(kq + kof[p] + e) : 0.f;
                }
            }
        }
#pragma unroll
        for (int c = 0; c < VC; ++c) v[c] = col[c] == dv ? 1.0f : (col[c] >= 0 ? ml_ld(vp + col[c]) : 0.f);
        float li, lf;
        ml_gates<T>(a, t, h, li, lf);
        const float mn = fmaxf(lf + m, li), keep = expf(lf + m - mn), put = expf(li - mn);
        m = mn;
        float rq[VC];
#pragma unroll
        for (int c = 0; c < VC; ++c) {
            const float pv = put * v[c];
            rq[c] = 0.f;
#pragma unroll
            for (int i = 0; i < ML_NK; ++i) {
                S[c][i] = fmaf(k[i], pv, keep * S[c][i]);
                rq[c] = fmaf(S[c][i], q[i], rq[c]);
            }
        }
        for (int off = 1; off < KP; off <<= 1) {
#pragma unroll
            for (int c = 0; c < VC; ++c) rq[c] += __shfl_xor(rq[c], off, 64);
        }
        if (kp == 0 && slot0 + VC == CB) den[t & 1] = fmaxf(fabsf(rq[VC - 1] * a.scale), expf(-m)) + 1e-6f;
        __syncthreads();
        const float to_o = a.scale / den[t & 1];
        float ov[VC];
#pragma unroll
        for (int c = 0; c < VC; ++c) ov[c] = rq[c] * to_o;
        if constexpr (NORM) {
            float ss = 0.f;
            if (kp == 0) {
#pragma unroll
                for (int c = 0; c < VC; ++c) ss = (col[c] >= 0 && col[c] < dv) ? fmaf(ov[c], ov[c], ss) : ss;
            }
            const float rstd = 1.0f / sqrtf(block_sum<THREADS / 64>(ss, red) / (float)dv + a.eps);
#pragma unroll
            for (int c = 0; c < VC; ++c)
                if (kp == c % KP && col[c] >= 0 && col[c] < dv) {      // (the columns' ends spread over the lanes)
                    const int j = h * dv + col[c];
                    const float z = ov[c] * rstd * ml_any(a.norm_w, a.w_dt, j) * ml_sigmoid(ml_ld(row + a.g_off + j));
                    if (y_dt == ILM_DTYPE_F32) ((float*)y)[(size_t)t * y_stride + j] = z;
                    else ((bf16*)y)[(size_t)t * y_stride + j] = from_f32<bf16>(z);
                }
        } else {
#pragma unroll
            for (int c = 0; c < VC; ++c)
                if (kp == c % KP && col[c] >= 0 && col[c] < dv) o[((size_t)t * H + h) * dv + col[c]] = ov[c];
        }
    }
    const bool whole = gridDim.x == 1;
    float* dst = pool + ((size_t)state_out[r] * H + h) * hs;
#pragma unroll
    for (int c = 0; c < VC; ++c)
        if (col[c] >= 0 && (whole || col[c] < dv)) {
#pragma unroll
            for (int p = 0; p < 2; ++p) {
                float* at = dst + (size_t)col[c] * dk + kof[p];
                if (v4) {
                    if (kof[p] < dk) *reinterpret_cast<float4*>(at) = make_float4(S[c][4 * p], S[c][4 * p + 1], S[c][4 * p + 2], S[c][4 * p + 3]);
                } else {
#pragma unroll
                    for (int e = 0; e < 4; ++e)
                        if (kof[p] + e < dk) at[e] = S[c][4 * p + e];
                }
            }
        }
    if (whole && threadIdx.x == 0) pool_m[(size_t)state_out[r] * H + h] = m;
}

// n and m of the heads whose columns are spread over several blocks of the step kernel (which all read the old ones): a block a
// (head, request), run after it.
template <typename T>
__global__ void __launch_bounds__(256)
mlstm_step_norms_kernel(MlRows a, float* __restrict__ pool, float* __restrict__ pool_m, const int* __restrict__ state_in,
                        const int* __restrict__ state_out, const int* __restrict__ seg_offsets, int H, int dk, int dv, int max_len) {
    const int h = blockIdx.x, r = blockIdx.y;
    const int t0 = seg_offsets[r], t1 = seg_offsets[r + 1];
    if (t0 >= t1 || t1 - t0 > max_len) return;
    const size_t hs = (size_t)dk * (dv + 1);
    const float* src = pool + ((size_t)state_in[r] * H + h) * hs + (size_t)dv * dk;
    float* dst = pool + ((size_t)state_out[r] * H + h) * hs + (size_t)dv * dk;
    const float m0 = pool_m[(size_t)state_in[r] * H + h];
    float m = m0;
    __syncthreads();
    for (int d0 = 0; d0 < dk; d0 += 256) {
        const int d = d0 + threadIdx.x;
        float n = d < dk ? src[d] : 0.f;
        m = m0;
        for (int t = t0; t < t1; ++t) {
            float li, lf;
            ml_gates<T>(a, t, h, li, lf);
            const float mn = fmaxf(lf + m, li), keep = expf(lf + m - mn), put = expf(li - mn);
            m = mn;
            if (d < dk) n = fmaf(ml_ld((const T*)a.rows + (size_t)t * a.stride + (size_t)(H + h) * dk + d), put, keep * n);
        }
        if (d < dk) dst[d] = n;
    }
    if (threadIdx.x == 0) pool_m[(size_t)state_out[r] * H + h] = m;
}

extern "C" int ilm_mlstm_max_dk() { return ML_NK * 64; }

static int ml_lanes(int dk) {
    int KP = 1;
    while (KP * ML_NK < dk) KP <<= 1;
    return KP;
}
// What a block of the step kernel must look like to hold a head's [dk, dv + 1] state whole: (threads, columns a thread), or 0.
static int ml_whole(int KP, int dv, int* threads, int* vc) {
    // (64 threads more than a power of two make room for n beside a power of two of columns)
    static const int shapes[][2] = {{256, 1}, {320, 1}, {256, 2}, {320, 2}, {256, 4}, {320, 4}, {512, 4}, {576, 4}, {1024, 4}};
    for (const auto& s : shapes)
        if ((s[0] / KP) * s[1] >= dv + 1) { *threads = s[0]; *vc = s[1]; return 1; }
    return 0;
}
// Whether the step kernel can end with the output norm (a block holds a head's state whole).
extern "C" int ilm_mlstm_step_norm_ok(int dk, int dv) {
    int th, vc;
    return dk <= ML_NK * 64 && ml_whole(ml_lanes(dk), dv, &th, &vc);
}

#define ML_CHECK_ROWS(what)                                                                                                            \
    ILM_REQUIRE(R > 0 && R <= 65535 && H > 0 && H <= 65535 && dk > 0 && dv > 0, what ": bad sizes");                                    \
    ILM_REQUIRE(rows_dt == ILM_DTYPE_F32 || rows_dt == ILM_DTYPE_BF16, what ": unknown dtype %d of the rows", rows_dt);                 \
    ILM_REQUIRE(row_stride % 8 == 0 && (((uintptr_t)rows | (uintptr_t)pool) & 15) == 0, what ": rows must be 16-byte aligned");         \
    ILM_REQUIRE(bias_i != nullptr && bias_f != nullptr && norm_w != nullptr, what ": gate biases and the norm's weight are needed");    \
    ILM_REQUIRE(i_off >= 0 && f_off >= 0 && g_off >= 0 && i_off + H <= row_stride && f_off + H <= row_stride                             \
                && (long)g_off + (long)H * dv <= row_stride && (long)H * (2L * dk + dv) <= row_stride, what ": rows of %d are too short", row_stride); \
    ILM_REQUIRE(cap > 0.f, what ": the gates' cap must be positive");                                                                   \
    const MlRows a = {rows, bias_i, bias_f, norm_w, (long)row_stride, i_off, f_off, g_off, b_dt, w_dt, cap, scale, eps}

// y != null: with the output norm (see ilm_mlstm_step_norm_ok); else o [T, H dv] float.  Segments of more than max_len tokens are
// passed over.
extern "C" int ilm_mlstm_step(void* o, void* y, const void* rows, int row_stride, int rows_dt, const void* bias_i, const void* bias_f, int b_dt,
                              int i_off, int f_off, int g_off, float cap, float scale, void* pool, void* pool_m, const void* state_in,
                              const void* state_out, const void* seg_offsets, int R, int H, int dk, int dv, int max_len, const void* norm_w, int w_dt,
                              float eps, int y_stride, int y_dt, hipStream_t stream) {
    ML_CHECK_ROWS("mlstm_step");
    ILM_REQUIRE(dk <= ML_NK * 64, "mlstm_step: keys of %d, at most %d", dk, ML_NK * 64);
    ILM_REQUIRE((y != nullptr) != (o != nullptr), "mlstm_step: one kind of result");
    const int KP = ml_lanes(dk);
#define ML_ARGS (float*)o, y, a, (float*)pool, (float*)pool_m, (const int*)state_in, (const int*)state_out, (const int*)seg_offsets, H, dk, dv,  \
                KP, max_len, y_stride, y_dt
#define ML_T(TH_, VC_, N_, GRID_)                                                                                                      \
    {                                                                                                                                  \
        if (rows_dt == ILM_DTYPE_F32) mlstm_step_kernel<float, TH_, VC_, N_><<<GRID_, TH_, 0, stream>>>(ML_ARGS);                       \
        else mlstm_step_kernel<bf16, TH_, VC_, N_><<<GRID_, TH_, 0, stream>>>(ML_ARGS);                                                 \
    }
    if (y != nullptr) {
        int th = 0, vc = 0;
        ILM_REQUIRE(ml_whole(KP, dv, &th, &vc), "mlstm_step: a head's state of %d x %d does not fit a block", dk, dv);
        const dim3 grid(1, H, R);
        if (th == 256 && vc == 1) ML_T(256, 1, true, grid)
        else if (th == 320 && vc == 1) ML_T(320, 1, true, grid)
        else if (th == 256 && vc == 2) ML_T(256, 2, true, grid)
        else if (th == 320 && vc == 2) ML_T(320, 2, true, grid)
        else if (th == 256) ML_T(256, 4, true, grid)
        else if (th == 320) ML_T(320, 4, true, grid)
        else if (th == 512) ML_T(512, 4, true, grid)
        else if (th == 576) ML_T(576, 4, true, grid)
        else ML_T(1024, 4, true, grid)
        ILM_LAUNCH_CHECK("mlstm_step (with the output norm)");
        return 0;
    }
    const int per = 256 / KP * 4 - 1;      // (at least three columns of v a block: KP is at most 64)
    const int blocks = (dv + per - 1) / per;
    const dim3 grid(blocks, H, R);
    ML_T(256, 4, false, grid)
    ILM_LAUNCH_CHECK("mlstm_step");
    if (blocks > 1) {
        if (rows_dt == ILM_DTYPE_F32)
            mlstm_step_norms_kernel<float><<<dim3(H, R), 256, 0, stream>>>(a, (float*)pool, (float*)pool_m, (const int*)state_in, (const int*)state_out,
                                                                           (const int*)seg_offsets, H, dk, dv, max_len);
        else
            mlstm_step_norms_kernel<bf16><<<dim3(H, R), 256, 0, stream>>>(a, (float*)pool, (float*)pool_m, (const int*)state_in, (const int*)state_out,
                                                                          (const int*)seg_offsets, H, dk, dv, max_len);
        ILM_LAUNCH_CHECK("mlstm_step (norms)");
    }
#undef ML_T
#undef ML_ARGS
    return 0;
}

// ---- long segments in pieces ------------------------------------------------------------------------------------------------
#define MC 64              // tokens a chunk
#define MW 8               // waves a block; a wave owns 16 columns of v
#define MCOLS (16 * MW)    // columns a block

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

// the segment whose slots hold slot s (-1: none), its piece p
__device__ __forceinline__ int ml_find(const int* __restrict__ seg_offsets, int R, int piece, int s, int& p) {
    int lo = 0, hi = R - 1;     // the last segment whose first slot is <= s
    while (lo < hi) {
        const int mid = (lo + hi + 1) >> 1;
        if (seg_offsets[mid] / piece + mid <= s) lo = mid; else hi = mid - 1;
    }
    p = s - (seg_offsets[lo] / piece + lo);
    return (p >= 0 && p * piece < seg_offsets[lo + 1] - seg_offsets[lo]) ? lo : -1;
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
template <int KT>
__global__ void __launch_bounds__(256)
mlstm_combine_kernel(float4* __restrict__ ws_s, float* __restrict__ ws_n, double* __restrict__ ws_m, float* __restrict__ pool,
                     const float* __restrict__ pool_m, const int* __restrict__ state_in, const int* __restrict__ state_out,
                     const int* __restrict__ seg_offsets, int H, int dk, int dv, int CT, int piece, int min_len) {
    constexpr int DK = KT * 16;
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
extern "C" int ilm_mlstm_chunk() { return MC; }
extern "C" int ilm_mlstm_chunk_max_dk() { return 16 * ML_MAX_KT; }
extern "C" int ilm_mlstm_chunk_cols() { return MCOLS; }
// floats of workspace a (slot, head) takes
extern "C" int ilm_mlstm_chunk_ws(int dk, int dv) {
    const int DK = ml_key_tiles(dk) * 16, CT = (dv + 15) / 16;
    return CT * 16 * DK + DK + 6;
}

// Segments of at least min_len tokens; the others are passed over.  piece: a multiple of 64; ws: (T / piece + R) * H *
// ilm_mlstm_chunk_ws floats.  y != null: with the output norm (dv <= ilm_mlstm_chunk_cols()); else o [T, H dv] float.
extern "C" int ilm_mlstm_chunks(void* o, void* y, const void* rows, int row_stride, int rows_dt, const void* bias_i, const void* bias_f, int b_dt,
                                int i_off, int f_off, int g_off, float cap, float scale, void* pool, void* pool_m, const void* state_in,
                                const void* state_out, const void* seg_offsets, int R, int H, int dk, int dv, int T_, int min_len, int piece,
                                const void* norm_w, int w_dt, float eps, int y_stride, int y_dt, void* ws, hipStream_t stream) {
    ML_CHECK_ROWS("mlstm_chunks");
    ILM_REQUIRE(T_ > 0 && dk <= 16 * ML_MAX_KT && piece > 0 && piece % MC == 0, "mlstm_chunks: keys of %d (at most %d), pieces of %d", dk,
                16 * ML_MAX_KT, piece);
    ILM_REQUIRE((y != nullptr) != (o != nullptr) && (y == nullptr || dv <= MCOLS), "mlstm_chunks: one kind of result, a norm over at most %d columns", MCOLS);
    const int slots = T_ / piece + R, KT = ml_key_tiles(dk), CT = (dv + 15) / 16, groups = (CT + MW - 1) / MW;
    ILM_REQUIRE(slots <= 65535 && ws != nullptr && ((uintptr_t)ws & 15) == 0, "mlstm_chunks: %d pieces in a step, at most 65535", slots);
    const size_t sh = (size_t)slots * H;
    float4* ws_s = (float4*)ws;
    float* ws_n = (float*)(ws_s + sh * CT * KT * 64);
    double* ws_m = (double*)(ws_n + sh * KT * 16);
    const dim3 grid(H * groups, slots), gc((CT * KT * 64 + KT * 4 + 255) / 256, H, R);
#define MLC_T(T__, KT_)                                                                                                                   \
    {                                                                                                                                     \
        mlstm_states_kernel<T__, KT_><<<grid, MW * 64, 0, stream>>>(ws_s, ws_n, ws_m, a, (const int*)seg_offsets, R, H, dk, dv, CT, piece, min_len); \
        ILM_LAUNCH_CHECK("mlstm_chunks (states)");                                                                                        \
        mlstm_combine_kernel<KT_><<<gc, 256, 0, stream>>>(ws_s, ws_n, ws_m, (float*)pool, (const float*)pool_m, (const int*)state_in,       \
                                                          (const int*)state_out, (const int*)seg_offsets, H, dk, dv, CT, piece, min_len);   \
        ILM_LAUNCH_CHECK("mlstm_chunks (combine)");                                                                                       \
        if (y != nullptr)                                                                                                                 \
            mlstm_outputs_kernel<T__, KT_, true><<<grid, MW * 64, 0, stream>>>(nullptr, y, ws_s, ws_n, ws_m, a, (float*)pool_m, (const int*)state_out, \
                                                                               (const int*)seg_offsets, R, H, dk, dv, CT, piece, min_len, y_stride, y_dt); \
        else                                                                                                                              \
            mlstm_outputs_kernel<T__, KT_, false><<<grid, MW * 64, 0, stream>>>((float*)o, nullptr, ws_s, ws_n, ws_m, a, (float*)pool_m,     \
                                                                                (const int*)state_out, (const int*)seg_offsets, R, H, dk, dv, CT,  \
                                                                                piece, min_len, y_stride, y_dt);                           \
    }
#define MLC_CASE(KT_)                                                                 \
    case KT_:                                                                         \
        if (rows_dt == ILM_DTYPE_F32) MLC_T(float, KT_) else MLC_T(bf16, KT_)          \
        break
    switch (KT) {
        MLC_CASE(1); MLC_CASE(2); MLC_CASE(3); MLC_CASE(4); MLC_CASE(5); MLC_CASE(6); MLC_CASE(7); MLC_CASE(8);
        MLC_CASE(12); MLC_CASE(16);
        default: ILM_REQUIRE(false, "mlstm_chunks: keys of %d", dk);
    }
#undef MLC_CASE
#undef MLC_T
    ILM_LAUNCH_CHECK("mlstm_chunks (outputs)");
    return 0;
}
