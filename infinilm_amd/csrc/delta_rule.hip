// The gated delta rule: a linear attention whose state forgets by a decay per head and step and is corrected by the
// difference between a token's value and what the state already holds under the token's key.  Per head, all in float:
//
//   D_t = g_t S_{t-1},   u_t = beta_t (v_t - k_t D_t),   S_t = D_t + outer(k_t, u_t),   o_t = q_t S_t
//
// with the vectors of token t as rows; S [dk, dv] is zero before a sequence's start.
//
// Inputs are float rows [q: G dkp | k: G dkp | v: H dv] (query and key heads filled up with zeros to dkp entries; head h reads
// query/key head h / (H / G)) and [beta: H | log g: H].  A request's state passes from step to step through a row of a pool,
// [H, dv, dk] (the key index fastest).
//
//   ilm_delta_step     token by token, a block a (request, head, columns).  A thread keeps DS_NK state entries (two pieces of
//       four, KP pieces apart, so that the lanes of a column read whole lines) of VC value columns in registers; the two sums a
//       token needs, k D and q D (the read-out after the write is q D + (k . q) u), and k . q are folded over the lanes of a
//       column together.  Where a block holds all columns of its head it can end with the head's output norm, weight and gate:
//       y = o / sqrt(mean(o^2) + eps) * w * silu(gate), in the activations' dtype.
//
//   ilm_delta_chunks   long segments (portions of prompts), in chunks of DC = 64 tokens on the float matrix instruction
//       (v_mfma_f32_16x16x4_f32: IEEE float products and sums).  With L_t the sum of the log-decays of a chunk's tokens up to t,
//       S_0 the state at its start, and A[t, i] = beta_t exp(L_t - L_i) k_t . k_i for i < t (0 elsewhere), the corrections u of
//       a chunk solve  (I + A) U = diag(beta) (V - diag(exp L) K S_0), so that
//           U  = V' - W S_0,     V' = (I + A)^-1 diag(beta) V,     W = (I + A)^-1 diag(beta exp L) K
//           o_t = exp(L_t) S_0^T q_t + sum_{i <= t} exp(L_t - L_i) (k_i . q_t) u_i
//           S   = exp(L_end) S_0 + sum_i exp(L_end - L_i) k_i u_i^T.
//       Two kernels: the first makes V', W, the weights of the second sum and the decayed keys of every chunk, all chunks and
//       heads side by side; the second walks a segment's chunks in order with 16 value columns of a head's state a block.
//       Differences of L are taken in double, so that a token's decay keeps its float precision however much has been
//       forgotten before it.  What passes from the first to the second lies in memory as the matrix instruction takes it (tiles of
//       16 x 16, a lane's 16 bytes after another's), so that a wave reads it in whole kilobytes.
//       Chunk p of segment r has the workspace slot floor(first row of r / DC) + r + p.
#include "common.h"

typedef __attribute__((ext_vector_type(4))) float f32x4;

#define DS_NK 8

template <int THREADS, int VC, bool NORM>
__global__ void __launch_bounds__(THREADS)
delta_step_kernel(float* __restrict__ o, void* __restrict__ y, const float* __restrict__ rows, int row_stride,
                  const float* __restrict__ gates, float* __restrict__ pool, const int* __restrict__ state_in,
                  const int* __restrict__ state_out, const int* __restrict__ seg_offsets, int H, int G, int dk, int dkp, int dv, int KP,
                  int max_len, const void* __restrict__ norm_w, const void* __restrict__ gate, int gate_stride, float eps, int y_stride,
                  int y_dt, int w_dt, int gate_dt) {
    __shared__ float red[THREADS / 64];
    const int h = blockIdx.y, r = blockIdx.z;
    const int t0 = seg_offsets[r], t1 = seg_offsets[r + 1];
    if (t0 >= t1 || t1 - t0 > max_len) return;       // (longer segments are another kernel's)
    const int kp = threadIdx.x % KP, c0 = (blockIdx.x * (THREADS / KP) + threadIdx.x / KP) * VC;
    const size_t hs = (size_t)dk * dv;
    const float* src = pool + ((size_t)state_in[r] * H + h) * hs;
    const bool v4 = dk % 4 == 0;
    // the thread's entries 4 p .. 4 p + 3 are k = kof[p] .. kof[p] + 3
    const int kof[2] = {4 * kp, 4 * (KP + kp)};
    float S[VC][DS_NK];
#pragma unroll
    for (int c = 0; c < VC; ++c) {
#pragma unroll
        for (int p = 0; p < 2; ++p) {
            const bool ok = c0 + c < dv && kof[p] < dk;
            const float* at = src + (size_t)(c0 + c) * dk + kof[p];
            if (v4) {
                const float4 t = ok ? *reinterpret_cast<const float4*>(at) : make_float4(0.f, 0.f, 0.f, 0.f);
                S[c][4 * p] = t.x; S[c][4 * p + 1] = t.y; S[c][4 * p + 2] = t.z; S[c][4 * p + 3] = t.w;
            } else {
#pragma unroll
                for (int e = 0; e < 4; ++e) S[c][4 * p + e] = (ok && kof[p] + e < dk) ? at[e] : 0.f;
            }
        }
    }
    const int g = h / (H / G);
    const float* qp = rows + (size_t)g * dkp;           // (dkp is a multiple of 4: a piece lies inside it whole, or beyond it whole)
    const float* kq = qp + (size_t)G * dkp;
    const float* vp = rows + (size_t)2 * G * dkp + (size_t)h * dv;
    for (int t = t0; t < t1; ++t) {
        float q[DS_NK], k[DS_NK], v[VC];
#pragma unroll
        for (int p = 0; p < 2; ++p) {
            const bool in = kof[p] < dkp;
            const float4 a = *reinterpret_cast<const float4*>(qp + (size_t)t * row_stride + (in ? kof[p] : 0));
            const float4 b = *reinterpret_cast<const float4*>(kq + (size_t)t * row_stride + (in ? kof[p] : 0));
            q[4 * p] = in ? a.x : 0.f; q[4 * p + 1] = in ? a.y : 0.f; q[4 * p + 2] = in ? a.z : 0.f; q[4 * p + 3] = in ? a.w : 0.f;
            k[4 * p] = in ? b.x : 0.f; k[4 * p + 1] = in ? b.y : 0.f; k[4 * p + 2] = in ? b.z : 0.f; k[4 * p + 3] = in ? b.w : 0.f;
        }
#pragma unroll
        for (int c = 0; c < VC; ++c) v[c] = vp[(size_t)t * row_stride + (c0 + c < dv ? c0 + c : 0)];
        const float beta = gates[(size_t)t * 2 * H + h], dec = expf(gates[(size_t)t * 2 * H + H + h]);
        float rk[VC], rq[VC], kdq = 0.f;
#pragma unroll
        for (int i = 0; i < DS_NK; ++i) kdq = fmaf(k[i], q[i], kdq);
#pragma unroll
        for (int c = 0; c < VC; ++c) {
            rk[c] = 0.f;
            rq[c] = 0.f;
#pragma unroll
            for (int i = 0; i < DS_NK; ++i) {
                S[c][i] *= dec;
                rk[c] = fmaf(S[c][i], k[i], rk[c]);
                rq[c] = fmaf(S[c][i], q[i], rq[c]);
            }
        }
        for (int off = 1; off < KP; off <<= 1) {
            kdq += __shfl_xor(kdq, off, 64);
#pragma unroll
            for (int c = 0; c < VC; ++c) {
                rk[c] += __shfl_xor(rk[c], off, 64);
                rq[c] += __shfl_xor(rq[c], off, 64);
            }
        }
        float ov[VC];
#pragma unroll
        for (int c = 0; c < VC; ++c) {
            const float u = beta * (v[c] - rk[c]);
            ov[c] = fmaf(u, kdq, rq[c]);
#pragma unroll
            for (int i = 0; i < DS_NK; ++i) S[c][i] = fmaf(k[i], u, S[c][i]);
        }
        if constexpr (NORM) {
            float ss = 0.f;
            if (kp == 0) {
#pragma unroll
                for (int c = 0; c < VC; ++c) ss = c0 + c < dv ? fmaf(ov[c], ov[c], ss) : ss;
            }
            const float rstd = 1.0f / sqrtf(block_sum<THREADS / 64>(ss, red) / (float)dv + eps);
#pragma unroll
            for (int c = 0; c < VC; ++c)
                if (kp == c % KP && c0 + c < dv) {      // (the columns' ends spread over the lanes)
                    const int j = c0 + c;
                    const float gv = gate_dt == ILM_DTYPE_F32 ? ((const float*)gate)[(size_t)t * gate_stride + h * dv + j]
                                                              : to_f32(((const bf16*)gate)[(size_t)t * gate_stride + h * dv + j]);
                    const float wv = w_dt == ILM_DTYPE_F32 ? ((const float*)norm_w)[j] : to_f32(((const bf16*)norm_w)[j]);
                    const float z = ov[c] * rstd * wv * (gv / (1.0f + expf(-gv)));
                    if (y_dt == ILM_DTYPE_F32) ((float*)y)[(size_t)t * y_stride + h * dv + j] = z;
                    else ((bf16*)y)[(size_t)t * y_stride + h * dv + j] = from_f32<bf16>(z);
                }
        } else {
#pragma unroll
            for (int c = 0; c < VC; ++c)
                if (kp == c % KP && c0 + c < dv) o[((size_t)t * H + h) * dv + c0 + c] = ov[c];
        }
    }
    float* dst = pool + ((size_t)state_out[r] * H + h) * hs;
#pragma unroll
    for (int c = 0; c < VC; ++c)
        if (c0 + c < dv) {
#pragma unroll
            for (int p = 0; p < 2; ++p) {
                float* at = dst + (size_t)(c0 + c) * dk + kof[p];
                if (v4) {
                    if (kof[p] < dk) *reinterpret_cast<float4*>(at) = make_float4(S[c][4 * p], S[c][4 * p + 1], S[c][4 * p + 2], S[c][4 * p + 3]);
                } else {
#pragma unroll
                    for (int e = 0; e < 4; ++e)
                        if (kof[p] + e < dk) at[e] = S[c][4 * p + e];
                }
            }
        }
}

extern "C" int ilm_delta_max_dk() { return DS_NK * 64; }

// What a block of the step kernel must look like to hold a head's [dk, dv] state whole: (threads, columns a thread), or 0.
static int ds_whole(int KP, int dv, int* threads, int* vc) {
    for (int th = 256; th <= 1024; th <<= 1)      // (four columns a thread leave four waves a SIMD their registers)
        for (int c = th == 256 ? 1 : 4; c <= 4; c <<= 1)
            if ((th / KP) * c >= dv) { *threads = th; *vc = c; return 1; }
    return 0;
}
static int ds_lanes(int dk) {
    int KP = 1;
    while (KP * DS_NK < dk) KP <<= 1;
    return KP;
}

// Whether the step kernel can end with the output norm (a block holds a head's state whole).
extern "C" int ilm_delta_step_norm_ok(int dk, int dv) {
    int th, vc;
    return dk <= DS_NK * 64 && ds_whole(ds_lanes(dk), dv, &th, &vc);
}

// y != null: with the output norm (see ilm_delta_step_norm_ok); else o [T, H dv] float.  Segments of more than max_len tokens are
// passed over.
extern "C" int ilm_delta_step(void* o, void* y, const void* rows, int row_stride, const void* gates, void* pool, const void* state_in,
                              const void* state_out, const void* seg_offsets, int R, int H, int G, int dk, int dkp, int dv, int max_len,
                              const void* norm_w, const void* gate, int gate_stride, float eps, int y_stride, int y_dt, int w_dt, int gate_dt,
                              hipStream_t stream) {
    ILM_REQUIRE(R > 0 && R <= 65535 && H > 0 && H <= 65535 && G > 0 && H % G == 0 && dk > 0 && dv > 0, "delta_step: bad sizes");
    ILM_REQUIRE(dk <= DS_NK * 64 && dkp >= dk && dkp % 8 == 0, "delta_step: keys of %d in %d, at most %d", dk, dkp, DS_NK * 64);
    ILM_REQUIRE(row_stride % 4 == 0 && ((uintptr_t)rows & 15) == 0 && ((uintptr_t)pool & 15) == 0, "delta_step: rows must be 16-byte aligned");
    ILM_REQUIRE((y != nullptr) != (o != nullptr), "delta_step: one kind of result");
    const int KP = ds_lanes(dk);
#define DS_ARGS (float*)o, y, (const float*)rows, row_stride, (const float*)gates, (float*)pool, (const int*)state_in,               \
                (const int*)state_out, (const int*)seg_offsets, H, G, dk, dkp, dv, KP, max_len, norm_w, gate, gate_stride, eps,      \
                y_stride, y_dt, w_dt, gate_dt
    if (y != nullptr) {
        int th = 0, vc = 0;
        ILM_REQUIRE(ds_whole(KP, dv, &th, &vc), "delta_step: a head's state of %d x %d does not fit a block", dk, dv);
        ILM_REQUIRE(norm_w != nullptr && gate != nullptr, "delta_step: the output norm needs its weight and the gate rows");
        const dim3 grid(1, H, R);
#define DS_N(TH_, VC_) if (th == TH_ && vc == VC_) delta_step_kernel<TH_, VC_, true><<<grid, TH_, 0, stream>>>(DS_ARGS)
        DS_N(256, 1); DS_N(256, 2); DS_N(256, 4); DS_N(512, 4); DS_N(1024, 4);
#undef DS_N
        ILM_LAUNCH_CHECK("delta_step (with the output norm)");
        return 0;
    }
    const int VT = 256 / KP;
    const int g4 = (dv + 4 * VT - 1) / (4 * VT);
    if ((long)g4 * H * R >= 2L * ilm_num_cus()) delta_step_kernel<256, 4, false><<<dim3(g4, H, R), 256, 0, stream>>>(DS_ARGS);
    else delta_step_kernel<256, 1, false><<<dim3((dv + VT - 1) / VT, H, R), 256, 0, stream>>>(DS_ARGS);
#undef DS_ARGS
    ILM_LAUNCH_CHECK("delta_step");
    return 0;
}

// ---- long segments in chunks ----------------------------------------------------------------------------------------------
#define DC 64
#define DC_MAX_DK 128
#define DC_EL (DC + 4)       // exp(L_t) of a chunk's tokens, then exp(L_end)

__device__ __forceinline__ f32x4 dc_mfma(float a, float b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }
// D += A[16 x 16] B[16 x 16]: lane (r, q) brings A[r][4q .. 4q + 3] and holds B and D as rows 4q .. 4q + 3 of column r
__device__ __forceinline__ f32x4 dc_mma(const float4& a, const f32x4& b, f32x4 c) {
    c = dc_mfma(a.x, b[0], c);
    c = dc_mfma(a.y, b[1], c);
    c = dc_mfma(a.z, b[2], c);
    return dc_mfma(a.w, b[3], c);
}
// D += A[16 x 16] B^T: both sides as rows, lane (r, q) brings A[r][4q ..] and B[r][4q ..]
__device__ __forceinline__ f32x4 dc_mmt(const float4& a, const float4& b, f32x4 c) {
    c = dc_mfma(a.x, b.x, c);
    c = dc_mfma(a.y, b.y, c);
    c = dc_mfma(a.z, b.z, c);
    return dc_mfma(a.w, b.w, c);
}

// the segment whose slots hold slot s (-1: none), its chunk p
__device__ __forceinline__ int dc_find(const int* __restrict__ seg_offsets, int R, int s, int& p) {
    int lo = 0, hi = R - 1;     // the last segment whose first slot is <= s
    while (lo < hi) {
        const int mid = (lo + hi + 1) >> 1;
        if (seg_offsets[mid] / DC + mid <= s) lo = mid; else hi = mid - 1;
    }
    p = s - (seg_offsets[lo] / DC + lo);
    return (p >= 0 && p * DC < seg_offsets[lo + 1] - seg_offsets[lo]) ? lo : -1;
}

#define DC_PW 8      // waves of the first kernel's blocks
#define DC_XT 2      // column tiles of [V | K] a wave solves together

// KT: key entries / 16
template <int KT>
__global__ void __launch_bounds__(DC_PW * 64, 4)
delta_chunk_prepare_kernel(float4* __restrict__ ws_v, float4* __restrict__ ws_w, float4* __restrict__ ws_q, float4* __restrict__ ws_k,
                           float4* __restrict__ ws_p, float* __restrict__ ws_e, const float* __restrict__ rows, int row_stride, const float* __restrict__ gates,
                           const int* __restrict__ seg_offsets, int R, int H, int G, int dv, int dvp, int min_len) {
    constexpr int DK = KT * 16, KS = DK + 4, AS = DC + 4, TS = 20;
    __shared__ __attribute__((aligned(16))) float Ks[DC * KS];
    __shared__ __attribute__((aligned(16))) float An[DC * AS];          // -A
    __shared__ __attribute__((aligned(16))) float Ti[4 * 16 * TS];      // inverses of the diagonal blocks of I + A
    __shared__ __attribute__((aligned(16))) float Tp[DC_PW * 16 * TS];      // a wave's tile on its way into fragment order
    __shared__ double Ls[DC];
    __shared__ float bs[DC], fs[DC], es[DC];                            // beta; exp(L_end - L); beta exp(L)
    const int h = blockIdx.x, slot = blockIdx.y;
    int p;
    const int seg = dc_find(seg_offsets, R, slot, p);
    if (seg < 0) return;
    const int len = seg_offsets[seg + 1] - seg_offsets[seg];
    if (len < min_len) return;                         // (the step kernel's)
    const int t0 = seg_offsets[seg] + p * DC, n = min(DC, len - p * DC);
    const int tid = threadIdx.x, lane = tid & 63, r = lane & 15, q = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int g = h / (H / G);
    const float* qrow = rows + (size_t)t0 * row_stride + (size_t)g * DK;
    const float* krow = qrow + (size_t)G * DK;
    const float* vrow = rows + (size_t)t0 * row_stride + (size_t)2 * G * DK + (size_t)h * dv;
    const size_t sh = (size_t)slot * H + h;
    // the values of the wave's first column tiles, on their way from the start
    const int nv = dvp / 16, nt = nv + KT;
    float rv[4][DC_XT][4];
    auto load_values = [&](int c0) {
#pragma unroll
        for (int c = 0; c < DC_XT; ++c) {
            if (c0 + c >= nv) continue;                // wave-uniform
            const int col = 16 * (c0 + c) + r;
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const int t = 16 * i + 4 * q + e;
                    rv[i][c][e] = vrow[(size_t)(t < n ? t : n - 1) * row_stride + (col < dv ? col : dv - 1)];
                }
        }
    };
    for (int i = tid; i < DC * (DK / 4); i += DC_PW * 64) {
        const int t = i / (DK / 4), c = (i % (DK / 4)) * 4;
        const float4 v = *reinterpret_cast<const float4*>(krow + (size_t)(t < n ? t : n - 1) * row_stride + c);
        *reinterpret_cast<float4*>(&Ks[t * KS + c]) = t < n ? v : make_float4(0.f, 0.f, 0.f, 0.f);
    }
    load_values(wave * DC_XT);
    if (wave == 0) {
        const float* gt = gates + (size_t)(t0 + (lane < n ? lane : n - 1)) * 2 * H + h;
        double L = lane < n ? (double)gt[H] : 0.0;
#pragma unroll
        for (int off = 1; off < 64; off <<= 1) {
            const double up = __shfl_up(L, off, 64);
            if (lane >= off) L += up;
        }
        Ls[lane] = L;
        bs[lane] = lane < n ? gt[0] : 0.f;
        fs[lane] = expf((float)(__shfl(L, 63, 64) - L));
        const float eL = expf((float)L);
        es[lane] = bs[lane] * eL;
        ws_e[sh * DC_EL + lane] = eL;
        if (lane == 63) ws_e[sh * DC_EL + DC] = eL;
    }
    __syncthreads();
    // ---- k_t . k_i and q_t . k_i by tiles of 16 x 16 at and below the diagonal
    for (int task = wave; task < 20; task += DC_PW) {
        const int tile = task >> 1, rt = tile < 1 ? 0 : (tile < 3 ? 1 : (tile < 6 ? 2 : 3)), ct = tile - rt * (rt + 1) / 2;
        f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
        if (task & 1) {      // k_i . q_t as [i, t]
            const int tq = 16 * rt + r < n ? 16 * rt + r : n - 1;
            float4 qa[KT];
#pragma unroll
            for (int j = 0; j < KT; ++j) qa[j] = *reinterpret_cast<const float4*>(qrow + (size_t)tq * row_stride + 16 * j + 4 * q);
#pragma unroll
            for (int j = 0; j < KT; ++j) {
                acc = dc_mmt(*reinterpret_cast<const float4*>(&Ks[(16 * ct + r) * KS + 16 * j + 4 * q]), qa[j], acc);
                if (ct == rt) ws_q[((sh * 4 + rt) * KT + j) * 64 + lane] = qa[j];
            }
            const double Lt = Ls[16 * rt + r];
            float4 pw;
            float* pe = reinterpret_cast<float*>(&pw);
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int i = 16 * ct + 4 * q + e;
                pe[e] = i <= 16 * rt + r ? expf((float)(Lt - Ls[i])) * acc[e] : 0.f;
            }
            ws_p[((sh * 4 + rt) * 4 + ct) * 64 + lane] = pw;
        } else {             // k_t . k_i as [t, i]
#pragma unroll
            for (int j = 0; j < KT; ++j)
                acc = dc_mmt(*reinterpret_cast<const float4*>(&Ks[(16 * rt + r) * KS + 16 * j + 4 * q]),
                             *reinterpret_cast<const float4*>(&Ks[(16 * ct + r) * KS + 16 * j + 4 * q]), acc);
            const double Li = Ls[16 * ct + r];
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int t = 16 * rt + 4 * q + e;
                An[t * AS + 16 * ct + r] = 16 * ct + r < t ? -bs[t] * expf((float)(Ls[t] - Li)) * acc[e] : 0.f;
            }
        }
    }
    __syncthreads();
    if (wave == 0) {      // column r of the inverse of diagonal block q, by substitution
        float x[16];
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            float v = i == r ? 1.0f : 0.f;
#pragma unroll
            for (int j = 0; j < i; j += 4) {
                const float4 a = *reinterpret_cast<const float4*>(&An[(16 * q + i) * AS + 16 * q + j]);
                v = fmaf(a.x, x[j], v);
                if (j + 1 < i) v = fmaf(a.y, x[j + 1], v);
                if (j + 2 < i) v = fmaf(a.z, x[j + 2], v);
                if (j + 3 < i) v = fmaf(a.w, x[j + 3], v);
            }
            x[i] = v;
        }
#pragma unroll
        for (int i = 0; i < 16; ++i) Ti[(q * 16 + i) * TS + r] = x[i];
    } else {              // the decayed keys, transposed: tile (m, j) holds keys' entries 16 m .. by tokens 16 j ..
        for (int i = wave - 1; i < KT * 4; i += DC_PW - 1) {
            const int m = i >> 2, j = i & 3;
            float4 v;
            float* ve = reinterpret_cast<float*>(&v);
#pragma unroll
            for (int e = 0; e < 4; ++e) ve[e] = fs[16 * j + 4 * q + e] * Ks[(16 * j + 4 * q + e) * KS + 16 * m + r];
            ws_k[((sh * KT + m) * 4 + j) * 64 + lane] = v;
        }
    }
    __syncthreads();
    // ---- (I + A) X = [beta V | beta exp(L) K], DC_XT column tiles of 16 a wave, the rows' blocks one after the other
    for (int c0 = wave * DC_XT; c0 < nt; c0 += DC_PW * DC_XT) {
        f32x4 X[4][DC_XT];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            f32x4 acc[DC_XT];
#pragma unroll
            for (int c = 0; c < DC_XT; ++c) {
                const int ct = c0 + c;                 // wave-uniform
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const int t = 16 * i + 4 * q + e;
                    float v = 0.f;
                    if (ct < nv) v = 16 * ct + r < dv ? rv[i][c][e] * bs[t] : 0.f;
                    else if (ct < nt) v = es[t] * Ks[t * KS + 16 * (ct - nv) + r];
                    acc[c][e] = v;
                }
            }
#pragma unroll
            for (int j = 0; j < i; ++j) {
                const float4 a = *reinterpret_cast<const float4*>(&An[(16 * i + r) * AS + 16 * j + 4 * q]);
#pragma unroll
                for (int c = 0; c < DC_XT; ++c) acc[c] = dc_mma(a, X[j][c], acc[c]);
            }
            const float4 d = *reinterpret_cast<const float4*>(&Ti[(i * 16 + r) * TS + 4 * q]);
#pragma unroll
            for (int c = 0; c < DC_XT; ++c) X[i][c] = dc_mma(d, acc[c], f32x4{0.f, 0.f, 0.f, 0.f});
        }
        load_values(c0 + DC_PW * DC_XT);
#pragma unroll
        for (int c = 0; c < DC_XT; ++c) {
            const int ct = c0 + c;
            if (ct >= nt) break;
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                if (ct < nv) {       // V' as the walk's results lie: rows 4 q .. 4 q + 3 of column r
                    ws_v[((sh * 4 + i) * nv + ct) * 64 + lane] = make_float4(X[i][c][0], X[i][c][1], X[i][c][2], X[i][c][3]);
                } else {             // W as an operand: row r, entries 4 q .. 4 q + 3
                    float* tp = Tp + wave * 16 * TS;
#pragma unroll
                    for (int e = 0; e < 4; ++e) tp[(4 * q + e) * TS + r] = X[i][c][e];
                    __builtin_amdgcn_wave_barrier();
                    ws_w[((sh * 4 + i) * KT + ct - nv) * 64 + lane] = *reinterpret_cast<const float4*>(&tp[r * TS + 4 * q]);
                    __builtin_amdgcn_wave_barrier();
                }
            }
        }
    }
}

// The walk: eight waves a block.  Waves 0 to 3 form a chunk's corrections, U = V' - W S_0, 16 rows each; waves 4 to 7 its outputs,
// exp(L) (Q S_0) + P U; every wave makes one tile of 16 entries of the next state.  What a wave reads of a chunk:
template <int KT>
struct dc_operands {
    float4 a[KT];       // its 16 rows of W, or of q
    float4 k[4];        // its tile of the decayed keys
    float4 p[4];        // outputs: the second sum's weights; corrections: V' (the first of them)
    float4 e;           // outputs: exp(L) of the lane's four rows
    float end;          // exp(L_end)
};

struct dc_source {
    const float4 *a, *k, *p;
    const float *e, *end;
};

template <int KT>
__global__ void __launch_bounds__(512, 2)
delta_chunk_walk_kernel(float* __restrict__ out, const float4* __restrict__ ws_v, const float4* __restrict__ ws_w, const float4* __restrict__ ws_q,
                        const float4* __restrict__ ws_k, const float4* __restrict__ ws_p, const float* __restrict__ ws_e,
                        float* __restrict__ pool, const int* __restrict__ state_in, const int* __restrict__ state_out,
                        const int* __restrict__ seg_offsets, int H, int dk, int dv, int dvp, int min_len) {
    static_assert(KT <= 8, "a wave makes one tile of the state");
    __shared__ f32x4 Us[4][64];
    __shared__ f32x4 Ss[KT][64];
    // blocks go to the eight dies in turn; with this numbering the column blocks of a head share a die, whose cache then holds
    // the operands that they all read
    const int nb = dvp / 16, items = nb * H, per = (items + 7) / 8;
    const int item = (int)(blockIdx.x & 7) * per + (int)(blockIdx.x >> 3);
    if ((int)(blockIdx.x >> 3) >= per || item >= items) return;
    const int h = item / nb, blk = item % nb, col0 = blk * 16, seg = blockIdx.y;
    const int s0 = seg_offsets[seg], len = seg_offsets[seg + 1] - s0;
    if (len <= 0 || len < min_len) return;
    const int chunks = (len + DC - 1) / DC;
    const int lane = threadIdx.x & 63, r = lane & 15, q = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), wr = wave & 3;      // wr: its tile of 16 rows
    const bool outputs = wave >= 4, makes = wave < KT;
    const bool col_ok = col0 + r < dv, v4 = dk % 4 == 0;
    // state tile m: entries 16 m + 4 q + e of column col0 + r
    const float* src = pool + (((size_t)state_in[seg] * H + h) * dv + (col_ok ? col0 + r : 0)) * dk;
    auto state_tile = [&](int m) -> f32x4 {
        const int k0 = 16 * m + 4 * q;
        f32x4 s = f32x4{0.f, 0.f, 0.f, 0.f};
        if (v4) {
            const float4 t = *reinterpret_cast<const float4*>(src + (k0 < dk ? k0 : 0));
            if (col_ok && k0 < dk) s = f32x4{t.x, t.y, t.z, t.w};
        } else {
#pragma unroll
            for (int e = 0; e < 4; ++e)
                if (col_ok && k0 + e < dk) s[e] = src[k0 + e];
        }
        return s;
    };
    f32x4 S[KT], own = state_tile(makes ? wave : 0);      // every wave holds the whole state, and the tile it makes once more
#pragma unroll
    for (int m = 0; m < KT; ++m) S[m] = state_tile(m);
    // (every piece is 64 consecutive 16-byte entries, one a lane; a chunk's pieces lie H heads after the last chunk's)
    dc_source at;
    {
        const size_t sh = (size_t)(s0 / DC + seg) * H + h;
        at.a = (outputs ? ws_q : ws_w) + (sh * 4 + wr) * KT * 64 + lane;
        at.k = ws_k + (sh * KT + (makes ? wave : 0)) * 4 * 64 + lane;
        at.p = outputs ? ws_p + (sh * 4 + wr) * 4 * 64 + lane : ws_v + ((sh * 4 + wr) * nb + blk) * 64 + lane;
        at.e = ws_e + sh * DC_EL + 16 * wr + 4 * q;
        at.end = ws_e + sh * DC_EL + DC;
    }
    const size_t step_a = (size_t)H * 4 * KT * 64, step_p = (size_t)H * 4 * (outputs ? 4 : nb) * 64, step_e = (size_t)H * DC_EL;
    auto load = [&](dc_operands<KT>& o) {
#pragma unroll
        for (int j = 0; j < KT; ++j) o.a[j] = at.a[j * 64];
#pragma unroll
        for (int j = 0; j < 4; ++j) o.k[j] = at.k[j * 64];
        o.p[0] = at.p[0];
        if (outputs) {
            // (blocks above the diagonal are not in memory: the diagonal's own is read in their place and not used)
#pragma unroll
            for (int j = 1; j < 4; ++j) o.p[j] = at.p[(j <= wr ? j : wr) * 64];
            o.e = *reinterpret_cast<const float4*>(at.e);
        }
        o.end = *at.end;
        at.a += step_a;
        at.k += step_a;
        at.p += step_p;
        at.e += step_e;
        at.end += step_e;
    };
    auto chunk = [&](int c, dc_operands<KT>& cur, dc_operands<KT>& nxt) {
        if (c + 1 < chunks) load(nxt);
        f32x4 x0 = f32x4{0.f, 0.f, 0.f, 0.f}, x1 = x0;
#pragma unroll
        for (int m = 0; m < KT; ++m) {
            if (m & 1) x1 = dc_mma(cur.a[m], S[m], x1);
            else x0 = dc_mma(cur.a[m], S[m], x0);
        }
        x0 = x0 + x1;
        if (!outputs) Us[wr][lane] = f32x4{cur.p[0].x, cur.p[0].y, cur.p[0].z, cur.p[0].w} - x0;
        __syncthreads();
        f32x4 U[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) U[j] = Us[j][lane];
        if (makes) {
            own = own * cur.end;
#pragma unroll
            for (int j = 0; j < 4; ++j) own = dc_mma(cur.k[j], U[j], own);
            Ss[wave][lane] = own;
        }
        __syncthreads();
#pragma unroll
        for (int m = 0; m < KT; ++m) S[m] = Ss[m][lane];
        if (outputs) {       // (off the path from state to state)
            f32x4 o = f32x4{x0[0] * cur.e.x, x0[1] * cur.e.y, x0[2] * cur.e.z, x0[3] * cur.e.w};
#pragma unroll
            for (int j = 0; j < 4; ++j)
                if (j <= wr) o = dc_mma(cur.p[j], U[j], o);
            const int t0 = c * DC + 16 * wr + 4 * q;
#pragma unroll
            for (int e = 0; e < 4; ++e)
                if (col_ok && t0 + e < len) out[((size_t)(s0 + t0 + e) * H + h) * dv + col0 + r] = o[e];
        }
    };
    dc_operands<KT> A, B;
    load(A);
    for (int c = 0; c < chunks; c += 2) {
        chunk(c, A, B);
        if (c + 1 < chunks) chunk(c + 1, B, A);
    }
    if (!col_ok || !makes) return;
    float* dst = pool + (((size_t)state_out[seg] * H + h) * dv + col0 + r) * dk;
    const int k0 = 16 * wave + 4 * q;
    if (v4) {
        if (k0 < dk) *reinterpret_cast<float4*>(dst + k0) = make_float4(own[0], own[1], own[2], own[3]);
    } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
            if (k0 + e < dk) dst[k0 + e] = own[e];
    }
}

extern "C" int ilm_delta_chunk() { return DC; }
extern "C" int ilm_delta_chunk_max_dk() { return DC_MAX_DK; }
// floats of workspace a (slot, head) takes
extern "C" int ilm_delta_chunk_ws(int dkp, int dvp) { return DC * dvp + 3 * DC * dkp + DC * DC + DC_EL; }

// Segments of at least min_len tokens; the others are passed over.  ws: (T / DC + R) * H * ilm_delta_chunk_ws floats.
extern "C" int ilm_delta_chunks(void* o, const void* rows, int row_stride, const void* gates, void* pool, const void* state_in,
                                const void* state_out, const void* seg_offsets, int R, int H, int G, int dk, int dkp, int dv, int T_, int min_len,
                                void* ws, hipStream_t stream) {
    ILM_REQUIRE(T_ > 0 && R > 0 && R <= 65535 && H > 0 && G > 0 && H % G == 0 && dk > 0 && dv > 0, "delta_chunks: bad sizes");
    ILM_REQUIRE(dk <= DC_MAX_DK && dkp == (dk + 15) / 16 * 16, "delta_chunks: keys of %d in %d, at most %d", dk, dkp, DC_MAX_DK);
    ILM_REQUIRE(row_stride % 4 == 0 && (((uintptr_t)rows | (uintptr_t)pool | (uintptr_t)ws) & 15) == 0, "delta_chunks: rows must be 16-byte aligned");
    const int slots = T_ / DC + R, dvp = (dv + 15) / 16 * 16;
    ILM_REQUIRE(slots <= 65535 && ws != nullptr, "delta_chunks: %d chunks in a step, at most 65535", slots);
    const size_t sh = (size_t)slots * H;
    float4* ws_v = (float4*)ws;
    float4* ws_w = ws_v + sh * (DC / 4) * dvp;
    float4* ws_q = ws_w + sh * (DC / 4) * dkp;
    float4* ws_k = ws_q + sh * (DC / 4) * dkp;
    float4* ws_p = ws_k + sh * (DC / 4) * dkp;
    float* ws_e = (float*)(ws_p + sh * (DC / 4) * DC);
    const dim3 ga(H, slots), gb(8 * ((dvp / 16 * H + 7) / 8), R);
#define DC_CASE(KT_)                                                                                                                  \
    case KT_:                                                                                                                         \
        delta_chunk_prepare_kernel<KT_><<<ga, DC_PW * 64, 0, stream>>>(ws_v, ws_w, ws_q, ws_k, ws_p, ws_e, (const float*)rows, row_stride,    \
                                                                (const float*)gates, (const int*)seg_offsets, R, H, G, dv, dvp, min_len); \
        ILM_LAUNCH_CHECK("delta_chunks (prepare)");                                                                                   \
        delta_chunk_walk_kernel<KT_><<<gb, 512, 0, stream>>>((float*)o, ws_v, ws_w, ws_q, ws_k, ws_p, ws_e, (float*)pool,              \
                                                             (const int*)state_in, (const int*)state_out, (const int*)seg_offsets, H,  \
                                                             dk, dv, dvp, min_len);                                                    \
        break
    switch (dkp / 16) {
        DC_CASE(1); DC_CASE(2); DC_CASE(3); DC_CASE(4); DC_CASE(5); DC_CASE(6); DC_CASE(7); DC_CASE(8);
        default: ILM_REQUIRE(false, "delta_chunks: keys of %d", dk);
    }
#undef DC_CASE
    ILM_LAUNCH_CHECK("delta_chunks (walk)");
    return 0;
}
