// Gated delta rules of the layer-list decoders (layered.h), sizes and constants as arguments, and the latent row's way into the cache.
//
//   S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q          per head, state S [d][e]
//
// with g one decay per head or one per key channel, q and k of unit length behind a short causal convolution and SiLU.  Everything is f32
// in both number formats.  Three forms: decode steps (one launch does convolution, unit lengths, gates and the recurrence, a second one
// the head norm, the output gate and the convolution's tail), short portions (preparation, then token by token with the state in
// registers), long portions (parallel over chunks of 64 tokens on the f32 matrix cores).
#include <hip/hip_runtime.h>

#include <algorithm>

#include "dev_common.h"
#include "layered.h"

namespace cm {

namespace {
constexpr float UNIT_EPS = 1e-6f;          // inside the root of a unit vector's length
constexpr size_t LD_LDS_PLAIN = 64 * 1024, LD_LDS_MAX = 160 * 1024;

__device__ __forceinline__ float dl_silu(float v) { return v / (1.f + expf(-v)); }
__device__ __forceinline__ float dl_sigmoid(float v) { return 1.f / (1.f + expf(-v)); }
__device__ __forceinline__ float dl_softplus(float v) { return fmaxf(v, 0.f) + log1pf(expf(-fabsf(v))); }

// output gates (not part of the recurrence): the hardware exponential
__device__ __forceinline__ float dl_gate(float v, int act) { return (act == LACT_SILU ? v : 1.f) / (1.f + __expf(-v)); }

// workgroup barrier for LDS hand-offs: waits for this wave's LDS operations, not for its outstanding global loads
__device__ __forceinline__ void dl_lds_barrier() {
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
}
// c += a . b over 16 values of k: lane's a = A[i = lane % 16][k = 4 (lane / 16) ..], b = B[k = 4 (lane / 16) ..][j = lane % 16], and
// c = C[i = 4 (lane / 16) ..][j = lane % 16] -- the layout of b is the layout of c, so a result is the next product's b as it stands
__device__ __forceinline__ f32x4 dl_mfma(const f32x4& a, const f32x4& b, f32x4 c) {
    c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[0], b[0], c, 0, 0, 0);
    c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[1], b[1], c, 0, 0, 0);
    c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[2], b[2], c, 0, 0, 0);
    c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[3], b[3], c, 0, 0, 0);
    return c;
}
}  // namespace

// ------------------------------------------------------------------------------------------------------------------
// latent row: norm and cache append, one block per row
// ------------------------------------------------------------------------------------------------------------------
template <int KVT>
__global__ __launch_bounds__(256) void lay_latent_append_kernel(const float* __restrict__ proj, int ldp, int k_off, int n, const float* __restrict__ w,
                                                                float eps, void* __restrict__ kpool, const int32_t* __restrict__ bt,
                                                                const LaySegDev* __restrict__ segs, const int32_t* __restrict__ rowseg, int page) {
    __shared__ float red[4];
    const int r = blockIdx.x, tid = threadIdx.x;
    const float* x = proj + (size_t)r * ldp + k_off;
    float v[2], ss = 0.f;                  // the thread's first two elements stay in registers (the whole row up to a latent of 512)
#pragma unroll
    for (int i = 0; i < 2; ++i) {
        const int c = tid + 256 * i;
        v[i] = c < n ? x[c] : 0.f;
        ss = fmaf(v[i], v[i], ss);
    }
    for (int c = tid + 512; c < n; c += 256) ss = fmaf(x[c], x[c], ss);
    const LaySegDev sg = segs[rowseg[r]];
    const int pos = sg.start_pos + (r - sg.row0);
    const size_t row = ((size_t)bt[sg.bt_off + pos / page] * page + (size_t)(pos % page)) * n;
    ss = wave_sum(ss);
    if ((tid & 63) == 0) red[tid >> 6] = ss;
    __syncthreads();
    const float rs = 1.f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)n + eps);
    auto put = [&](int c, float y) {
        if (KVT == KV_F32) ((float*)kpool)[row + c] = y;
        else ((uint16_t*)kpool)[row + c] = f32_to_bf16(y);
    };
#pragma unroll
    for (int i = 0; i < 2; ++i)
        if (tid + 256 * i < n) put(tid + 256 * i, v[i] * rs * w[tid + 256 * i]);
    for (int c = tid + 512; c < n; c += 256) put(c, x[c] * rs * w[c]);
}
void launch_lay_latent_append(const float* proj, int ldp, int k_off, int n, const float* w, float eps, void* kpool, int kvt, const int32_t* bt,
                              const LaySegDev* segs, const int32_t* rowseg, int T, int page, hipStream_t s) {
    if (T <= 0 || n <= 0) return;
    if (kvt == KV_F32) hipLaunchKernelGGL(lay_latent_append_kernel<KV_F32>, dim3((unsigned)T), dim3(256), 0, s, proj, ldp, k_off, n, w, eps, kpool, bt, segs, rowseg, page);
    else hipLaunchKernelGGL(lay_latent_append_kernel<KV_BF16>, dim3((unsigned)T), dim3(256), 0, s, proj, ldp, k_off, n, w, eps, kpool, bt, segs, rowseg, page);
}

// ------------------------------------------------------------------------------------------------------------------
// preparation of a portion: convolution + SiLU, unit lengths, write strengths, decays.  A wave owns one query or key head (or 64 VPL value
// channels) for LP_ROWS consecutive rows of the pass; TAPS > 0: the convolution's window rolls in registers
// ------------------------------------------------------------------------------------------------------------------
constexpr int LP_ROWS = 8;
template <int VPL, int TAPS>
__global__ __launch_bounds__(256) void lay_delta_prep_kernel(LDeltaArgs a) {
    const int lane = threadIdx.x & 63, unit = blockIdx.y * 4 + (threadIdx.x >> 6);
    const int r0 = blockIdx.x * LP_ROWS, nr = min(LP_ROWS, a.T - r0);
    const int qk = 2 * a.G, C = 2 * a.G * a.d + a.H * a.e, taps = TAPS > 0 ? TAPS : a.taps;
    const int nv = (a.H * a.e + 64 * VPL - 1) / (64 * VPL);
    if (unit > qk + nv) return;
    if (unit == qk + nv) {                 // per head: write strength, and the decay of the head form
        for (int i = lane; i < nr * a.H; i += 64) {
            const int r = r0 + i / a.H, h = i % a.H;
            const float* p = a.proj + (size_t)r * a.ldp;
            a.beta[(size_t)r * a.H + h] = dl_sigmoid(p[a.b_off + h]);
            if (!a.channel) a.ldec[(size_t)r * a.H + h] = a.a_neg[h] * dl_softplus(p[a.a_off + h] + a.dt_bias[h]);
        }
        return;
    }
    const bool head = unit < qk;
    const int c0 = head ? unit * a.d : qk * a.d + (unit - qk) * 64 * VPL;
    const int nc = head ? a.d : min(64 * VPL, C - c0);
    const float qs = unit < a.G ? 1.f / sqrtf((float)a.d) : 1.f;
    int ch[VPL];
#pragma unroll
    for (int v = 0; v < VPL; ++v) ch[v] = c0 + min(lane + 64 * v, nc - 1);      // lanes past the end repeat the last channel; nothing of theirs is stored
    constexpr int NT = TAPS > 0 ? TAPS : 1;
    float cw[NT][VPL], x[LP_ROWS][VPL], win[NT][VPL];
    if (TAPS > 0) {
#pragma unroll
        for (int j = 0; j < NT; ++j)
#pragma unroll
            for (int v = 0; v < VPL; ++v) cw[j][v] = a.conv_w[(size_t)ch[v] * taps + j];
    }
#pragma unroll
    for (int i = 0; i < LP_ROWS; ++i)
#pragma unroll
        for (int v = 0; v < VPL; ++v) x[i][v] = a.proj[(size_t)min(r0 + i, a.T - 1) * a.ldp + a.q_off + ch[v]];
#pragma unroll
    for (int i = 0; i < LP_ROWS; ++i) {
        if (i >= nr) break;
        const int r = r0 + i;
        const LaySegDev sg = a.segs[a.rowseg[r]];
        const int local = r - sg.row0;
        const float* tail = a.conv_pool + (size_t)sg.slot * a.conv_stride + a.cv_off;
        // input `back` tokens before this row's
        auto earlier = [&](int back, int v) {
            const int src = local - back;
            return src >= 0 ? a.proj[(size_t)(sg.row0 + src) * a.ldp + a.q_off + ch[v]] : tail[(size_t)(taps - 1 + src) * C + ch[v]];
        };
        float y[VPL], ss = 0.f;
        if (TAPS > 0) {
            if (i == 0 || local == 0) {
#pragma unroll
                for (int j = 0; j + 1 < NT; ++j)
#pragma unroll
                    for (int v = 0; v < VPL; ++v) win[j][v] = earlier(NT - 1 - j, v);
            }
#pragma unroll
            for (int v = 0; v < VPL; ++v) {
                float acc = 0.f;
#pragma unroll
                for (int j = 0; j + 1 < NT; ++j) acc = fmaf(cw[j][v], win[j][v], acc);
                y[v] = fmaf(cw[NT - 1][v], x[i][v], acc);
#pragma unroll
                for (int j = 0; j + 2 < NT; ++j) win[j][v] = win[j + 1][v];
                if (NT > 1) win[NT > 1 ? NT - 2 : 0][v] = x[i][v];
            }
        } else {
#pragma unroll
            for (int v = 0; v < VPL; ++v) {
                float acc = 0.f;
                for (int j = 0; j + 1 < taps; ++j) acc = fmaf(a.conv_w[(size_t)ch[v] * taps + j], earlier(taps - 1 - j, v), acc);
                y[v] = fmaf(a.conv_w[(size_t)ch[v] * taps + taps - 1], x[i][v], acc);
            }
        }
#pragma unroll
        for (int v = 0; v < VPL; ++v) {
            y[v] = dl_silu(y[v]);
            if (lane + 64 * v < nc) ss = fmaf(y[v], y[v], ss);
        }
        float f = 1.f;
        if (head) f = qs / sqrtf(wave_sum(ss) + UNIT_EPS);
#pragma unroll
        for (int v = 0; v < VPL; ++v)
            if (lane + 64 * v < nc) a.xb[(size_t)r * C + ch[v]] = y[v] * f;
    }
}

// ------------------------------------------------------------------------------------------------------------------
// token by token.  A block owns 32 value columns of one (sequence, head): thread = (column, 1/8 of the key rows), NR rows in registers.
// With p = (g S)^T k and r = (g S)^T q both summed before the write: u = beta (v - p), o = r + (k . q) u -- one barrier per token.
// FUSED (decode steps): the block forms its own q, k, v, write strength and decay; only lay_delta_out replaces the convolution's tail.
// ------------------------------------------------------------------------------------------------------------------
constexpr int LQ_COLS = 32, LQ_GRP = 8;
constexpr int lq_batch(bool fused, int nr) { return fused ? 1 : (nr > 16 ? 8 : 16); }      // tokens staged at once
template <bool FUSED, int NR>
__global__ __launch_bounds__(256) void lay_delta_seq_kernel(LDeltaArgs a, int max_n) {
    constexpr int TB = lq_batch(FUSED, NR), ROWS = NR * LQ_GRP;
    __shared__ __attribute__((aligned(16))) f32x4 qkg[TB][ROWS];       // {q, k, g, -} per key row; rows past d are zero
    __shared__ float vs[TB][LQ_COLS], bs[TB], part[2][LQ_GRP][LQ_COLS][2], kqs[2][LQ_GRP], red[4];
    const LaySegDev sg = a.segs[blockIdx.x];
    if (sg.n > max_n) return;              // the chunk-parallel form takes this portion
    const int d = a.d, e = a.e, h = blockIdx.y, kh = h / (a.H / a.G), j0 = blockIdx.z * LQ_COLS;
    const int C = 2 * a.G * d + a.H * e;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, j = tid & (LQ_COLS - 1), rg = tid / LQ_COLS;
    const int col = j0 + j;
    const bool ok = col < e;
    float* st = a.state_pool + (size_t)sg.slot * a.slot_stride + a.st_off + (size_t)h * d * e + min(col, e - 1);
    float S[NR];
#pragma unroll
    for (int i = 0; i < NR; ++i) { const int row = rg + LQ_GRP * i; S[i] = row < d ? st[(size_t)row * e] : 0.f; }
    const float an = a.a_neg[h];
    for (int t0 = 0; t0 < sg.n; t0 += TB) {
        const int nt = min(TB, sg.n - t0);
        if (!FUSED) __syncthreads();       // the previous batch is consumed
        if (FUSED) {
            // the head's query (waves 0, 1) and key channels (waves 2, 3), a thread's channels in registers until their length is known
            const float* tail = a.conv_pool + (size_t)sg.slot * a.conv_stride + a.cv_off;
            const float* x = a.proj + (size_t)sg.row0 * a.ldp + a.q_off;
            auto conv = [&](int c) {
                float acc = 0.f;
                for (int k0 = 0; k0 < a.taps; k0 += 4) {             // four taps' loads in flight
                    float w[4], v[4];
#pragma unroll
                    for (int k = 0; k < 4; ++k) {
                        const int kk = min(k0 + k, a.taps - 1);
                        w[k] = a.conv_w[(size_t)c * a.taps + kk];
                        const float* p = kk < a.taps - 1 ? tail + (size_t)kk * C : x;
                        v[k] = p[c];
                    }
#pragma unroll
                    for (int k = 0; k < 4; ++k) if (k0 + k < a.taps) acc = fmaf(w[k], v[k], acc);
                }
                return dl_silu(acc);
            };
            constexpr int PT = (ROWS + 127) / 128;
            const int i0 = (wave & 1) * 64 + lane, base = (wave < 2 ? 0 : a.G * d) + kh * d;
            float y[PT], ss = 0.f;
#pragma unroll
            for (int p = 0; p < PT; ++p) {
                y[p] = i0 + 128 * p < d ? conv(base + i0 + 128 * p) : 0.f;
                ss = fmaf(y[p], y[p], ss);
            }
            ss = wave_sum(ss);
            if (lane == 0) red[wave] = ss;
            if (tid < LQ_COLS) vs[0][tid] = j0 + tid < e ? conv(2 * a.G * d + h * e + j0 + tid) : 0.f;
            if (tid == 64) bs[0] = dl_sigmoid(a.proj[(size_t)sg.row0 * a.ldp + a.b_off + h]);
            float gh = 0.f;
            if (!a.channel) gh = expf(an * dl_softplus(a.proj[(size_t)sg.row0 * a.ldp + a.a_off + h] + a.dt_bias[h]));
            for (int i = tid; i < ROWS; i += 256)
                qkg[0][i][2] = i < d ? (a.channel ? expf(an * dl_softplus(a.ldec[((size_t)sg.row0 * a.H + h) * d + i])) : gh) : 0.f;
            __syncthreads();
            const float f = wave < 2 ? 1.f / (sqrtf(red[0] + red[1] + UNIT_EPS) * sqrtf((float)d)) : 1.f / sqrtf(red[2] + red[3] + UNIT_EPS);
#pragma unroll
            for (int p = 0; p < PT; ++p)
                if (i0 + 128 * p < ROWS) qkg[0][i0 + 128 * p][wave < 2 ? 0 : 1] = y[p] * f;
        } else {
            for (int idx = tid; idx < nt * ROWS; idx += 256) {
                const int t = idx / ROWS, i = idx % ROWS;
                const size_t row = (size_t)(sg.row0 + t0 + t);
                f32x4 v = {0.f, 0.f, 0.f, 0.f};
                if (i < d) {
                    v[0] = a.xb[row * C + kh * d + i];
                    v[1] = a.xb[row * C + (a.G + kh) * d + i];
                    v[2] = expf(a.channel ? an * dl_softplus(a.ldec[(row * a.H + h) * d + i]) : a.ldec[row * a.H + h]);
                }
                qkg[t][i] = v;
            }
            for (int idx = tid; idx < nt * LQ_COLS; idx += 256) {
                const int t = idx / LQ_COLS, c = j0 + idx % LQ_COLS;
                vs[t][idx % LQ_COLS] = c < e ? a.xb[(size_t)(sg.row0 + t0 + t) * C + 2 * a.G * d + h * e + c] : 0.f;
            }
            for (int t = tid; t < nt; t += 256) bs[t] = a.beta[(size_t)(sg.row0 + t0 + t) * a.H + h];
        }
        __syncthreads();
        for (int t = 0; t < nt; ++t) {
            float p = 0.f, r = 0.f, kq = 0.f, k[NR];
#pragma unroll
            for (int i = 0; i < NR; ++i) {
                const f32x4 c = qkg[t][rg + LQ_GRP * i];
                S[i] *= c[2];
                k[i] = c[1];
                p = fmaf(S[i], c[1], p);
                r = fmaf(S[i], c[0], r);
                kq = fmaf(c[1], c[0], kq);
            }
            part[t & 1][rg][j][0] = p;
            part[t & 1][rg][j][1] = r;
            if (j == 0) kqs[t & 1][rg] = kq;
            __syncthreads();
            p = r = kq = 0.f;
#pragma unroll
            for (int x = 0; x < LQ_GRP; ++x) { p += part[t & 1][x][j][0]; r += part[t & 1][x][j][1]; kq += kqs[t & 1][x]; }
            const float u = bs[t] * (vs[t][j] - p);
#pragma unroll
            for (int i = 0; i < NR; ++i) S[i] = fmaf(k[i], u, S[i]);
            if (rg == 0 && ok) a.o_raw[(size_t)(sg.row0 + t0 + t) * a.H * e + (size_t)h * e + col] = fmaf(kq, u, r);
        }
    }
    if (ok) {
#pragma unroll
        for (int i = 0; i < NR; ++i) { const int row = rg + LQ_GRP * i; if (row < d) st[(size_t)row * e] = S[i]; }
    }
}

// head norm and output gate of the rows that went token by token, a wave per (row, head); TAIL (decode steps): blocks past the heads shift
// the convolution's tail
template <bool TAIL>
__global__ __launch_bounds__(256) void lay_delta_out_kernel(LDeltaArgs a, int max_n, int head_blocks) {
    const int r = blockIdx.x, lane = threadIdx.x & 63;
    const LaySegDev sg = a.segs[a.rowseg[r]];
    if (sg.n > max_n) return;
    if (TAIL && (int)blockIdx.y >= head_blocks) {
        const int C = 2 * a.G * a.d + a.H * a.e, c = ((int)blockIdx.y - head_blocks) * 256 + threadIdx.x;
        if (c >= C || a.taps < 2) return;
        float* tail = a.conv_pool + (size_t)sg.slot * a.conv_stride + a.cv_off;
        for (int k = 0; k + 2 < a.taps; ++k) tail[(size_t)k * C + c] = tail[(size_t)(k + 1) * C + c];
        tail[(size_t)(a.taps - 2) * C + c] = a.proj[(size_t)r * a.ldp + a.q_off + c];
        return;
    }
    const int h = blockIdx.y * 4 + (threadIdx.x >> 6), e = a.e;
    if (h >= a.H) return;
    const float* o = a.o_raw + ((size_t)r * a.H + h) * e;
    float ss = 0.f;
    for (int c = lane; c < e; c += 64) ss = fmaf(o[c], o[c], ss);
    const float rs = 1.f / sqrtf(wave_sum(ss) / (float)e + a.eps);
    for (int c = lane; c < e; c += 64)
        a.out[((size_t)r * a.H + h) * e + c] = o[c] * rs * a.norm_w[c] * dl_gate(a.gate[(size_t)r * a.ldg + (size_t)h * e + c], a.gate_act);
}

// ------------------------------------------------------------------------------------------------------------------
// Long portions, parallel over chunks of C = 64 tokens.  b_t: sum of ln g up to and including token t of the chunk (per key channel, or one
// number), S0 the state in front of the chunk:
//   (I + A) U = beta V - (beta e^b K) S0,   A[t][s] = beta_t sum_i k_t[i] k_s[i] e^(b_t[i] - b_s[i])  (s < t)
//   o_t = (e^b q)_t S0 + sum_(s <= t) P[t][s] u_s,   P[t][s] = sum_i q_t[i] k_s[i] e^(b_t[i] - b_s[i])
//   S_C = diag(e^(b_C)) S0 + (e^(b_C - b) K)^T U
// With W = (I + A)^-1 (beta e^b K), U0 = (I + A)^-1 (beta V), Kd = e^(b_C - b) K, Qd = e^b Q, the state drops out of all but two products:
//   S_C = M S0 + B,   M = diag(e^(b_C)) - Kd^T W,   B = Kd^T U0
//   O   = R S0 + Y0,  R = Qd - P W,                 Y0 = P U0
// chunk_prep (chunk, head, value slice): M, B, R, Y0;  chunk_scan (sequence, head, 16 value columns): the states S0 of all chunks, the only
// sequential part, one product per chunk;  chunk_out (chunk, head): O with the head norm and the output gate.
// Every exponent is a difference <= 0: tiles of A and P off the diagonal take the last position in front of the row tile as reference
// (e^(b_t - ref) e^(ref - b_s)), tiles on it form each pair's own.  So that strong decays earlier in a chunk do not cost the later small
// differences their digits, the head form keeps b in 64 bits; the channel form keeps the sums of each tile of 16 tokens by themselves and
// stops ln g at LN_FLOOR, where everything older is far below the rounding of what is written next.
// Scratch per (chunk, head), DP = 64 or 128 >= d, EP = e rounded up to 16: M [DP][DP] | B, then S0, transposed [EP][DP] | R [64][DP] | Y0 [64][EP]
// ------------------------------------------------------------------------------------------------------------------
constexpr int DC = LAY_DELTA_CHUNK, DCP = DC + 4, DV = 128;
constexpr float LN_FLOOR = -30.f;
static int ld_dp(int d) { return d <= 64 ? 64 : 128; }
__host__ __device__ static inline int ld_ep(int e) { return (e + 15) / 16 * 16; }
__host__ __device__ static inline size_t ld_floats(int dp, int e) { return (size_t)dp * dp + (size_t)ld_ep(e) * dp + (size_t)DC * dp + (size_t)DC * ld_ep(e); }
bool lay_delta_chunk_fits(int d, int e) { return d > 0 && e > 0 && d <= 128 && e <= 256; }
size_t lay_delta_chunk_floats(int d, int e) { return ld_floats(ld_dp(d), e); }

static size_t lay_delta_prep_lds(int DP) { return (size_t)(3 * DC * (DP + 4) + 2 * DC * DCP + 4 * 16 * 20 + 3 * DC + 4 * DP) * sizeof(float); }
template <bool CH, int DP>
__global__ __launch_bounds__(512) void lay_delta_chunk_prep_kernel(LDeltaArgs a) {
    extern __shared__ __attribute__((aligned(16))) float sm[];
    constexpr int KP = DP + 4, ND = DP / 16;
    float (*Ks)[KP] = (float (*)[KP])sm;                       // K, then beta e^b K
    float (*Qs)[KP] = (float (*)[KP])(sm + DC * KP);           // Q, then e^b Q
    float (*Bs)[KP] = (float (*)[KP])(sm + 2 * DC * KP);       // channel form: b from the start of the token's tile; then Kd
    float (*Am)[DCP] = (float (*)[DCP])(sm + 3 * DC * KP);     // -A
    float (*Pm)[DCP] = (float (*)[DCP])(sm + 3 * DC * KP + DC * DCP);
    float (*Ti)[16][20] = (float (*)[16][20])(sm + 3 * DC * KP + 2 * DC * DCP);      // inverses of the diagonal tiles of I + A
    double* lg = (double*)(sm + 3 * DC * KP + 2 * DC * DCP + 4 * 16 * 20);           // head form: b
    float* bt = (float*)(lg + DC);                             // beta
    float (*tot)[DP] = (float (*)[DP])(bt + DC);               // channel form: the tiles' sums
    const int2 chk = a.chunks[blockIdx.x];
    const LaySegDev sg = a.segs[chk.x];
    const int n = min(DC, sg.n - chk.y), row0 = sg.row0 + chk.y;
    const int d = a.d, e = a.e, h = blockIdx.y, kh = h / (a.H / a.G), v0 = blockIdx.z * DV;
    const int C = 2 * a.G * d + a.H * e;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r = lane & 15, kq = lane >> 4;
    const float an = a.a_neg[h];
    for (int idx = tid; idx < DC * DP; idx += 512) {
        const int t = idx / DP, i = idx % DP;
        const bool in = t < n && i < d;
        const float* x = a.xb + (size_t)(row0 + (in ? t : 0)) * C + kh * d + (in ? i : 0);
        Qs[t][i] = in ? x[0] : 0.f;
        Ks[t][i] = in ? x[a.G * d] : 0.f;
        if (CH) Bs[t][i] = in ? fmaxf(an * dl_softplus(a.ldec[((size_t)(row0 + t) * a.H + h) * d + i]), LN_FLOOR) : 0.f;
    }
    for (int idx = tid; idx < 2 * DC * DCP; idx += 512) (&Am[0][0])[idx] = 0.f;
    if (wave == 0) {
        bt[lane] = lane < n ? a.beta[(size_t)(row0 + lane) * a.H + h] : 0.f;
        if (!CH) {
            double g = lane < n ? (double)a.ldec[(size_t)(row0 + lane) * a.H + h] : 0.0;
#pragma unroll
            for (int s = 1; s < 64; s <<= 1) { const double o = __shfl_up(g, s); if (lane >= s) g += o; }
            lg[lane] = g;
        }
    }
    __syncthreads();
    if (CH) {                              // running sums down the tokens of each tile
        const int i = tid % DP, q4 = tid / DP;
        if (q4 < 4) {
            float run = 0.f;
#pragma unroll
            for (int t = 0; t < 16; ++t) { run += Bs[16 * q4 + t][i]; Bs[16 * q4 + t][i] = run; }
            tot[q4][i] = run;
        }
        __syncthreads();
    }
    // ---- A and P, lower tiles: six off the diagonal, then the four on it (channel form: below)
    for (int u = wave; u < (CH ? 12 : 20); u += 8) {
        const int tile = u >> 1, which = u & 1;
        int tr, tc;
        if (tile >= 6) tr = tc = tile - 6;
        else if (tile == 0) { tr = 1; tc = 0; }
        else if (tile < 3) { tr = 2; tc = tile - 1; }
        else { tr = 3; tc = tile - 3; }
        f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int jj = 0; jj < ND; ++jj) {
            f32x4 av = *(const f32x4*)&(which ? Qs : Ks)[16 * tr + r][16 * jj + 4 * kq];
            f32x4 bv = *(const f32x4*)&Ks[16 * tc + r][16 * jj + 4 * kq];
            if (CH) {
                const f32x4 ba = *(const f32x4*)&Bs[16 * tr + r][16 * jj + 4 * kq];
                f32x4 bb = *(const f32x4*)&tot[tc][16 * jj + 4 * kq] - *(const f32x4*)&Bs[16 * tc + r][16 * jj + 4 * kq];
                for (int m = tc + 1; m < tr; ++m) bb += *(const f32x4*)&tot[m][16 * jj + 4 * kq];
#pragma unroll
                for (int i = 0; i < 4; ++i) { av[i] *= __expf(ba[i]); bv[i] *= __expf(bb[i]); }
            }
            acc = dl_mfma(av, bv, acc);
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int t = 16 * tr + 4 * kq + i, s = 16 * tc + r;
            const float f = CH ? 1.f : (s <= t ? expf((float)(lg[t] - lg[s])) : 0.f);
            if (which) Pm[t][s] = f * acc[i];
            else Am[t][s] = s < t ? -bt[t] * f * acc[i] : 0.f;
        }
    }
    if (CH) {
        if (tid < 480) {                   // 4 tiles x 120 pairs s < t
            const int tile = tid / 120, p = tid % 120;
            int tl = (int)((1.f + sqrtf(1.f + 8.f * (float)p)) * 0.5f);
            while (tl * (tl - 1) / 2 > p) --tl;
            while ((tl + 1) * tl / 2 <= p) ++tl;
            const int t = 16 * tile + tl, s = 16 * tile + (p - tl * (tl - 1) / 2);
            float sa = 0.f, sp = 0.f;
            for (int i0 = 0; i0 < d; i0 += 4) {
                const f32x4 kt = *(const f32x4*)&Ks[t][i0], qt = *(const f32x4*)&Qs[t][i0], kk = *(const f32x4*)&Ks[s][i0];
                const f32x4 b1 = *(const f32x4*)&Bs[t][i0], b2 = *(const f32x4*)&Bs[s][i0];
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const float x = kk[i] * __expf(b1[i] - b2[i]);
                    sa = fmaf(kt[i], x, sa);
                    sp = fmaf(qt[i], x, sp);
                }
            }
            Am[t][s] = -bt[t] * sa;
            Pm[t][s] = sp;
        } else {
            for (int t = tid - 480; t < DC; t += 32) {
                float sp = 0.f;
                for (int i = 0; i < d; ++i) sp = fmaf(Qs[t][i], Ks[t][i], sp);
                Pm[t][t] = sp;
            }
        }
    }
    __syncthreads();
    // ---- K, Q -> beta e^b K, e^b Q, Kd (a thread touches its own elements only); inverses of the diagonal tiles by the last wave
    for (int idx = tid; idx < DC * DP; idx += 512) {
        const int t = idx / DP, i = idx % DP;
        const float k = Ks[t][i];
        float b, rest;                     // ln of the decay from the chunk's start to token t, and from there to its end
        if (CH) {
            b = Bs[t][i]; rest = tot[t >> 4][i] - b;
            for (int m = 0; m < t >> 4; ++m) b += tot[m][i];
            for (int m = (t >> 4) + 1; m < 4; ++m) rest += tot[m][i];
        } else { b = (float)lg[t]; rest = (float)(lg[DC - 1] - lg[t]); }
        const float eb = expf(b);
        Bs[t][i] = k * expf(rest);
        Ks[t][i] = bt[t] * k * eb;
        Qs[t][i] *= eb;
    }
    if (wave == 7) {
        const int tile = kq, c = r;
        float x[16];
#pragma unroll
        for (int t = 0; t < 16; ++t) {
            float v = t == c ? 1.f : 0.f;
#pragma unroll
            for (int s4 = 0; s4 < t; s4 += 4) {
                const f32x4 av = *(const f32x4*)&Am[16 * tile + t][16 * tile + s4];      // zero from the diagonal on
#pragma unroll
                for (int i = 0; i < 4; ++i) if (s4 + i < t) v = fmaf(av[i], x[s4 + i], v);
            }
            x[t] = v;
            Ti[tile][t][c] = v;
        }
    }
    __syncthreads();
    // ---- column tiles [W | U0]: a wave owns whole columns, so nothing below waits for another wave
    float* base = a.scratch + ((size_t)blockIdx.x * a.H + h) * ld_floats(DP, e);
    const int EP = ld_ep(e);
    float *Mg = base, *Bg = Mg + DP * DP, *Rg = Bg + (size_t)EP * DP, *Yg = Rg + DC * DP;
    const int nW = blockIdx.z == 0 ? ND : 0, nV = (min(DV, e - v0) + 15) / 16;
#pragma unroll 1
    for (int ct = wave; ct < nW + nV; ct += 8) {
        asm volatile("" ::: "memory");     // the operands in LDS are read per column tile: kept in registers across tiles they would spill
        const bool isw = ct < nW;
        const int c = 16 * (isw ? ct : ct - nW) + r, vc = v0 + c;      // this lane's column (of W, of the value slice)
        f32x4 X[4];
#pragma unroll
        for (int I = 0; I < 4; ++I)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int t = 16 * I + 4 * kq + i;
                if (isw) X[I][i] = Ks[t][c];
                else {
                    const bool in = t < n && vc < e;
                    const float v = a.xb[(size_t)(row0 + (in ? t : 0)) * C + 2 * a.G * d + (size_t)h * e + (in ? vc : 0)];
                    X[I][i] = in ? bt[t] * v : 0.f;
                }
            }
#pragma unroll
        for (int I = 0; I < 4; ++I) {
            f32x4 acc = X[I];
#pragma unroll
            for (int L = 0; L < I; ++L) acc = dl_mfma(*(const f32x4*)&Am[16 * I + r][16 * L + 4 * kq], X[L], acc);
            X[I] = dl_mfma(*(const f32x4*)&Ti[I][r][4 * kq], acc, (f32x4){0.f, 0.f, 0.f, 0.f});
        }
        if (isw) {
#pragma unroll
            for (int I = 0; I < 4; ++I) X[I] = -X[I];
        }
#pragma unroll
        for (int I = 0; I < 4; ++I) {
            f32x4 acc = {0.f, 0.f, 0.f, 0.f};
            if (isw) {
#pragma unroll
                for (int i = 0; i < 4; ++i) acc[i] = Qs[16 * I + 4 * kq + i][c];
            }
#pragma unroll
            for (int L = 0; L <= I; ++L) acc = dl_mfma(*(const f32x4*)&Pm[16 * I + r][16 * L + 4 * kq], X[L], acc);
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int t = 16 * I + 4 * kq + i;
                if (isw) Rg[t * DP + c] = acc[i];
                else Yg[(size_t)t * EP + vc] = acc[i];
            }
        }
#pragma unroll
        for (int m = 0; m < ND; ++m) {
            f32x4 acc = {0.f, 0.f, 0.f, 0.f};
            if (isw) {
#pragma unroll
                for (int i = 0; i < 4; ++i) if (16 * m + 4 * kq + i == c) acc[i] = expf(CH ? (tot[0][c] + tot[1][c]) + (tot[2][c] + tot[3][c]) : (float)lg[DC - 1]);
            }
#pragma unroll
            for (int L = 0; L < 4; ++L) {
                f32x4 av;
#pragma unroll
                for (int i = 0; i < 4; ++i) av[i] = Bs[16 * L + 4 * kq + i][16 * m + r];
                acc = dl_mfma(av, X[L], acc);
            }
            if (isw) {
#pragma unroll
                for (int i = 0; i < 4; ++i) Mg[(16 * m + 4 * kq + i) * DP + c] = acc[i];
            } else *(f32x4*)(Bg + (size_t)vc * DP + 16 * m + 4 * kq) = acc;
        }
    }
}

// the states in front of the chunks, in place of B: S <- M S + B.  Wave w owns DP / 4 state rows of 16 value columns; the columns meet in LDS.
// M and B of a chunk are requested two chunks ahead into two register sets.
template <int DP>
__global__ __launch_bounds__(256) void lay_delta_chunk_scan_kernel(LDeltaArgs a) {
    constexpr int KP = DP + 4, ND = DP / 16, RT = DP / 64;
    __shared__ __attribute__((aligned(16))) float St[2][16][KP];
    const LaySegDev sg = a.segs[blockIdx.x];
    if (sg.n <= LAY_DELTA_SEQ) return;
    const int d = a.d, e = a.e, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r = lane & 15, kq = lane >> 4;
    const int c0 = blockIdx.z * 16, nch = (sg.n + DC - 1) / DC;
    const size_t fl = ld_floats(DP, e);
    float* base = a.scratch + ((size_t)sg.pad1 * a.H + h) * fl;
    const size_t step = (size_t)a.H * fl;
    float* st = a.state_pool + (size_t)sg.slot * a.slot_stride + a.st_off + (size_t)h * d * e;
    for (int idx = tid; idx < 16 * DP; idx += 256) {
        const int i = idx >> 4, c = idx & 15;
        St[0][c][i] = i < d && c0 + c < e ? st[(size_t)i * e + c0 + c] : 0.f;
    }
    f32x4 mA[RT][ND], mB[RT][ND], bA[RT], bB[RT], S[RT];
    auto fetch = [&](int c, f32x4 (&m)[RT][ND], f32x4 (&b)[RT]) __attribute__((always_inline)) {
        const float* p = base + (size_t)min(c, nch - 1) * step;
#pragma unroll
        for (int x = 0; x < RT; ++x) {
            const int row = 16 * (RT * wave + x);
#pragma unroll
            for (int jj = 0; jj < ND; ++jj) m[x][jj] = *(const f32x4*)(p + (row + r) * DP + 16 * jj + 4 * kq);
            b[x] = *(const f32x4*)(p + DP * DP + (size_t)(c0 + r) * DP + row + 4 * kq);
        }
    };
    fetch(0, mA, bA);
    fetch(1, mB, bB);
    __syncthreads();
#pragma unroll
    for (int x = 0; x < RT; ++x) S[x] = *(const f32x4*)&St[0][r][16 * (RT * wave + x) + 4 * kq];
    auto chunk = [&](int c, f32x4 (&m)[RT][ND], f32x4 (&b)[RT]) __attribute__((always_inline)) {
        float* p = base + (size_t)c * step + DP * DP + (size_t)(c0 + r) * DP;
        f32x4 acc[RT];
#pragma unroll
        for (int x = 0; x < RT; ++x) {
            acc[x] = b[x];
            *(f32x4*)(p + 16 * (RT * wave + x) + 4 * kq) = S[x];
        }
#pragma unroll
        for (int jj = 0; jj < ND; ++jj) {
            const f32x4 sv = *(const f32x4*)&St[c & 1][r][16 * jj + 4 * kq];
#pragma unroll
            for (int x = 0; x < RT; ++x) acc[x] = dl_mfma(m[x][jj], sv, acc[x]);
        }
        if (c + 2 < nch) fetch(c + 2, m, b);
#pragma unroll
        for (int x = 0; x < RT; ++x) {
            S[x] = acc[x];
            *(f32x4*)&St[(c & 1) ^ 1][r][16 * (RT * wave + x) + 4 * kq] = acc[x];
        }
        dl_lds_barrier();
    };
    for (int c = 0; c < nch; c += 2) {
        chunk(c, mA, bA);
        if (c + 1 < nch) chunk(c + 1, mB, bB);
    }
    if (c0 + r < e) {
#pragma unroll
        for (int x = 0; x < RT; ++x)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int row = 16 * (RT * wave + x) + 4 * kq + i;
                if (row < d) st[(size_t)row * e + c0 + r] = S[x][i];
            }
    }
}

// outputs of a chunk, a wave per 16 tokens: R S0 + Y0, head norm, output gate.  NE: value size in units of 16 the registers are laid out for
template <int DP, int NE>
__global__ __launch_bounds__(256) void lay_delta_chunk_out_kernel(LDeltaArgs a) {
    constexpr int ND = DP / 16;
    const int2 chk = a.chunks[blockIdx.x];
    const LaySegDev sg = a.segs[chk.x];
    const int n = min(DC, sg.n - chk.y), row0 = sg.row0 + chk.y;
    const int e = a.e, EP = ld_ep(e), ne = EP / 16, h = blockIdx.y;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r = lane & 15, kq = lane >> 4;
    if (16 * wave >= n) return;
    const float* base = a.scratch + ((size_t)blockIdx.x * a.H + h) * ld_floats(DP, e);
    const float *Sg = base + DP * DP, *Rg = Sg + (size_t)EP * DP, *Yg = Rg + DC * DP;
    f32x4 R[ND], acc[NE];
#pragma unroll
    for (int jj = 0; jj < ND; ++jj) R[jj] = *(const f32x4*)(Rg + (16 * wave + r) * DP + 16 * jj + 4 * kq);
    f32x4 ss = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int m = 0; m < NE; ++m) {
        if (m < ne) {
            f32x4 c;
#pragma unroll
            for (int i = 0; i < 4; ++i) c[i] = Yg[(size_t)(16 * wave + 4 * kq + i) * EP + 16 * m + r];
#pragma unroll
            for (int jj = 0; jj < ND; ++jj) c = dl_mfma(R[jj], *(const f32x4*)(Sg + (size_t)(16 * m + r) * DP + 16 * jj + 4 * kq), c);
            acc[m] = c;
            ss += c * c;                   // (columns past e are zero)
        }
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) ss[i] = 1.f / sqrtf(row16_sum(ss[i]) / (float)e + a.eps);
#pragma unroll
    for (int m = 0; m < NE; ++m) {
        const int col = 16 * m + r;
        if (m < ne && col < e) {
            const float w = a.norm_w[col];
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int t = 16 * wave + 4 * kq + i;
                if (t < n)
                    a.out[((size_t)(row0 + t) * a.H + h) * e + col] = acc[m][i] * ss[i] * w * dl_gate(a.gate[(size_t)(row0 + t) * a.ldg + (size_t)h * e + col], a.gate_act);
            }
        }
    }
}

// ------------------------------------------------------------------------------------------------------------------
// launches
// ------------------------------------------------------------------------------------------------------------------
template <bool FUSED, int NR>
static void lay_delta_seq_go(const LDeltaArgs& a, int max_n, hipStream_t s) {
    hipLaunchKernelGGL((lay_delta_seq_kernel<FUSED, NR>), dim3((unsigned)a.nseg, (unsigned)a.H, (unsigned)((a.e + LQ_COLS - 1) / LQ_COLS)), dim3(256),
                       0, s, a, max_n);
}
template <bool FUSED>
static void lay_delta_seq(const LDeltaArgs& a, int max_n, hipStream_t s) {
    if (a.d <= 64) lay_delta_seq_go<FUSED, 8>(a, max_n, s);
    else if (a.d <= 128) lay_delta_seq_go<FUSED, 16>(a, max_n, s);
    else lay_delta_seq_go<FUSED, 32>(a, max_n, s);
}
template <int VPL>
static void lay_delta_prep(const LDeltaArgs& a, hipStream_t s) {
    const int units = 2 * a.G + (a.H * a.e + 64 * VPL - 1) / (64 * VPL) + 1;
    const dim3 grid((unsigned)((a.T + LP_ROWS - 1) / LP_ROWS), (unsigned)((units + 3) / 4));
    switch (a.taps) {
        case 2: hipLaunchKernelGGL((lay_delta_prep_kernel<VPL, 2>), grid, dim3(256), 0, s, a); break;
        case 3: hipLaunchKernelGGL((lay_delta_prep_kernel<VPL, 3>), grid, dim3(256), 0, s, a); break;
        case 4: hipLaunchKernelGGL((lay_delta_prep_kernel<VPL, 4>), grid, dim3(256), 0, s, a); break;
        default: hipLaunchKernelGGL((lay_delta_prep_kernel<VPL, 0>), grid, dim3(256), 0, s, a);
    }
}
template <bool CH, int DP>
static void lay_delta_chunked(const LDeltaArgs& a, hipStream_t s) {
    static bool raised = false;            // per instantiation
    const size_t lds = lay_delta_prep_lds(DP);
    if (!raised && lds > LD_LDS_PLAIN) {
        (void)hipFuncSetAttribute(reinterpret_cast<const void*>(&lay_delta_chunk_prep_kernel<CH, DP>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)LD_LDS_MAX);
        raised = true;
    }
    hipLaunchKernelGGL((lay_delta_chunk_prep_kernel<CH, DP>), dim3((unsigned)a.nchunks, (unsigned)a.H, (unsigned)((a.e + DV - 1) / DV)), dim3(512), lds, s, a);
    hipLaunchKernelGGL(lay_delta_chunk_scan_kernel<DP>, dim3((unsigned)a.nseg, (unsigned)a.H, (unsigned)(ld_ep(a.e) / 16)), dim3(256), 0, s, a);
    const dim3 go((unsigned)a.nchunks, (unsigned)a.H);
    if (a.e <= 128) hipLaunchKernelGGL((lay_delta_chunk_out_kernel<DP, 8>), go, dim3(256), 0, s, a);
    else hipLaunchKernelGGL((lay_delta_chunk_out_kernel<DP, 16>), go, dim3(256), 0, s, a);
}
void launch_lay_delta(const LDeltaArgs& a, hipStream_t s) {
    if (a.T <= 0 || a.nseg <= 0) return;
    const int head_blocks = (a.H + 3) / 4, C = 2 * a.G * a.d + a.H * a.e;
    if (a.all_single) {
        lay_delta_seq<true>(a, 1, s);
        hipLaunchKernelGGL(lay_delta_out_kernel<true>, dim3((unsigned)a.T, (unsigned)(head_blocks + (C + 255) / 256)), dim3(256), 0, s, a, 1, head_blocks);
        return;
    }
    if (a.d <= 64) lay_delta_prep<1>(a, s);
    else if (a.d <= 128) lay_delta_prep<2>(a, s);
    else lay_delta_prep<4>(a, s);
    LConvArgs c{};
    c.src = a.proj; c.lds = a.ldp; c.off = a.q_off; c.C = C; c.taps = a.taps; c.conv_pool = a.conv_pool; c.slot_stride = a.conv_stride; c.cv_off = a.cv_off;
    c.segs = a.segs; c.rowseg = a.rowseg;
    launch_lay_conv_tail(c, a.nseg, s);
    const bool chunked = a.chunks && a.nchunks > 0 && a.scratch && lay_delta_chunk_fits(a.d, a.e);
    const int max_n = chunked ? LAY_DELTA_SEQ : 0x7fffffff;
    if (a.min_n <= max_n) {
        lay_delta_seq<false>(a, max_n, s);
        hipLaunchKernelGGL(lay_delta_out_kernel<false>, dim3((unsigned)a.T, (unsigned)head_blocks), dim3(256), 0, s, a, max_n, head_blocks);
    }
    if (!chunked) return;
    if (a.channel) { if (a.d <= 64) lay_delta_chunked<true, 64>(a, s); else lay_delta_chunked<true, 128>(a, s); }
    else { if (a.d <= 64) lay_delta_chunked<false, 64>(a, s); else lay_delta_chunked<false, 128>(a, s); }
}

}  // namespace cm
